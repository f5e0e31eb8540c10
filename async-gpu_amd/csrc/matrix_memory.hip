// Matrix memory (matrix_memory.h).
//
// One token: a state column per 16 lanes, every workgroup a slice of columns of one head; each computes the normaliser for
// itself and the first one keeps it.
//
// Many tokens, in chunks of 64.  With F the running sum of the log forget gates of a chunk and a_s = i_s - F_s, the weight of
// token s in the state after token t is exp(a_s - M_t) with M_t = max(m, max_{s <= t} a_s), m the running maximum in front of
// the chunk, and m_t = F_t + M_t.  All of it is at most 1, however strong the gates.  F, a and M are kept in double precision:
// their differences are small where a weight matters, themselves they are not.  Four launches:
//   scores  P[t][s] = (q_t . k_s) exp(a_s - A_t), A_t = max_{s <= t} a_s, its row sums, the weights exp(a_s - A_last)
//   increments, scan  S and n in front of every chunk: S <- exp(m - M) S + exp(A - M) sum_s weight_s k_s v_s^T
//   outputs o_t = (exp(m - M_t) S^T q_t + exp(A_t - M_t) P v) / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)
// The products run on the fp32 matrix cores (v_mfma_f32_32x32x2_f32).
#include "matrix_memory.h"

namespace {

typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr int C = kMemoryChunk;
constexpr int kMaxDim = 256;
constexpr double kNever = -1.0e300;

__device__ __forceinline__ float capped(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }

// Where the pieces of one (sequence, head, chunk) lie in the scratch.
struct Scratch {
    double *total;  // [chunk] F of the chunk's last token, A of it
    double *fa;     // [chunk][2][C]: F_t, A_t
    float *weight;  // [chunk][C]
    float *sums;    // [chunk][C]
    float *p;       // [chunk][C][C]
    float *s;       // [chunk][vdimp][dimp]
    float *n;       // [chunk and behind the last][dimp]
    double *m;      // [chunk and behind the last]
};
__host__ __device__ inline size_t scratch_per_head(int chunks, int dimp, int vdimp) {  // in floats
    return (size_t)chunks * (4 + 4 * C + C + C + C * C + (size_t)vdimp * dimp) + (size_t)(chunks + 1) * (dimp + 4);
}
__host__ __device__ inline Scratch scratch_of(void *base, size_t bh, int chunks, int dimp, int vdimp) {
    Scratch x;
    float *p = (float *)base + bh * scratch_per_head(chunks, dimp, vdimp);
    x.total = (double *)p;
    x.fa = (double *)(p += (size_t)chunks * 4);
    x.weight = p += (size_t)chunks * 4 * C;
    x.sums = p += (size_t)chunks * C;
    x.p = p += (size_t)chunks * C;
    x.s = p += (size_t)chunks * C * C;
    x.n = p += (size_t)chunks * vdimp * dimp;
    x.m = (double *)(p + (size_t)(chunks + 1) * dimp);
    return x;
}

// grid (column slices of 16, heads, batch): NF float4 of a state column per lane.
template <int NF>
__global__ __launch_bounds__(256) void memory_step_kernel(MemoryArgs a, int dimp, int vdimp) {
    const MemoryShape &s = a.s;
    const int t = threadIdx.x, kl = t & 15, h = blockIdx.y, b = blockIdx.z, j = blockIdx.x * 16 + (t >> 4), pos = *a.pos_dev;
    const size_t bh = (size_t)b * s.heads + h;
    float *state = a.state + (bh * vdimp + j) * dimp, *norm = a.norm + bh * 2 * (dimp + 4);
    const float *old = norm + (pos & 1) * (dimp + 4);
    float *next = norm + (1 - (pos & 1)) * (dimp + 4);
    const float *q = a.q + (size_t)b * a.ld + h * dimp, *k = a.k + (size_t)b * a.ld + h * dimp;
    float4 S[NF], Q[NF], K[NF], N[NF];
#pragma unroll
    for (int f = 0; f < NF; ++f) {
        const int d = min(kl * 4 + 64 * f, dimp - 4);
        S[f] = *(const float4 *)(state + d);
        Q[f] = *(const float4 *)(q + d);
        K[f] = *(const float4 *)(k + d);
        N[f] = *(const float4 *)(old + d);
    }
    const float v = a.v[(size_t)b * a.ld + h * vdimp + j], m = old[dimp];
    const float li = capped(a.i[(size_t)b * a.ld + h], s.cap), lf = log_sigmoid(capped(a.f[(size_t)b * a.ld + h], s.cap));
    const float m_new = fmaxf(lf + m, li), keep = expf(lf + m - m_new), take = expf(li - m_new), tv = take * v;
    float o = 0.0f, nq = 0.0f;
#pragma unroll
    for (int f = 0; f < NF; ++f) {
        const int d = kl * 4 + 64 * f;
        if (d >= dimp) continue;
        float4 &x = S[f], &n = N[f];
        x.x = fmaf(K[f].x, tv, keep * x.x);
        x.y = fmaf(K[f].y, tv, keep * x.y);
        x.z = fmaf(K[f].z, tv, keep * x.z);
        x.w = fmaf(K[f].w, tv, keep * x.w);
        n.x = fmaf(K[f].x, take, keep * n.x);
        n.y = fmaf(K[f].y, take, keep * n.y);
        n.z = fmaf(K[f].z, take, keep * n.z);
        n.w = fmaf(K[f].w, take, keep * n.w);
        o += x.x * Q[f].x + x.y * Q[f].y + x.z * Q[f].z + x.w * Q[f].w;
        nq += n.x * Q[f].x + n.y * Q[f].y + n.z * Q[f].z + n.w * Q[f].w;
        *(float4 *)(state + d) = x;
        if (blockIdx.x == 0 && t < 16) *(float4 *)(next + d) = n;
    }
    const float scale = 1.0f / sqrtf((float)s.dim);
    o = row16_sum(o) * scale;
    nq = row16_sum(nq) * scale;
    if (kl == 0) a.out[(size_t)b * a.ldo + h * vdimp + j] = o / (fmaxf(fabsf(nq), expf(-m_new)) + 1e-6f);
    if (blockIdx.x == 0 && t == 0) next[dimp] = m_new;
}

// acc += rows of sa [64][LD] (this wave's 32 from r0 on) times rows of sb (32 from c0 on), 32 k; the halves of a wave take
// k 0 .. 15 and 16 .. 31.
constexpr int LD = 36;
__device__ __forceinline__ f32x16 tile_product(const float *sa, const float *sb, int r0, int c0, int lane, f32x16 acc) {
    const float *ar = sa + (r0 + (lane & 31)) * LD + (lane >> 5) * 16, *br = sb + (c0 + (lane & 31)) * LD + (lane >> 5) * 16;
#pragma unroll
    for (int s = 0; s < 16; s += 4) {
        const float4 av = *(const float4 *)(ar + s), bv = *(const float4 *)(br + s);
        acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av.x, bv.x, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av.y, bv.y, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av.z, bv.z, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av.w, bv.w, acc, 0, 0, 0);
    }
    return acc;
}

// grid (chunks, heads, batch)
__global__ __launch_bounds__(256) void memory_scores_kernel(MemoryArgs a, int dimp, int vdimp) {
    __shared__ __align__(16) float sab[2 * C * LD];
    __shared__ double sa_[C], sA[C];
    __shared__ float tile[C][C + 1];
    const MemoryShape &s = a.s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave >> 1, wn = wave & 1;
    const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z, T = a.new_len, t0 = chunk * C, nt = min(C, T - t0);
    const size_t row0 = (size_t)b * T + t0;
    const Scratch x = scratch_of(a.scratch, (size_t)b * s.heads + h, gridDim.x, dimp, vdimp);
    if (wave == 0) {  // the gates of the chunk, a token per lane
        const size_t at = (row0 + min(lane, nt - 1)) * a.ld + h;
        double F = lane < nt ? (double)log_sigmoid(capped(a.f[at], s.cap)) : 0.0;
        const double li = lane < nt ? (double)capped(a.i[at], s.cap) : kNever;
#pragma unroll
        for (int o = 1; o < C; o <<= 1) {
            const double v = __shfl_up(F, o);
            F += lane >= o ? v : 0.0;
        }
        const double as = lane < nt ? li - F : kNever;
        double A = as;
#pragma unroll
        for (int o = 1; o < C; o <<= 1) {
            const double v = __shfl_up(A, o);
            A = lane >= o ? fmax(A, v) : A;
        }
        sa_[lane] = as;
        sA[lane] = A;
        const double last = __shfl(A, C - 1);
        x.fa[(size_t)chunk * 2 * C + lane] = F;
        x.fa[(size_t)chunk * 2 * C + C + lane] = A;
        x.weight[(size_t)chunk * C + lane] = lane < nt ? expf((float)(as - last)) : 0.0f;
        if (lane == C - 1) {
            x.total[2 * chunk] = F;
            x.total[2 * chunk + 1] = A;
        }
    }
    f32x16 acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.0f;
    const int row = tid >> 2, c8 = (tid & 3) * 8;
    const float *qp = a.q + (row0 + min(row, nt - 1)) * a.ld + h * dimp + c8, *kp = a.k + (row0 + min(row, nt - 1)) * a.ld + h * dimp + c8;
    float *sq = sab, *sk = sab + C * LD;
    for (int k0 = 0; k0 < dimp; k0 += 32) {
        const float4 q0 = *(const float4 *)(qp + k0), q1 = *(const float4 *)(qp + k0 + 4);
        const float4 k0v = *(const float4 *)(kp + k0), k1v = *(const float4 *)(kp + k0 + 4);
        __syncthreads();
        *(float4 *)(sq + row * LD + c8) = q0;
        *(float4 *)(sq + row * LD + c8 + 4) = q1;
        *(float4 *)(sk + row * LD + c8) = k0v;
        *(float4 *)(sk + row * LD + c8 + 4) = k1v;
        __syncthreads();
        if (wm >= wn) acc = tile_product(sq, sk, wm * 32, wn * 32, lane, acc);  // nothing above the diagonal
    }
    const float scale = 1.0f / sqrtf((float)s.dim);
    const int sc = wn * 32 + (lane & 31);
#pragma unroll
    for (int r = 0; r < 16; ++r) {
        const int t = wm * 32 + 8 * (r >> 2) + 4 * (lane >> 5) + (r & 3);
        tile[t][sc] = sc <= t && sc < nt ? acc[r] * scale * expf((float)(sa_[sc] - sA[t])) : 0.0f;
    }
    __syncthreads();
    {
        const int t = tid >> 2;
        float v = 0.0f;
        for (int i = tid & 3; i < C; i += 4) v += tile[t][i];
        v += dpp_move<0xb1, 0xf>(0.0f, v);
        v += dpp_move<0x4e, 0xf>(0.0f, v);
        if ((tid & 3) == 0) x.sums[(size_t)chunk * C + t] = v;
    }
    float *p = x.p + (size_t)chunk * C * C;
    for (int i = tid; i < C * C; i += 256) p[i] = tile[i / C][i % C];
}

// grid (tiles of 64 dimensions * chunks, tiles of 64 value dimensions, heads * batch), 2 x 2 waves: what the chunk adds to S and n,
// sum_s weight_s v_s k_s^T and sum_s weight_s k_s.
__global__ __launch_bounds__(256) void memory_increments_kernel(MemoryArgs a, int dimp, int vdimp, int chunks) {
    __shared__ __align__(16) float sk[C][64], sv[C][64];
    const MemoryShape &s = a.s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave >> 1, wn = wave & 1, lr = lane & 31, lh = lane >> 5;
    const int d0 = blockIdx.x / chunks * 64, chunk = blockIdx.x % chunks, j0 = blockIdx.y * 64, h = blockIdx.z % s.heads, b = blockIdx.z / s.heads;
    const int T = a.new_len, t0 = chunk * C, nt = min(C, T - t0);
    const size_t row0 = (size_t)b * T + t0;
    const Scratch x = scratch_of(a.scratch, (size_t)b * s.heads + h, chunks, dimp, vdimp);
    const int e = (tid & 15) * 4;
    float4 rk[4], rv[4];
    float rw[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int t = (tid >> 4) + 16 * i;
        const float *row = a.k + (row0 + min(t, nt - 1)) * a.ld;
        rk[i] = *(const float4 *)(row + h * dimp + min(d0 + e, dimp - 4));
        rv[i] = *(const float4 *)(a.v + (row0 + min(t, nt - 1)) * a.ld + h * vdimp + min(j0 + e, vdimp - 4));
        rw[i] = x.weight[(size_t)chunk * C + t];  // 0 behind the last token
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int t = (tid >> 4) + 16 * i;
        *(float4 *)&sk[t][e] = make_float4(rk[i].x * rw[i], rk[i].y * rw[i], rk[i].z * rw[i], rk[i].w * rw[i]);
        *(float4 *)&sv[t][e] = rv[i];
    }
    __syncthreads();
    f32x16 acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.0f;
#pragma unroll 8
    for (int t = 0; t < C; t += 2) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(sv[t + lh][32 * wm + lr], sk[t + lh][32 * wn + lr], acc, 0, 0, 0);
    const int d = d0 + 32 * wn + lr;
    if (d < dimp) {
        float *out = x.s + (size_t)chunk * vdimp * dimp + d;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int j = j0 + 32 * wm + 8 * (r >> 2) + 4 * lh + (r & 3);
            if (j < vdimp) out[(size_t)j * dimp] = acc[r];
        }
    }
    if (blockIdx.y == 0 && tid < 64 && d0 + tid < dimp) {
        float v = 0.0f;
#pragma unroll 16
        for (int t = 0; t < C; ++t) v += sk[t][tid];
        x.n[(size_t)chunk * dimp + d0 + tid] = v;
    }
}

// grid (groups of 1024 values of S and then n, heads * batch): the chunks one after the other; every increment gives way to the
// state in front of its chunk.
__global__ __launch_bounds__(256) void memory_scan_kernel(MemoryArgs a, int dimp, int vdimp, int chunks) {
    extern __shared__ double sm[];  // [chunks + 1] running maximum in front of every chunk, [chunks][2] totals; [chunks] float2 factors
    double *st = sm + chunks + 1;
    float2 *sf = (float2 *)(st + 2 * chunks);
    const int tid = threadIdx.x, pos = *a.pos_dev;
    const size_t bh = blockIdx.y;  // sequence * heads + head
    const Scratch x = scratch_of(a.scratch, bh, chunks, dimp, vdimp);
    const float *old = a.norm + (bh * 2 + (pos & 1)) * (dimp + 4);
    const int values = vdimp * dimp, at = (blockIdx.x * 256 + tid) * 4;
    const bool on = at < values + dimp, is_n = at >= values;
    float *buf = is_n ? x.n + min(at - values, dimp - 4) : x.s + at;
    const size_t step = is_n ? dimp : values;
    float4 S = *(const float4 *)(is_n ? old + min(at - values, dimp - 4) : a.state + bh * values + at);
    for (int i = tid; i < 2 * chunks; i += 256) st[i] = x.total[i];
    __syncthreads();
    if (tid == 0) {
        double m = (double)old[dimp];
        for (int c = 0; c < chunks; ++c) {
            sm[c] = m;
            m = st[2 * c] + fmax(m, st[2 * c + 1]);
        }
        sm[chunks] = m;
    }
    __syncthreads();
    for (int c = tid; c < chunks; c += 256) {
        const double M = fmax(sm[c], st[2 * c + 1]);
        sf[c] = make_float2(expf((float)(sm[c] - M)), expf((float)(st[2 * c + 1] - M)));
    }
    if (blockIdx.x == 0)
        for (int c = tid; c <= chunks; c += 256) x.m[c] = sm[c];
    __syncthreads();
    if (!on) return;
    constexpr int U = 8;
#pragma unroll 1
    for (int c0 = 0; c0 < chunks; c0 += U) {
        float4 u[U];
#pragma unroll
        for (int i = 0; i < U; ++i) u[i] = *(const float4 *)(buf + (size_t)min(c0 + i, chunks - 1) * step);
#pragma unroll
        for (int i = 0; i < U; ++i) {
            if (c0 + i >= chunks) break;
            const float2 f = sf[c0 + i];
            *(float4 *)(buf + (size_t)(c0 + i) * step) = S;
            S.x = fmaf(f.y, u[i].x, f.x * S.x);
            S.y = fmaf(f.y, u[i].y, f.x * S.y);
            S.z = fmaf(f.y, u[i].z, f.x * S.z);
            S.w = fmaf(f.y, u[i].w, f.x * S.w);
        }
    }
    // the other workgroups may still read the slot that n and m go to: the next launch moves them
    *(float4 *)(is_n ? buf + (size_t)chunks * step : a.state + bh * values + at) = S;
}

// grid (tiles of 64 value dimensions, chunks, heads * batch): 64 tokens x 64 value dimensions on 2 x 2 waves.
__global__ __launch_bounds__(256) void memory_outputs_kernel(MemoryArgs a, int dimp, int vdimp, int chunks) {
    __shared__ __align__(16) float sab[2 * C * LD];
    __shared__ float carry[C], local[C], den[C];  // per token: exp(m - M_t), exp(A_t - M_t), the denominator
    const MemoryShape &s = a.s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave >> 1, wn = wave & 1;
    const int j0 = blockIdx.x * 64, chunk = blockIdx.y, h = blockIdx.z % s.heads, b = blockIdx.z / s.heads, T = a.new_len, t0 = chunk * C, nt = min(C, T - t0);
    const size_t bh = (size_t)b * s.heads + h, row0 = (size_t)b * T + t0;
    const Scratch x = scratch_of(a.scratch, bh, chunks, dimp, vdimp);
    if (blockIdx.x == 0 && chunk == 0) {  // what the scan left for the next call
        float *norm = a.norm + (bh * 2 + ((*a.pos_dev + T) & 1)) * (dimp + 4);
        for (int d = tid; d < dimp; d += 256) norm[d] = x.n[(size_t)chunks * dimp + d];
        if (tid == 0) norm[dimp] = (float)x.m[chunks];
    }
    const float scale = 1.0f / sqrtf((float)s.dim);
    const double m = x.m[chunk];
    if (tid < C) {
        const double F = x.fa[(size_t)chunk * 2 * C + tid], A = x.fa[(size_t)chunk * 2 * C + C + tid], M = fmax(m, A);
        carry[tid] = expf((float)(m - M));
        local[tid] = expf((float)(A - M));
        den[tid] = expf((float)-(F + M));  // exp(-m_t) for now
    }
    f32x16 acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.0f;
    float *sa = sab, *sb = sab + C * LD;
    const int row = tid >> 2, c8 = (tid & 3) * 8;
    const float *qp = a.q + (row0 + min(row, nt - 1)) * a.ld + h * dimp + c8;
    const float *sp = x.s + ((size_t)chunk * vdimp + min(j0 + row, vdimp - 1)) * dimp + c8, *np = x.n + (size_t)chunk * dimp + c8;
    float nq = 0.0f;  // of token `row`: this thread's eighth of every 32 dimensions
    for (int k0 = 0; k0 < dimp; k0 += 32) {
        const float4 q0 = *(const float4 *)(qp + k0), q1 = *(const float4 *)(qp + k0 + 4);
        const float4 s0 = *(const float4 *)(sp + k0), s1 = *(const float4 *)(sp + k0 + 4);
        const float4 n0 = *(const float4 *)(np + k0), n1 = *(const float4 *)(np + k0 + 4);
        nq += q0.x * n0.x + q0.y * n0.y + q0.z * n0.z + q0.w * n0.w + q1.x * n1.x + q1.y * n1.y + q1.z * n1.z + q1.w * n1.w;
        __syncthreads();
        *(float4 *)(sa + row * LD + c8) = q0;
        *(float4 *)(sa + row * LD + c8 + 4) = q1;
        *(float4 *)(sb + row * LD + c8) = s0;
        *(float4 *)(sb + row * LD + c8 + 4) = s1;
        __syncthreads();
        acc = tile_product(sa, sb, wm * 32, wn * 32, lane, acc);
    }
    nq += dpp_move<0xb1, 0xf>(0.0f, nq);
    nq += dpp_move<0x4e, 0xf>(0.0f, nq);
    if ((tid & 3) == 0) den[row] = fmaxf(fabsf(carry[row] * nq * scale + local[row] * x.sums[(size_t)chunk * C + row]), den[row]) + 1e-6f;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] *= carry[wm * 32 + 8 * (r >> 2) + 4 * (lane >> 5) + (r & 3)] * scale;
    for (int k0 = 0; k0 < C; k0 += 32) {  // the chunk's own tokens: P and the transposed values
        const float f = local[row];
        const float *pp = x.p + ((size_t)chunk * C + row) * C + k0 + c8;
        const float4 p0 = *(const float4 *)pp, p1 = *(const float4 *)(pp + 4);
        const int t = tid & 31, j8 = (tid >> 5) * 8;
        const float *vp = a.v + (row0 + min(k0 + t, nt - 1)) * a.ld + h * vdimp;
        float v[8];
        *(float4 *)&v[0] = *(const float4 *)(vp + min(j0 + j8, vdimp - 8));
        *(float4 *)&v[4] = *(const float4 *)(vp + min(j0 + j8, vdimp - 8) + 4);
        __syncthreads();
        *(float4 *)(sa + row * LD + c8) = make_float4(p0.x * f, p0.y * f, p0.z * f, p0.w * f);
        *(float4 *)(sa + row * LD + c8 + 4) = make_float4(p1.x * f, p1.y * f, p1.z * f, p1.w * f);
#pragma unroll
        for (int e = 0; e < 8; ++e) sb[(j8 + e) * LD + t] = v[e];
        __syncthreads();
        acc = tile_product(sa, sb, wm * 32, wn * 32, lane, acc);
    }
    const int j = j0 + wn * 32 + (lane & 31);
    if (j >= vdimp) return;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
        const int t = wm * 32 + 8 * (r >> 2) + 4 * (lane >> 5) + (r & 3);
        if (t < nt) a.out[(row0 + t) * a.ldo + h * vdimp + j] = acc[r] / den[t];
    }
}

}  // namespace

bool memory_supported(const MemoryShape &s) {
    return s.heads > 0 && s.dim > 0 && s.dim <= kMaxDim && s.vdim > 0 && s.cap > 0.0f;
}

size_t memory_scratch_bytes(const MemoryShape &s, int batch, int new_len) {
    return (size_t)batch * s.heads * scratch_per_head(ceil_div(new_len, C), s.dimp(), s.vdimp()) * sizeof(float);
}

int32_t memory_launch(agpu_ctx *ctx, const MemoryArgs &a) {
    const MemoryShape &s = a.s;
    const int dimp = s.dimp(), vdimp = s.vdimp();
    if (!memory_supported(s) || a.batch <= 0 || a.new_len <= 0 || a.ld % 4 != 0 || (int64_t)a.batch * s.heads > 65535 || (int64_t)a.batch * a.new_len > 65535)
        return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "matrix_memory: heads %d, dim %d, vdim %d, %d new tokens not supported", s.heads, s.dim, s.vdim, a.new_len);
    if (a.new_len == 1) {
        const dim3 grid((unsigned)(vdimp / 16), (unsigned)s.heads, (unsigned)a.batch);
        if (dimp <= 64) hipLaunchKernelGGL(memory_step_kernel<1>, grid, dim3(256), 0, ctx->stream, a, dimp, vdimp);
        else if (dimp <= 128) hipLaunchKernelGGL(memory_step_kernel<2>, grid, dim3(256), 0, ctx->stream, a, dimp, vdimp);
        else hipLaunchKernelGGL(memory_step_kernel<4>, grid, dim3(256), 0, ctx->stream, a, dimp, vdimp);
        return AGPU_LAUNCH_CHECK(ctx, "memory_step_kernel");
    }
    const int chunks = ceil_div(a.new_len, C);
    int32_t rc;
    hipLaunchKernelGGL(memory_scores_kernel, dim3((unsigned)chunks, (unsigned)s.heads, (unsigned)a.batch), dim3(256), 0, ctx->stream, a, dimp, vdimp);
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "memory_scores_kernel")) != AGPU_OK) return rc;
    hipLaunchKernelGGL(memory_increments_kernel, dim3((unsigned)(ceil_div(dimp, 64) * chunks), (unsigned)ceil_div(vdimp, 64), (unsigned)(s.heads * a.batch)), dim3(256),
                       0, ctx->stream, a, dimp, vdimp, chunks);
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "memory_increments_kernel")) != AGPU_OK) return rc;
    hipLaunchKernelGGL(memory_scan_kernel, dim3((unsigned)ceil_div((vdimp + 1) * dimp, 1024), (unsigned)(s.heads * a.batch)), dim3(256),
                       (size_t)(chunks + 1) * 4 * sizeof(double), ctx->stream, a, dimp, vdimp, chunks);
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "memory_scan_kernel")) != AGPU_OK) return rc;
    hipLaunchKernelGGL(memory_outputs_kernel, dim3((unsigned)ceil_div(vdimp, 64), (unsigned)chunks, (unsigned)(s.heads * a.batch)), dim3(256), 0, ctx->stream, a,
                       dimp, vdimp, chunks);
    return AGPU_LAUNCH_CHECK(ctx, "memory_outputs_kernel");
}
