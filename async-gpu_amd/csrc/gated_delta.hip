// Gated delta rule (gated_delta.h).  The columns of a head's state evolve independently given q, k, g and beta, so the
// recurrence over a prompt runs token by token with the state in registers: a column is spread over 32 lanes, a wave
// holds two, and the token vectors come through LDS in chunks.  With S the state before the token,
//   S^T diag(g) k and S^T diag(g) q are summed together, u = beta (v - S^T diag(g) k),
//   o = S^T diag(g) q + (k . q) u      (the read-out of the updated state), S <- diag(g) S + k u^T,
// so only one reduction over lanes sits between a token and the next.
#include "gated_delta.h"

namespace {

constexpr int kMaxDim = 256;
constexpr int kChunk = 16;  // tokens staged at a time
constexpr int kRecWaves = 4;

__device__ __forceinline__ float softplus_dev(float v) { return fmaxf(v, 0.0f) + log1pf(expf(-fabsf(v))); }
__device__ __forceinline__ float decay_dev(float a_log, float step) { return expf(-expf(a_log) * softplus_dev(step)); }

// The convolution input of channel c (source column `col` of the projection) at token `s` of the portion; before the
// portion the ring, before the sequence zero.
__device__ __forceinline__ float conv_input(const DeltaArgs &a, int channels, int b, int pos, int s, int c, int col) {
    if (s >= 0) return a.proj[(size_t)(b * a.new_len + s) * a.ld + col];
    const int p = pos + s;
    return p >= 0 ? a.ring[((size_t)b * a.s.taps + p % a.s.taps) * channels + c] : 0.0f;
}

__device__ __forceinline__ float conv_silu(const DeltaArgs &a, int channels, int b, int pos, int s, int c, int col) {
    const int n = a.s.taps;
    const float *w = a.w.conv + (size_t)c * n;
    float v = 0.0f;
    for (int j = 0; j < n; ++j) v = fmaf(w[j], conv_input(a, channels, b, pos, s - (n - 1) + j, c, col), v);
    return silu_dev(v);
}

// One workgroup per token row: convolution, unit vectors, decays, step sizes.
__global__ __launch_bounds__(256) void delta_prepare_kernel(DeltaArgs a, int channels) {
    const DeltaShape &s = a.s;
    const int row = blockIdx.x, b = row / a.new_len, t = row % a.new_len, pos = *a.pos_dev;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int nk = s.kv_heads * s.dim, nv = s.heads * s.vdim;
    float *qk = a.qk + (size_t)row * 2 * nk;
    float *bkq = a.bkq + (size_t)row * (s.heads + s.kv_heads);
    for (int h = wave; h < s.kv_heads; h += 4) {
        float q[kMaxDim / 64], k[kMaxDim / 64];
        float qq = 0.0f, kk = 0.0f;
#pragma unroll
        for (int i = 0; i < kMaxDim / 64; ++i) {
            const int d = lane + 64 * i, c = h * s.dim + d;
            q[i] = k[i] = 0.0f;
            if (d < s.dim) {
                q[i] = conv_silu(a, channels, b, pos, t, c, a.col_q + c);
                k[i] = conv_silu(a, channels, b, pos, t, nk + c, a.col_k + c);
            }
            qq += q[i] * q[i];
            kk += k[i] * k[i];
        }
        const float rq = 1.0f / sqrtf(wave_sum(qq) + 1e-6f) / sqrtf((float)s.dim), rk = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
        float dot = 0.0f;
#pragma unroll
        for (int i = 0; i < kMaxDim / 64; ++i) {
            const int d = lane + 64 * i;
            q[i] *= rq;
            k[i] *= rk;
            dot += q[i] * k[i];
            if (d < s.dim) {
                qk[h * s.dim + d] = q[i];
                qk[nk + h * s.dim + d] = k[i];
            }
        }
        dot = wave_sum(dot);
        if (lane == 0) bkq[s.heads + h] = dot;
    }
    for (int c = threadIdx.x; c < nv; c += 256) a.v[(size_t)row * nv + c] = conv_silu(a, channels, b, pos, t, 2 * nk + c, a.col_v + c);
    const float *p = a.proj + (size_t)row * a.ld;
    for (int h = threadIdx.x; h < s.heads; h += 256) bkq[h] = sigmoid_dev(p[a.col_b + h]);
    float *g = a.g + (size_t)row * s.heads * s.dim;
    for (int c = threadIdx.x; c < s.heads * s.dim; c += 256) g[c] = decay_dev(a.w.a_log[c / s.dim], g[c] + a.w.dt_bias[c]);
}

// The convolution inputs of the last `taps` tokens of the portion into the ring (after every read of the old ones).
__global__ __launch_bounds__(256) void delta_ring_kernel(DeltaArgs a, int channels) {
    const DeltaShape &s = a.s;
    const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.z, t = a.new_len - 1 - (int)blockIdx.y;
    if (c >= channels || t < 0) return;
    const int nk = s.kv_heads * s.dim;
    const int col = c < nk ? a.col_q + c : (c < 2 * nk ? a.col_k + c - nk : a.col_v + c - 2 * nk);
    a.ring[((size_t)b * s.taps + (*a.pos_dev + t) % s.taps) * channels + c] = a.proj[(size_t)(b * a.new_len + t) * a.ld + col];
}

// Sum over each half of a wave, in every lane of the half.
__device__ __forceinline__ float half_sum(float v) {
    v = row16_sum(v);
    const auto sw = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return __uint_as_float(sw[0]) + __uint_as_float(sw[1]);
}

// grid (column groups of 8, heads, batch).  DR values of a column per lane.
template <int DR>
__global__ __launch_bounds__(64 * kRecWaves) void delta_recurrence_kernel(DeltaArgs a) {
    constexpr int DP = 32 * DR, NT = 64 * kRecWaves, COLS = 2 * kRecWaves;
    __shared__ __align__(16) float sv[2][kChunk][3][DP];  // q, k, g
    __shared__ float sc[2][kChunk][COLS + 2];             // v of the columns, beta, k . q
    const DeltaShape &s = a.s;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, l32 = lane & 31, half = lane >> 5;
    const int h = blockIdx.y, b = blockIdx.z, j0 = blockIdx.x * COLS, j = j0 + wave * 2 + half;
    const int hk = h / (s.heads / s.kv_heads), nk = s.kv_heads * s.dim, nv = s.heads * s.vdim, T = a.new_len;
    const size_t row0 = (size_t)b * T;
    float *st = a.state + (((size_t)b * s.heads + h) * s.vdim + min(j, s.vdim - 1)) * DP + l32 * DR;
    float S[DR];
#pragma unroll
    for (int r = 0; r < DR; ++r) S[r] = st[r];
    auto stage = [&](int buf, int t0) {
        for (int i = t; i < kChunk * 3 * DP; i += NT) {
            const int d = i % DP, w = (i / DP) % 3, tok = t0 + i / (3 * DP);
            const size_t row = row0 + min(tok, T - 1);
            const int dd = min(d, s.dim - 1);
            const float *src = w == 2 ? a.g + row * s.heads * s.dim + h * s.dim : a.qk + row * 2 * nk + w * nk + hk * s.dim;
            const float v = d < s.dim ? src[dd] : 0.0f;
            sv[buf][i / (3 * DP)][w][d] = tok < T ? v : (w == 2 ? 1.0f : 0.0f);  // behind the last token nothing moves
        }
        for (int i = t; i < kChunk * (COLS + 2); i += NT) {
            const int c = i % (COLS + 2);
            const size_t row = row0 + min(t0 + i / (COLS + 2), T - 1);
            const float *bkq = a.bkq + row * (s.heads + s.kv_heads);
            float v;
            if (c < COLS) v = a.v[row * nv + h * s.vdim + min(j0 + c, s.vdim - 1)];
            else v = c == COLS ? bkq[h] : bkq[s.heads + hk];
            sc[buf][i / (COLS + 2)][c] = v;
        }
    };
    stage(0, 0);
    int buf = 0;
    for (int t0 = 0; t0 < T; t0 += kChunk, buf ^= 1) {
        __syncthreads();
        if (t0 + kChunk < T) stage(buf ^ 1, t0 + kChunk);
        // the vectors of the next token are on their way while this one is worked on
        float q[DR], k[DR], g[DR], v, beta, kq;
        auto fetch = [&](int i) {
#pragma unroll
            for (int r = 0; r < DR; ++r) {
                q[r] = sv[buf][i][0][l32 * DR + r];
                k[r] = sv[buf][i][1][l32 * DR + r];
                g[r] = sv[buf][i][2][l32 * DR + r];
            }
            v = sc[buf][i][wave * 2 + half];
            beta = sc[buf][i][COLS];
            kq = sc[buf][i][COLS + 1];
        };
        fetch(0);
#pragma unroll 4
        for (int i = 0; i < kChunk; ++i) {
            float kc[DR];
            float ks = 0.0f, qs = 0.0f;
            const float vc = v, bc = beta, kqc = kq;
#pragma unroll
            for (int r = 0; r < DR; ++r) {
                kc[r] = k[r];
                S[r] *= g[r];
                ks = fmaf(S[r], kc[r], ks);
                qs = fmaf(S[r], q[r], qs);
            }
            fetch(min(i + 1, kChunk - 1));
            ks = half_sum(ks);
            qs = half_sum(qs);
            const float u = bc * (vc - ks);
#pragma unroll
            for (int r = 0; r < DR; ++r) S[r] = fmaf(kc[r], u, S[r]);
            if (l32 == 0 && j < s.vdim && t0 + i < T) a.o[(row0 + t0 + i) * nv + h * s.vdim + j] = fmaf(kqc, u, qs);
        }
    }
    if (j < s.vdim) {
#pragma unroll
        for (int r = 0; r < DR; ++r) st[r] = S[r];
    }
}

// Per head: o / rms(o) * norm * sigmoid(gate).  One workgroup per row, one wave per head.
__global__ __launch_bounds__(256) void delta_gate_kernel(DeltaArgs a) {
    const DeltaShape &s = a.s;
    const int row = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nv = s.heads * s.vdim;
    for (int h = wave; h < s.heads; h += 4) {
        const float *o = a.o + (size_t)row * nv + h * s.vdim;
        float sum = 0.0f;
        for (int d = lane; d < s.vdim; d += 64) sum += o[d] * o[d];
        const float rs = 1.0f / sqrtf(wave_sum(sum) / (float)s.vdim + s.eps);
        for (int d = lane; d < s.vdim; d += 64) {
            const float v = o[d] * rs * a.w.norm[d] * sigmoid_dev(a.gate[(size_t)row * nv + h * s.vdim + d]);
            const size_t at = (size_t)row * a.ldo + h * s.vdim + d;
            if (a.out_bf16) ((uint16_t *)a.out)[at] = f32_to_bf16(v);
            else ((float *)a.out)[at] = v;
        }
    }
}

// Low-rank product: out[r] = sum_k w[row0 + r][k] x[k] for r < n, rank a multiple of 32; 16 lanes per row.
__device__ __forceinline__ void low_rank(const uint16_t *w, int rank, const float *x, float *out, int n, int threads) {
    const int lane = threadIdx.x & 63, kl = lane & 15, group = threadIdx.x >> 4;
    for (int r = group; r < n; r += threads / 16) {
        float acc = 0.0f;
        for (int k = kl * 8; k < rank; k += 128) {
            const uint4 v = *(const uint4 *)(w + (size_t)r * rank + k);
            const uint32_t u[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                acc = fmaf(__uint_as_float(u[e] << 16), x[k + 2 * e], acc);
                acc = fmaf(__uint_as_float(u[e] & 0xffff0000u), x[k + 2 * e + 1], acc);
            }
        }
        acc = row16_sum(acc);
        if (kl == 0) out[r] = acc;
    }
}

constexpr int kStepThreads = 512;

// One token of one sequence and head: grid (heads, batch).  NF float4 of a state column per lane of 16.
template <int NF>
__global__ __launch_bounds__(kStepThreads) void delta_step_kernel(DeltaArgs a, int channels, int rank_ap, int rank_gp, int state_row) {
    extern __shared__ float low[];  // a1 [rank_ap], g1 [rank_gp]
    __shared__ __align__(16) float sq[kMaxDim], sk[kMaxDim], sg[kMaxDim];
    __shared__ float svv[kMaxDim], sgate[kMaxDim], so[kMaxDim];
    __shared__ float red[4];
    const DeltaShape &s = a.s;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int h = blockIdx.x, b = blockIdx.y, group = s.heads / s.kv_heads, hk = h / group, pos = *a.pos_dev;
    const int nk = s.kv_heads * s.dim;
    const float *p = a.proj + (size_t)b * a.ld;
    float *state = a.state + ((size_t)b * s.heads + h) * s.vdim * state_row;
    const int kl = lane & 15, col0 = t >> 4;  // 32 columns at a time
    constexpr int COLS = kStepThreads / 16;
    // the first columns of the state are requested before anything else
    float4 first[NF];
#pragma unroll
    for (int f = 0; f < NF; ++f) {
        const int d = kl * 4 + 64 * f;
        first[f] = (d < state_row && col0 < s.vdim) ? *(const float4 *)(state + (size_t)col0 * state_row + d) : make_float4(0, 0, 0, 0);
    }
    for (int k = t; k < rank_ap; k += kStepThreads) low[k] = p[a.col_a1 + k];
    for (int k = t; k < rank_gp; k += kStepThreads) low[rank_ap + k] = p[a.col_g1 + k];
    for (int d = t; d < kMaxDim; d += kStepThreads) {
        const int c = hk * s.dim + d;
        sq[d] = d < s.dim ? conv_silu(a, channels, b, pos, 0, c, a.col_q + c) : 0.0f;
        sk[d] = d < s.dim ? conv_silu(a, channels, b, pos, 0, nk + c, a.col_k + c) : 0.0f;
        sg[d] = 0.0f;
        const int cv = h * s.vdim + d;
        if (d < s.vdim) svv[d] = conv_silu(a, channels, b, pos, 0, 2 * nk + cv, a.col_v + cv);
    }
    // the new inputs into the ring: a slot that no tap of this token reads.  q and k by the first head of a group.
    float *slot = a.ring + ((size_t)b * s.taps + pos % s.taps) * channels;
    if (h % group == 0)
        for (int d = t; d < s.dim; d += kStepThreads) {
            const int c = hk * s.dim + d;
            slot[c] = p[a.col_q + c];
            slot[nk + c] = p[a.col_k + c];
        }
    for (int d = t; d < s.vdim; d += kStepThreads) slot[2 * nk + h * s.vdim + d] = p[a.col_v + h * s.vdim + d];
    __syncthreads();
    low_rank(a.w.a2 + (size_t)h * s.dim * rank_ap, rank_ap, low, sg, s.dim, kStepThreads);
    low_rank(a.w.g2 + (size_t)h * s.vdim * rank_gp, rank_gp, low + rank_ap, sgate, s.vdim, kStepThreads);
    if (wave < 3) {  // |q|^2, |k|^2, q . k
        float v = 0.0f;
        for (int d = lane; d < kMaxDim; d += 64) v += (wave == 1 ? sk[d] : sq[d]) * (wave == 0 ? sq[d] : sk[d]);
        v = wave_sum(v);
        if (lane == 0) red[wave] = v;
    }
    __syncthreads();
    const float rq = 1.0f / sqrtf(red[0] + 1e-6f) / sqrtf((float)s.dim), rk = 1.0f / sqrtf(red[1] + 1e-6f);
    const float kq = red[2] * rq * rk, beta = sigmoid_dev(p[a.col_b + h]);
    for (int d = t; d < s.dim; d += kStepThreads) sg[d] = decay_dev(a.w.a_log[h], sg[d] + a.w.dt_bias[h * s.dim + d]);
    __syncthreads();
    for (int j = col0; j < s.vdim; j += COLS) {
        float4 S[NF], k4[NF];
        float ks = 0.0f, qs = 0.0f;
#pragma unroll
        for (int f = 0; f < NF; ++f) {
            const int d = kl * 4 + 64 * f;
            S[f] = first[f];
            if (j != col0) S[f] = d < state_row ? *(const float4 *)(state + (size_t)j * state_row + d) : make_float4(0, 0, 0, 0);
            const float4 g4 = *(const float4 *)&sg[d], q4 = *(const float4 *)&sq[d];
            k4[f] = *(const float4 *)&sk[d];
            S[f].x *= g4.x; S[f].y *= g4.y; S[f].z *= g4.z; S[f].w *= g4.w;
            ks += S[f].x * k4[f].x + S[f].y * k4[f].y + S[f].z * k4[f].z + S[f].w * k4[f].w;
            qs += S[f].x * q4.x + S[f].y * q4.y + S[f].z * q4.z + S[f].w * q4.w;
        }
        ks = row16_sum(ks) * rk;
        qs = row16_sum(qs) * rq;
        const float u = beta * (svv[j] - ks), uk = u * rk;
#pragma unroll
        for (int f = 0; f < NF; ++f) {
            const int d = kl * 4 + 64 * f;
            S[f].x = fmaf(k4[f].x, uk, S[f].x);
            S[f].y = fmaf(k4[f].y, uk, S[f].y);
            S[f].z = fmaf(k4[f].z, uk, S[f].z);
            S[f].w = fmaf(k4[f].w, uk, S[f].w);
            if (d < state_row) *(float4 *)(state + (size_t)j * state_row + d) = S[f];
        }
        if (kl == 0) so[j] = fmaf(kq, u, qs);
    }
    __syncthreads();
    if (wave == 0) {
        float sum = 0.0f;
        for (int d = lane; d < s.vdim; d += 64) sum += so[d] * so[d];
        sum = wave_sum(sum);
        if (lane == 0) red[3] = 1.0f / sqrtf(sum / (float)s.vdim + s.eps);
    }
    __syncthreads();
    for (int d = t; d < s.vdim; d += kStepThreads) {
        const float v = so[d] * red[3] * a.w.norm[d] * sigmoid_dev(sgate[d]);
        const size_t at = (size_t)b * a.ldo + h * s.vdim + d;
        if (a.out_bf16) ((uint16_t *)a.out)[at] = f32_to_bf16(v);
        else ((float *)a.out)[at] = v;
    }
}

int32_t check(agpu_ctx *ctx, const DeltaArgs &a) {
    if (!delta_supported(a.s) || a.batch <= 0 || a.new_len <= 0)
        return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "gated_delta: heads %d/%d, dim %d, vdim %d, taps %d not supported", a.s.heads, a.s.kv_heads, a.s.dim,
                         a.s.vdim, a.s.taps);
    return AGPU_OK;
}

}  // namespace

bool delta_supported(const DeltaShape &s) {
    return s.heads > 0 && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim > 0 && s.dim <= kMaxDim && s.vdim > 0 && s.vdim <= kMaxDim && s.taps >= 1 &&
           s.rank_a > 0 && s.rank_g > 0 && s.rank_ap() + s.rank_gp() <= 8192;
}

int32_t delta_step_launch(agpu_ctx *ctx, const DeltaArgs &a) {
    int32_t rc = check(ctx, a);
    if (rc != AGPU_OK) return rc;
    if (a.new_len != 1) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "gated_delta: the step takes one token per sequence");
    const DeltaShape &s = a.s;
    const dim3 grid((unsigned)s.heads, (unsigned)a.batch), block(kStepThreads);
    const size_t lds = (size_t)(s.rank_ap() + s.rank_gp()) * sizeof(float);
    const int nf = ceil_div(s.state_row(), 64);
#define AGPU_DELTA_STEP(NF) \
    hipLaunchKernelGGL(delta_step_kernel<NF>, grid, block, lds, ctx->stream, a, s.channels(), s.rank_ap(), s.rank_gp(), s.state_row())
    if (nf <= 1) AGPU_DELTA_STEP(1);
    else if (nf <= 2) AGPU_DELTA_STEP(2);
    else AGPU_DELTA_STEP(4);
#undef AGPU_DELTA_STEP
    return AGPU_LAUNCH_CHECK(ctx, "delta_step_kernel");
}

int32_t delta_prefill_launch(agpu_ctx *ctx, const DeltaArgs &a) {
    int32_t rc = check(ctx, a);
    if (rc != AGPU_OK) return rc;
    const DeltaShape &s = a.s;
    const unsigned rows = (unsigned)(a.batch * a.new_len);
    hipLaunchKernelGGL(delta_prepare_kernel, dim3(rows), dim3(256), 0, ctx->stream, a, s.channels());
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "delta_prepare_kernel")) != AGPU_OK) return rc;
    hipLaunchKernelGGL(delta_ring_kernel, dim3((unsigned)ceil_div(s.channels(), 256), (unsigned)s.taps, (unsigned)a.batch), dim3(256), 0, ctx->stream, a,
                       s.channels());
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "delta_ring_kernel")) != AGPU_OK) return rc;
    const dim3 grid((unsigned)ceil_div(s.vdim, 2 * kRecWaves), (unsigned)s.heads, (unsigned)a.batch), block(64 * kRecWaves);
    switch (s.state_row() / 32) {
#define AGPU_DELTA_REC(DR) \
    case DR: hipLaunchKernelGGL(delta_recurrence_kernel<DR>, grid, block, 0, ctx->stream, a); break
        AGPU_DELTA_REC(1);
        AGPU_DELTA_REC(2);
        AGPU_DELTA_REC(3);
        AGPU_DELTA_REC(4);
        AGPU_DELTA_REC(5);
        AGPU_DELTA_REC(6);
        AGPU_DELTA_REC(7);
        AGPU_DELTA_REC(8);
#undef AGPU_DELTA_REC
    }
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "delta_recurrence_kernel")) != AGPU_OK) return rc;
    hipLaunchKernelGGL(delta_gate_kernel, dim3(rows), dim3(256), 0, ctx->stream, a);
    return AGPU_LAUNCH_CHECK(ctx, "delta_gate_kernel");
}
