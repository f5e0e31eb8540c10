// Latent attention (latent_attention.h).  Two forms of the same mathematics:
//
// absorbed (decode, short portions, fp32 models): the query of a head goes through W_uk^T once and then meets the cached
//   latents directly, so the cache is read as it is.  Launches: absorb (cache row, absorbed and rotated queries) -> attend
//   (keys split over workgroups) -> merge with the sink, then W_uv.  With a bf16 cache 16 heads meet the cache on the bf16
//   matrix cores, queries and probabilities as two bf16 pieces each (16 bits of mantissa); with an fp32 cache, or a latent
//   too wide for the LDS, four heads at a time on fp32 FMAs.
// tiled (prompts of a bf16 model): keys and transposed values of every head are expanded by two GEMMs, then S^T = K Q^T and
//   O^T = V^T P^T on v_mfma_f32_32x32x16_bf16 with an online softmax.  The key rows of a tile are dealt to the rows of
//   the first product so that the probabilities come out as the second product's operand: row i of a 32-key tile is key
//   16 ((i >> 2) & 1) + 4 (i >> 3) + (i & 3); a half-wave then holds 16 consecutive keys.
#include <algorithm>

#include "latent_attention.h"

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr int kHeadTile = 4;    // heads per workgroup of the absorbed kernel (one softmax per wave)
constexpr int kKeyChunk = 64;   // keys per step: one per lane
constexpr int kMaxSplits = 64;
constexpr int kMatrixHeads = 16;  // heads per workgroup of the matrix-core kernel
constexpr int kMatrixChunk = 32;  // keys per step of the matrix-core kernel
constexpr float kMinusInf = -3.0e38f;

// Element i of a rotated part v[0 .. rot): dimension i < dims / 2 turns with i + dims / 2.
__device__ __forceinline__ float rotated(const float *v, int i, int dims, const float2 *cs) {
    const int half = dims >> 1;
    if (i >= dims) return v[i];
    const float2 t = cs[i < half ? i : i - half];
    return i < half ? v[i] * t.x - v[i + half] * t.y : v[i] * t.x + v[i - half] * t.y;
}

template <typename CT>
__device__ __forceinline__ CT to_cache(float v);
template <>
__device__ __forceinline__ float to_cache<float>(float v) { return v; }
template <>
__device__ __forceinline__ uint16_t to_cache<uint16_t>(float v) { return f32_to_bf16(v); }

// The cache row of one token: normed latent and rotated key part.  256 threads.
template <typename CT>
__device__ __forceinline__ void write_cache_row(const LatentArgs &a, const LatentShape &s, int rankp, int row_len, int row, int pos, float *red) {
    const int t = threadIdx.x, b = row / a.new_len;
    const float *src = a.down + (size_t)row * a.ld;
    CT *dst = (CT *)a.cache + ((size_t)b * a.positions + pos) * row_len;
    float sum = 0.0f;
    for (int k = t; k < s.rank; k += 256) sum += src[k] * src[k];
    sum = wave_sum(sum);
    if ((t & 63) == 0) red[t >> 6] = sum;
    __syncthreads();
    const float rs = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)s.rank + s.eps);
    for (int k = t; k < rankp; k += 256) dst[k] = to_cache<CT>(k < s.rank ? src[k] * rs * a.w.norm[k] : 0.0f);
    const float2 *cs = a.w.rope + (size_t)pos * (s.rot_dims >> 1);
    for (int i = t; i < row_len - rankp; i += 256) dst[rankp + i] = to_cache<CT>(i < s.rot ? rotated(src + s.rank, i, s.rot_dims, cs) : 0.0f);
}

// A query value for the attend kernel: fp32, or two bf16 pieces whose sum carries 16 bits of its mantissa.
template <typename CT>
__device__ __forceinline__ void put_query(void *qlat, size_t at, size_t pieces, float v);
template <>
__device__ __forceinline__ void put_query<float>(void *qlat, size_t at, size_t, float v) { ((float *)qlat)[at] = v; }
template <>
__device__ __forceinline__ void put_query<uint16_t>(void *qlat, size_t at, size_t pieces, float v) {
    const uint16_t hi = f32_to_bf16(v);
    ((uint16_t *)qlat)[at] = hi;
    ((uint16_t *)qlat)[pieces + at] = f32_to_bf16(v - bf16_to_f32(hi));
}

// grid (1 + heads * ceil(rankp / 128), rows): block 0 writes the cache row, the others 128 columns of a head's absorbed query.
// QT: how the attend kernel reads queries (uint16_t: bf16 pieces).
template <typename CT, typename QT>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentArgs a, int rankp, int row_len, int dimp, int col_blocks) {
    __shared__ float part[16][128];
    __shared__ float red[4];
    const LatentShape &s = a.s;
    const int t = threadIdx.x, row = blockIdx.y;
    const int pos = *a.pos_dev + row % a.new_len;
    if (blockIdx.x == 0) {
        write_cache_row<CT>(a, s, rankp, row_len, row, pos, red);
        return;
    }
    const int h = (blockIdx.x - 1) / col_blocks, cb = (blockIdx.x - 1) % col_blocks;
    const float *q = a.q + (size_t)row * a.ld + (size_t)h * (s.dim + s.rot);
    const size_t at = ((size_t)row * s.heads + h) * row_len, pieces = (size_t)gridDim.y * s.heads * row_len;
    // 16 lanes take the columns, 16 groups the query's dimensions; loads are clamped, not skipped
    const int c = cb * 128 + (t & 15) * 8, g = t >> 4;
    const uint16_t *w = a.w.uk + (size_t)h * dimp * rankp + min(c, rankp - 8);
    float acc[8] = {0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll 1
    for (int d0 = g; d0 < s.dim; d0 += 16 * 8) {
        uint4 v[8];
        float x[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int d = min(d0 + 16 * u, s.dim - 1);
            v[u] = *(const uint4 *)(w + (size_t)d * rankp);
            x[u] = d0 + 16 * u < s.dim ? q[d] : 0.0f;
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const uint32_t p[4] = {v[u].x, v[u].y, v[u].z, v[u].w};
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                acc[2 * e] = fmaf(__uint_as_float(p[e] << 16), x[u], acc[2 * e]);
                acc[2 * e + 1] = fmaf(__uint_as_float(p[e] & 0xffff0000u), x[u], acc[2 * e + 1]);
            }
        }
    }
    *(float4 *)&part[g][(t & 15) * 8] = make_float4(acc[0], acc[1], acc[2], acc[3]);
    *(float4 *)&part[g][(t & 15) * 8 + 4] = make_float4(acc[4], acc[5], acc[6], acc[7]);
    if (cb == 0) {
        const float2 *cs = a.w.rope + (size_t)pos * (s.rot_dims >> 1);
        for (int i = t; i < row_len - rankp; i += 256)
            put_query<QT>(a.qlat, at + rankp + i, pieces, i < s.rot ? rotated(q + s.dim, i, s.rot_dims, cs) : 0.0f);
    }
    __syncthreads();
    if (t < 128 && cb * 128 + t < rankp) {
        float v = 0.0f;
#pragma unroll
        for (int i = 0; i < 16; ++i) v += part[i][t];
        put_query<QT>(a.qlat, at + cb * 128 + t, pieces, v);
    }
}

__device__ __forceinline__ void load8(const uint16_t *p, float (&v)[8]) {
    const uint4 w = *(const uint4 *)p;
    const uint32_t u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        v[2 * e] = __uint_as_float(u[e] << 16);
        v[2 * e + 1] = __uint_as_float(u[e] & 0xffff0000u);
    }
}
__device__ __forceinline__ void load8(const float *p, float (&v)[8]) {
    *(float4 *)&v[0] = *(const float4 *)p;
    *(float4 *)&v[4] = *(const float4 *)(p + 4);
}
__device__ __forceinline__ float2 load2(const uint16_t *p) {
    const uint32_t u = *(const uint32_t *)p;
    return make_float2(__uint_as_float(u << 16), __uint_as_float(u & 0xffff0000u));
}
__device__ __forceinline__ float2 load2(const float *p) { return *(const float2 *)p; }

// grid (splits, head tiles, rows), four waves.  Scores: one key per lane, the waves share the cache row's columns (the
// query values are the same for a whole wave).  Softmax: one head per wave.  Values: the waves share the keys, a lane owns
// columns 2 lane + 128 i, + 1.
template <typename CT, int NI>
__global__ __launch_bounds__(256) void latent_attend_kernel(LatentArgs a, const float *__restrict__ qlat, int rankp, int row_len, int splits) {
    __shared__ float sc[4][kHeadTile][kKeyChunk];
    __shared__ float4 pr[kKeyChunk];
    __shared__ float corr[kHeadTile];
    __shared__ float merge[4][kHeadTile][128];
    const LatentShape &s = a.s;
    const int lane = threadIdx.x & 63;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int row = blockIdx.z, h0 = blockIdx.y * kHeadTile, b = row / a.new_len;
    const int kv = *a.pos_dev + row % a.new_len + 1;
    const int chunks = (kv + kKeyChunk - 1) / kKeyChunk;
    const int per = (chunks + splits - 1) / splits;
    const int c_lo = min((int)blockIdx.x * per, chunks), c_hi = min(c_lo + per, chunks);
    const CT *cache = (const CT *)a.cache + (size_t)b * a.positions * row_len;
    const float *q[kHeadTile];
#pragma unroll
    for (int i = 0; i < kHeadTile; ++i) q[i] = qlat + ((size_t)row * s.heads + min(h0 + i, s.heads - 1)) * row_len;
    float acc[kHeadTile][NI][2];
#pragma unroll
    for (int i = 0; i < kHeadTile; ++i)
#pragma unroll
        for (int j = 0; j < NI; ++j) acc[i][j][0] = acc[i][j][1] = 0.0f;
    float m = kMinusInf, l = 0.0f;  // of head h0 + wave
    for (int ck = c_lo; ck < c_hi; ++ck) {
        const int k0 = ck * kKeyChunk;
        const CT *mine = cache + (size_t)min(k0 + lane, kv - 1) * row_len;
        float part[kHeadTile] = {0.0f, 0.0f, 0.0f, 0.0f};
        constexpr int U = 3;  // requests in flight; row_len is a multiple of 32, so every wave has row_len / 32 of them
        int c = wave * 8;
        auto add = [&](int at, const float (&v)[8]) {
#pragma unroll
            for (int i = 0; i < kHeadTile; ++i)
#pragma unroll
                for (int e = 0; e < 8; ++e) part[i] = fmaf(q[i][at + e], v[e], part[i]);
        };
#pragma unroll 1
        for (; c + 32 * (U - 1) < row_len; c += 32 * U) {
            float v[U][8];
#pragma unroll
            for (int u = 0; u < U; ++u) load8(mine + c + 32 * u, v[u]);
#pragma unroll
            for (int u = 0; u < U; ++u) add(c + 32 * u, v[u]);
        }
#pragma unroll 1
        for (; c < row_len; c += 32) {
            float v[8];
            load8(mine + c, v);
            add(c, v);
        }
#pragma unroll
        for (int i = 0; i < kHeadTile; ++i) sc[wave][i][lane] = part[i];
        __syncthreads();
        {
            float v = (sc[0][wave][lane] + sc[1][wave][lane] + sc[2][wave][lane] + sc[3][wave][lane]) * s.scale;
            const bool on = k0 + lane < kv;
            v = on ? v : kMinusInf;
            const float m_new = fmaxf(m, wave_max(v));
            const float p = on ? expf(v - m_new) : 0.0f;
            const float cr = expf(m - m_new);
            l = l * cr + wave_sum(p);
            m = m_new;
            ((float *)&pr[lane])[wave] = p;
            if (lane == 0) corr[wave] = cr;
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < kHeadTile; ++i) {
            const float cr = corr[i];
#pragma unroll
            for (int j = 0; j < NI; ++j) {
                acc[i][j][0] *= cr;
                acc[i][j][1] *= cr;
            }
        }
        constexpr int KU = NI <= 4 ? 16 / NI : 2;  // rows requested at a time
#pragma unroll KU
        for (int kk = 0; kk < 16; ++kk) {
            const int key = wave * 16 + kk;
            const CT *vr = cache + (size_t)min(k0 + key, kv - 1) * row_len;
            const float4 p = pr[key];
            const float pv[4] = {p.x, p.y, p.z, p.w};
#pragma unroll
            for (int j = 0; j < NI; ++j) {
                const int c = 2 * lane + 128 * j;
                const float2 v = load2(vr + min(c, rankp - 2));  // columns beyond the latent are dropped below
#pragma unroll
                for (int i = 0; i < kHeadTile; ++i) {
                    acc[i][j][0] = fmaf(pv[i], v.x, acc[i][j][0]);
                    acc[i][j][1] = fmaf(pv[i], v.y, acc[i][j][1]);
                }
            }
        }
    }
    // the waves' sums of each column, then the partial result of every head
    float *part_o = a.partial;
    float *part_ml = a.partial + (size_t)gridDim.z * s.heads * splits * rankp;
#pragma unroll
    for (int j = 0; j < NI; ++j) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < kHeadTile; ++i) *(float2 *)&merge[wave][i][2 * lane] = make_float2(acc[i][j][0], acc[i][j][1]);
        __syncthreads();
        for (int t = threadIdx.x; t < kHeadTile * 128; t += 256) {
            const int i = t >> 7, c = (t & 127) + 128 * j;
            if (h0 + i < s.heads && c < rankp)
                part_o[(((size_t)row * s.heads + h0 + i) * splits + blockIdx.x) * rankp + c] =
                    merge[0][i][t & 127] + merge[1][i][t & 127] + merge[2][i][t & 127] + merge[3][i][t & 127];
        }
    }
    if (lane == 0 && h0 + wave < s.heads)
        *(float2 *)(part_ml + (((size_t)row * s.heads + h0 + wave) * splits + blockIdx.x) * 2) = make_float2(m, l);
}

// grid (splits, ceil(heads / 16), rows), four waves; bf16 cache.  A chunk of 32 cache rows goes to LDS.  Scores
// (v_mfma_f32_16x16x32_bf16, queries as two pieces, in registers): the waves share the cache row's columns, 32 at a time, and
// add up in LDS; 16 threads per head do the softmax; the waves share the latent's columns of the second product
// (probabilities as two pieces).  CT column tiles of 16 per wave, NK steps of 32 cache columns per wave.
template <int CT, int NK>
__global__ __launch_bounds__(256, 2) void latent_attend_matrix_kernel(LatentArgs a, int rankp, int row_len, int splits) {
    extern __shared__ __align__(16) uint16_t tile[];  // [32][ld]
    __shared__ float sc[4][kMatrixHeads][kMatrixChunk + 4];
    __shared__ __align__(16) uint16_t pr[2][kMatrixHeads][kMatrixChunk + 8];
    __shared__ float corr[kMatrixHeads];
    const LatentShape &s = a.s;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, lr = lane & 15, lq = lane >> 4;
    const int row = blockIdx.z, h0 = blockIdx.y * kMatrixHeads, b = row / a.new_len, ld = row_len + 8, n32 = row_len >> 5;
    const int kv = *a.pos_dev + row % a.new_len + 1;
    const int chunks = (kv + kMatrixChunk - 1) / kMatrixChunk;
    const int per = (chunks + splits - 1) / splits;
    const int c_lo = min((int)blockIdx.x * per, chunks), c_hi = min(c_lo + per, chunks);
    const uint16_t *cache = (const uint16_t *)a.cache + (size_t)b * a.positions * row_len;
    const size_t pieces = (size_t)gridDim.z * s.heads * row_len;
    bf16x8 qf[NK][2];  // of column step wave + 4 n; zero beyond the row
    {
        const uint16_t *q = (const uint16_t *)a.qlat + ((size_t)row * s.heads + min(h0 + lr, s.heads - 1)) * row_len + lq * 8;
#pragma unroll
        for (int n = 0; n < NK; ++n)
#pragma unroll
            for (int pc = 0; pc < 2; ++pc) {
                const int step = wave + 4 * n;
                const uint4 v = *(const uint4 *)(q + pc * pieces + min(step, n32 - 1) * 32);
                qf[n][pc] = __builtin_bit_cast(bf16x8, step < n32 ? v : make_uint4(0, 0, 0, 0));
            }
    }
    f32x4 acc[CT];
#pragma unroll
    for (int i = 0; i < CT; ++i) acc[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    float m = kMinusInf, l = 0.0f;  // of head h0 + t / 16
    for (int ck = c_lo; ck < c_hi; ++ck) {
        const int k0 = ck * kMatrixChunk;
        {  // eight threads per key
            const uint16_t *src = cache + (size_t)min(k0 + (t >> 3), kv - 1) * row_len;
            uint16_t *dst = tile + (t >> 3) * ld;
            constexpr int U = 2 * NK;  // row_len / 8 pieces of 16 bytes over 8 threads
            uint4 v[U];
#pragma unroll
            for (int u = 0; u < U; ++u) v[u] = *(const uint4 *)(src + min(((t & 7) + 8 * u) * 8, row_len - 8));
#pragma unroll
            for (int u = 0; u < U; ++u) *(uint4 *)(dst + min(((t & 7) + 8 * u) * 8, row_len - 8)) = v[u];
        }
        __syncthreads();
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            f32x4 hi = {0.0f, 0.0f, 0.0f, 0.0f}, lo = hi;
            const uint16_t *kp = tile + (kt * 16 + lr) * ld + lq * 8;
#pragma unroll
            for (int n = 0; n < NK; ++n) {
                const bf16x8 kf = *(const bf16x8 *)(kp + min(wave + 4 * n, n32 - 1) * 32);
                lo = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[n][1], kf, lo, 0, 0, 0);
                hi = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[n][0], kf, hi, 0, 0, 0);
            }
            // result register r of lane l: head 4 (l / 16) + r, key l % 16
#pragma unroll
            for (int r = 0; r < 4; ++r) sc[wave][lq * 4 + r][kt * 16 + lr] = hi[r] + lo[r];
        }
        __syncthreads();
        {
            const int h = t >> 4;
            float v[2];
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const int k = lr + 16 * e;
                const float x = (sc[0][h][k] + sc[1][h][k] + sc[2][h][k] + sc[3][h][k]) * s.scale;
                v[e] = k0 + k < kv ? x : kMinusInf;
            }
            const float m_new = fmaxf(m, row16_max(fmaxf(v[0], v[1])));
            float sum = 0.0f;
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const float p = v[e] > kMinusInf ? expf(v[e] - m_new) : 0.0f;
                sum += p;
                const uint16_t hi = f32_to_bf16(p);
                pr[0][h][lr + 16 * e] = hi;
                pr[1][h][lr + 16 * e] = f32_to_bf16(p - bf16_to_f32(hi));
            }
            const float cr = expf(m - m_new);
            l = l * cr + row16_sum(sum);
            m = m_new;
            if (lr == 0) corr[h] = cr;
        }
        __syncthreads();
        float cr[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) cr[r] = corr[lq * 4 + r];
        const bf16x8 phi = *(const bf16x8 *)&pr[0][lr][8 * lq], plo = *(const bf16x8 *)&pr[1][lr][8 * lq];
#pragma unroll
        for (int i = 0; i < CT; ++i) {  // columns beyond the latent repeat its last ones and are dropped
            const int c = min((wave + 4 * i) * 16, rankp - 16);
            const uint16_t *vp = tile + 8 * lq * ld + c + lr;
            uint32_t w[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) w[e] = (uint32_t)vp[2 * e * ld] | ((uint32_t)vp[(2 * e + 1) * ld] << 16);
            const bf16x8 vf = __builtin_bit_cast(bf16x8, make_uint4(w[0], w[1], w[2], w[3]));
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[i][r] *= cr[r];
            acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(plo, vf, acc[i], 0, 0, 0);
            acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(phi, vf, acc[i], 0, 0, 0);
        }
        __syncthreads();  // the next chunk overwrites the tile
    }
    float *part_o = a.partial;
    float *part_ml = a.partial + (size_t)gridDim.z * s.heads * splits * rankp;
#pragma unroll
    for (int i = 0; i < CT; ++i) {
        const int c = (wave + 4 * i) * 16 + lr;
        if (c >= rankp) continue;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int h = h0 + lq * 4 + r;
            if (h < s.heads) part_o[(((size_t)row * s.heads + h) * splits + blockIdx.x) * rankp + c] = acc[i][r];
        }
    }
    if (lr == 0 && h0 + (t >> 4) < s.heads)
        *(float2 *)(part_ml + (((size_t)row * s.heads + h0 + (t >> 4)) * splits + blockIdx.x) * 2) = make_float2(m, l);
}

size_t matrix_lds_bytes(const LatentShape &s) { return (size_t)kMatrixChunk * (s.cache_row() + 8) * 2; }
bool matrix_supported(const LatentShape &s) { return s.cache_row() <= 24 * 32; }

// grid (ceil(vdim / 32), heads, rows): merges the key splits of a head, adds the sink to the denominator, applies W_uv.
__global__ __launch_bounds__(256) void latent_merge_kernel(LatentArgs a, int rankp, int vdimp, int splits, int chunk) {
    extern __shared__ float olat[];  // [4][rankp]: one quarter of the splits each, then their sum
    __shared__ float wt[kMaxSplits];
    const LatentShape &s = a.s;
    const int t = threadIdx.x, h = blockIdx.y, row = blockIdx.z;
    const int lane = t & 63, wave = t >> 6, sub = lane >> 4, kl = lane & 15;
    const size_t at = ((size_t)row * s.heads + h) * splits;
    const float *part_o = a.partial + at * rankp;
    const float *part_ml = a.partial + (size_t)gridDim.z * s.heads * splits * rankp + at * 2;
    // this thread's rows of W_uv, the first 512 columns: two rows of 16 lanes
    const uint16_t *wv = a.w.uv + ((size_t)h * vdimp + blockIdx.x * 32 + wave * 4 + sub) * rankp;
    uint4 first[2][4];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) first[i][j] = *(const uint4 *)(wv + (size_t)i * 16 * rankp + min(kl * 8 + 128 * j, rankp - 8));
    // every wave for itself: the weights of the splits
    // the splits that had keys
    const int chunks = (*a.pos_dev + row % a.new_len + chunk) / chunk, per = (chunks + splits - 1) / splits, used = (chunks + per - 1) / per;
    const float2 ml = lane < used ? *(const float2 *)(part_ml + 2 * lane) : make_float2(kMinusInf, 0.0f);
    const float sink = a.w.sink ? a.w.sink[h] : kMinusInf;
    const float top = fmaxf(wave_max(ml.x), sink);
    const float w = expf(ml.x - top);
    const float inv = 1.0f / (wave_sum(w * ml.y) + expf(sink - top));
    if (wave == 0) wt[lane] = w * inv;
    __syncthreads();
    for (int c = lane * 4; c < rankp; c += 256) {
        float4 v = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
#pragma unroll 4
        for (int i = wave; i < used; i += 4) {
            const float4 o = *(const float4 *)(part_o + (size_t)i * rankp + c);
            const float f = wt[i];
            v.x = fmaf(f, o.x, v.x);
            v.y = fmaf(f, o.y, v.y);
            v.z = fmaf(f, o.z, v.z);
            v.w = fmaf(f, o.w, v.w);
        }
        *(float4 *)(olat + wave * rankp + c) = v;
    }
    __syncthreads();
    for (int c = t; c < rankp; c += 256) olat[c] += olat[rankp + c] + olat[2 * rankp + c] + olat[3 * rankp + c];
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        float acc = 0.0f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int c = kl * 8 + 128 * j;
            const uint32_t u[4] = {first[i][j].x, first[i][j].y, first[i][j].z, first[i][j].w};
            float part = 0.0f;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                part = fmaf(__uint_as_float(u[e] << 16), olat[min(c, rankp - 8) + 2 * e], part);
                part = fmaf(__uint_as_float(u[e] & 0xffff0000u), olat[min(c, rankp - 8) + 2 * e + 1], part);
            }
            acc += c < rankp ? part : 0.0f;
        }
#pragma unroll 1
        for (int c = kl * 8 + 512; c < rankp; c += 128) {
            float v[8];
            load8(wv + (size_t)i * 16 * rankp + c, v);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc = fmaf(v[e], olat[c + e], acc);
        }
        acc = row16_sum(acc);
        const int dv = blockIdx.x * 32 + i * 16 + wave * 4 + sub;
        if (kl == 0 && dv < s.vdim) {
            const size_t o = (size_t)row * a.ldo + (size_t)h * s.vdim + dv;
            if (a.out_bf16) ((uint16_t *)a.out)[o] = f32_to_bf16(acc);
            else ((float *)a.out)[o] = acc;
        }
    }
}

// One workgroup per row: the cache row and the bf16 queries of every head.
__global__ __launch_bounds__(256) void latent_tiled_prepare_kernel(LatentArgs a, int rankp, int row_len, int dimp, int query_row) {
    __shared__ float red[4];
    const LatentShape &s = a.s;
    const int row = blockIdx.x, pos = *a.pos_dev + row % a.new_len;
    write_cache_row<uint16_t>(a, s, rankp, row_len, row, pos, red);
    const float2 *cs = a.w.rope + (size_t)pos * (s.rot_dims >> 1);
    const float *q = a.q + (size_t)row * a.ld;
    uint16_t *dst = a.qb + (size_t)row * s.heads * query_row;
    for (int i = threadIdx.x; i < s.heads * query_row; i += 256) {
        const int h = i / query_row, e = i % query_row;
        const float *qh = q + (size_t)h * (s.dim + s.rot);
        float v = 0.0f;
        if (e < s.dim) v = qh[e];
        else if (e >= dimp && e < dimp + s.rot) v = rotated(qh + s.dim, e - dimp, s.rot_dims, cs);
        dst[i] = f32_to_bf16(v);
    }
}

// One wave = 32 queries of a head; SPLIT: the four waves of a workgroup share one query block's key tiles (and merge),
// else each wave has its own query block.  DQ steps of 16 query dimensions, DV tiles of 32 value dimensions.
template <int DQ, int DV, bool SPLIT>
__global__ __launch_bounds__(256, 1) void latent_tiled_kernel(LatentArgs a, int rankp, int row_len, int rotp, int dimp, int vdimp, int query_row,
                                                              int kv_stride, int blocks) {
    extern __shared__ float shm[];
    const LatentShape &s = a.s;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, li = lane & 31, lh = lane >> 5;
    const int h = blockIdx.y, b = blockIdx.z, T = a.new_len;
    // late query blocks see the most keys: they start first
    const int qb = SPLIT ? blocks - 1 - (int)blockIdx.x : blocks - 1 - ((int)blockIdx.x * 4 + wave);
    const int kv = a.kv_max, pos = kv - T;
    const bool active = qb >= 0;
    const int q0 = (active ? qb : 0) * 32;
    const int qi = q0 + li;
    const int last_key = pos + min(q0 + 31, T - 1);
    const int tiles = active ? last_key / 32 + 1 : 0;
    const int ldk = s.heads * dimp;
    const uint16_t *qp = a.qb + ((size_t)(b * T + min(qi, T - 1)) * s.heads + h) * query_row;
    bf16x8 qf[DQ];
#pragma unroll
    for (int k = 0; k < DQ; ++k) {
        const int j = 2 * k + lh;
        qf[k] = __builtin_bit_cast(bf16x8, 8 * j < query_row ? *(const uint4 *)(qp + 8 * j) : make_uint4(0, 0, 0, 0));
    }
    f32x16 o[DV];
#pragma unroll
    for (int t = 0; t < DV; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[t][r] = 0.0f;
    float m = kMinusInf, l = 0.0f;
    const int key_of_row = 16 * ((li >> 2) & 1) + 4 * (li >> 3) + (li & 3);
    const uint16_t *kx = a.kx + (size_t)b * kv * ldk + (size_t)h * dimp;
    const uint16_t *kr = (const uint16_t *)a.cache + (size_t)b * a.positions * row_len + rankp;
    const uint16_t *vx = a.vx + ((size_t)b * s.heads + h) * vdimp * kv_stride;
    const int jn = dimp >> 3, jall = (dimp + rotp) >> 3;
    for (int tile = SPLIT ? wave : 0; tile < tiles; tile += SPLIT ? 4 : 1) {
        const int k0 = tile * 32;
        const int key = min(k0 + key_of_row, kv - 1);
        const uint16_t *kun = kx + (size_t)key * ldk, *krot = kr + (size_t)key * row_len;
        bf16x8 kf[DQ];
#pragma unroll
        for (int k = 0; k < DQ; ++k) {
            const int j = 2 * k + lh;
            const uint16_t *p = j < jn ? kun + 8 * j : krot + 8 * (j - jn);
            kf[k] = __builtin_bit_cast(bf16x8, j < jall ? *(const uint4 *)p : make_uint4(0, 0, 0, 0));
        }
        bf16x8 vf[DV][2];
#pragma unroll
        for (int t = 0; t < DV; ++t)
#pragma unroll
            for (int st = 0; st < 2; ++st) {
                const int dv = t * 32 + li;
                vf[t][st] = __builtin_bit_cast(
                    bf16x8, dv < vdimp ? *(const uint4 *)(vx + (size_t)dv * kv_stride + k0 + 16 * lh + 8 * st) : make_uint4(0, 0, 0, 0));
            }
        if (k0 + 32 > kv) {  // columns behind the last key hold nothing
#pragma unroll
            for (int t = 0; t < DV; ++t)
#pragma unroll
                for (int st = 0; st < 2; ++st)
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (k0 + 16 * lh + 8 * st + e >= kv) vf[t][st][e] = (__bf16)0.0f;
        }
        f32x16 sc;
#pragma unroll
        for (int r = 0; r < 16; ++r) sc[r] = 0.0f;
#pragma unroll
        for (int k = 0; k < DQ; ++k) sc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[k], qf[k], sc, 0, 0, 0);
        // register r of half lh: key k0 + 16 lh + r, query qi
        const int limit = pos + qi - (k0 + 16 * lh);  // keys r <= limit are visible
        float top = kMinusInf;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            sc[r] = r <= limit ? sc[r] * s.scale : kMinusInf;
            top = fmaxf(top, sc[r]);
        }
        top = fmaxf(top, __shfl_xor(top, 32));
        const float m_new = fmaxf(m, top);
        const float cr = __expf(m - m_new);
        m = m_new;
        float sum = 0.0f;
        bf16x8 pf[2];
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const float p = r <= limit ? __expf(sc[r] - m_new) : 0.0f;
            sum += p;
            pf[r >> 3][r & 7] = (__bf16)p;
        }
        l = l * cr + sum;
#pragma unroll
        for (int t = 0; t < DV; ++t) {
#pragma unroll
            for (int r = 0; r < 16; ++r) o[t][r] *= cr;
            o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[t][0], pf[0], o[t], 0, 0, 0);
            o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[t][1], pf[1], o[t], 0, 0, 0);
        }
    }
    l += __shfl_xor(l, 32);
    const float sink = a.w.sink ? a.w.sink[h] : kMinusInf;
    auto store4 = [&](int t, int g, const float (&v)[4]) {  // value dimensions t * 32 + 8 g + 4 lh .. + 3 of query qi
        if (!active || qi >= T) return;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int dv = t * 32 + 8 * g + 4 * lh + e;
            if (dv >= s.vdim) continue;
            const size_t at = (size_t)(b * T + qi) * a.ldo + (size_t)h * s.vdim + dv;
            if (a.out_bf16) ((uint16_t *)a.out)[at] = f32_to_bf16(v[e]);
            else ((float *)a.out)[at] = v[e];
        }
    };
    if (!SPLIT) {
        const float top = fmaxf(m, sink);
        const float f = __expf(m - top), inv = f / (l * f + expf(sink - top));
#pragma unroll
        for (int t = 0; t < DV; ++t)
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const float v[4] = {o[t][4 * g] * inv, o[t][4 * g + 1] * inv, o[t][4 * g + 2] * inv, o[t][4 * g + 3] * inv};
                store4(t, g, v);
            }
        return;
    }
    float *sm = shm, *sl = shm + 4 * 64, *so = shm + 8 * 64;  // [wave][lane], [wave][lane], [wave][DV * 16][64]
    sm[wave * 64 + lane] = m;
    sl[wave * 64 + lane] = l;
    __syncthreads();
    float top = sink;
#pragma unroll
    for (int w = 0; w < 4; ++w) top = fmaxf(top, sm[w * 64 + lane]);
    float den = expf(sink - top);
#pragma unroll
    for (int w = 0; w < 4; ++w) den += sl[w * 64 + lane] * __expf(sm[w * 64 + lane] - top);
    const float f = __expf(m - top) / den;
#pragma unroll
    for (int t = 0; t < DV; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) so[((size_t)wave * DV * 16 + t * 16 + r) * 64 + lane] = o[t][r] * f;
    __syncthreads();
#pragma unroll
    for (int t = 0; t < DV; ++t) {  // wave w finishes the registers 4 w .. 4 w + 3 of every tile
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            v[e] = 0.0f;
#pragma unroll
            for (int w = 0; w < 4; ++w) v[e] += so[((size_t)w * DV * 16 + t * 16 + 4 * wave + e) * 64 + lane];
        }
        store4(t, wave, v);
    }
}

template <typename CT>
int32_t attend_run(agpu_ctx *ctx, const LatentArgs &a, int rows, int splits) {
    const LatentShape &s = a.s;
    const dim3 grid((unsigned)splits, (unsigned)ceil_div(s.heads, kHeadTile), (unsigned)rows), block(256);
    const int ni = ceil_div(s.rankp(), 128);
    if (ni <= 1) hipLaunchKernelGGL((latent_attend_kernel<CT, 1>), grid, block, 0, ctx->stream, a, (const float *)a.qlat, s.rankp(), s.cache_row(), splits);
    else if (ni <= 2) hipLaunchKernelGGL((latent_attend_kernel<CT, 2>), grid, block, 0, ctx->stream, a, (const float *)a.qlat, s.rankp(), s.cache_row(), splits);
    else if (ni <= 4) hipLaunchKernelGGL((latent_attend_kernel<CT, 4>), grid, block, 0, ctx->stream, a, (const float *)a.qlat, s.rankp(), s.cache_row(), splits);
    else if (ni <= 8) hipLaunchKernelGGL((latent_attend_kernel<CT, 8>), grid, block, 0, ctx->stream, a, (const float *)a.qlat, s.rankp(), s.cache_row(), splits);
    else return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "latent_attention: latent size %d exceeds 1024", s.rank);
    return AGPU_LAUNCH_CHECK(ctx, "latent_attend_kernel");
}

template <int CT, int NK>
int32_t attend_matrix_run(agpu_ctx *ctx, const LatentArgs &a, int rows, int splits) {
    const LatentShape &s = a.s;
    const size_t lds = matrix_lds_bytes(s);
    if (lds > 48 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_attend_matrix_kernel<CT, NK>), hipFuncAttributeMaxDynamicSharedMemorySize, 148 * 1024);
    hipLaunchKernelGGL((latent_attend_matrix_kernel<CT, NK>), dim3((unsigned)splits, (unsigned)ceil_div(s.heads, kMatrixHeads), (unsigned)rows), dim3(256), lds,
                       ctx->stream, a, s.rankp(), s.cache_row(), splits);
    return AGPU_LAUNCH_CHECK(ctx, "latent_attend_matrix_kernel");
}

template <int DQ, int DV>
int32_t tiled_run(agpu_ctx *ctx, const LatentArgs &a) {
    const LatentShape &s = a.s;
    const int blocks = ceil_div(a.new_len, 32), kvs = latent_kv_stride(a.kv_max);
    const bool split = blocks * s.heads * a.batch < 8 * ctx->num_cus;
    if (split) {
        const size_t lds = (8 * 64 + (size_t)4 * DV * 16 * 64) * sizeof(float);
        if (lds > 64 * 1024)
            (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_tiled_kernel<DQ, DV, true>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                      160 * 1024);
        hipLaunchKernelGGL((latent_tiled_kernel<DQ, DV, true>), dim3((unsigned)blocks, (unsigned)s.heads, (unsigned)a.batch), dim3(256), lds, ctx->stream,
                           a, s.rankp(), s.cache_row(), s.rotp(), s.dimp(), s.vdimp(), s.query_row(), kvs, blocks);
    } else {
        hipLaunchKernelGGL((latent_tiled_kernel<DQ, DV, false>), dim3((unsigned)ceil_div(blocks, 4), (unsigned)s.heads, (unsigned)a.batch), dim3(256), 0,
                           ctx->stream, a, s.rankp(), s.cache_row(), s.rotp(), s.dimp(), s.vdimp(), s.query_row(), kvs, blocks);
    }
    return AGPU_LAUNCH_CHECK(ctx, "latent_tiled_kernel");
}

template <int DV>
int32_t tiled_run_dq(agpu_ctx *ctx, const LatentArgs &a) {
    const int dq = a.s.query_row() / 16;
    if (dq <= 4) return tiled_run<4, DV>(ctx, a);
    if (dq <= 8) return tiled_run<8, DV>(ctx, a);
    return tiled_run<12, DV>(ctx, a);
}

int32_t check_shape(agpu_ctx *ctx, const LatentArgs &a) {
    const LatentShape &s = a.s;
    if (s.heads <= 0 || s.dim <= 0 || s.rot < 0 || s.rot_dims > s.rot || s.rot_dims % 2 != 0 || s.vdim <= 0 || s.rank <= 0 || a.batch <= 0 ||
        a.new_len <= 0 || a.kv_max < a.new_len || a.kv_max > a.positions)
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "latent_attention: bad shape");
    if (s.dim > 1024 || s.rank > 1024) return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "latent_attention: head size %d or latent size %d exceeds 1024", s.dim, s.rank);
    return AGPU_OK;
}

}  // namespace

int latent_splits(const agpu_ctx *ctx, const LatentShape &s, int rows, int kv_max) {
    const int chunks = ceil_div(kv_max, kMatrixChunk), others = ceil_div(s.heads, kMatrixHeads) * rows;
    return std::max(1, std::min({chunks, kMaxSplits, ceil_div(2 * ctx->num_cus, others)}));
}

size_t latent_partial_floats(const LatentShape &s, int rows, int splits) { return (size_t)rows * s.heads * splits * (s.rankp() + 2); }

int32_t latent_absorbed_launch(agpu_ctx *ctx, const LatentArgs &a) {
    int32_t rc = check_shape(ctx, a);
    if (rc != AGPU_OK) return rc;
    const LatentShape &s = a.s;
    const int rows = a.batch * a.new_len, splits = latent_splits(ctx, s, rows, a.kv_max);
    const bool matrix = a.cache_bf16 && matrix_supported(s);
    const int col_blocks = ceil_div(s.rankp(), 128);
    const dim3 grid((unsigned)(1 + s.heads * col_blocks), (unsigned)rows), block(256);
#define AGPU_ABSORB(CT, QT) \
    hipLaunchKernelGGL((latent_absorb_kernel<CT, QT>), grid, block, 0, ctx->stream, a, s.rankp(), s.cache_row(), s.dimp(), col_blocks)
    if (matrix) AGPU_ABSORB(uint16_t, uint16_t);
    else if (a.cache_bf16) AGPU_ABSORB(uint16_t, float);
    else AGPU_ABSORB(float, float);
#undef AGPU_ABSORB
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "latent_absorb_kernel")) != AGPU_OK) return rc;
    if (matrix) {
        const int ct = ceil_div(s.rankp(), 64), nk = ceil_div(s.cache_row(), 128);
        if (ct <= 2 && nk <= 2) rc = attend_matrix_run<2, 2>(ctx, a, rows, splits);
        else if (ct <= 4 && nk <= 3) rc = attend_matrix_run<4, 3>(ctx, a, rows, splits);
        else if (ct <= 8 && nk <= 5) rc = attend_matrix_run<8, 5>(ctx, a, rows, splits);
        else rc = attend_matrix_run<12, 6>(ctx, a, rows, splits);
    } else {
        rc = a.cache_bf16 ? attend_run<uint16_t>(ctx, a, rows, splits) : attend_run<float>(ctx, a, rows, splits);
    }
    if (rc != AGPU_OK) return rc;
    hipLaunchKernelGGL(latent_merge_kernel, dim3((unsigned)(s.vdimp() / 32), (unsigned)s.heads, (unsigned)rows), dim3(256),
                       (size_t)4 * s.rankp() * sizeof(float), ctx->stream, a, s.rankp(), s.vdimp(), splits,
                       matrix ? kMatrixChunk : kKeyChunk);
    return AGPU_LAUNCH_CHECK(ctx, "latent_merge_kernel");
}

bool latent_tiled_supported(const LatentShape &s) { return s.query_row() <= 192 && s.vdim <= 128; }

int32_t latent_tiled_launch(agpu_ctx *ctx, const LatentArgs &a) {
    int32_t rc = check_shape(ctx, a);
    if (rc != AGPU_OK) return rc;
    const LatentShape &s = a.s;
    if (!a.cache_bf16 || !latent_tiled_supported(s)) return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "latent_attention: no tiled kernel for this shape");
    hipLaunchKernelGGL(latent_tiled_prepare_kernel, dim3((unsigned)(a.batch * a.new_len)), dim3(256), 0, ctx->stream, a, s.rankp(), s.cache_row(), s.dimp(),
                       s.query_row());
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "latent_tiled_prepare_kernel")) != AGPU_OK) return rc;
    const int kvs = latent_kv_stride(a.kv_max);
    for (int b = 0; b < a.batch; ++b) {
        const uint16_t *lat = (const uint16_t *)a.cache + (size_t)b * a.positions * s.cache_row();
        DenseOut ko;
        ko.n_plain = s.heads * s.dimp();
        ko.out_bf16 = a.kx + (size_t)b * a.kv_max * s.heads * s.dimp();
        ko.ldo = s.heads * s.dimp();
        if ((rc = dense_gemm_bf16_launch(ctx, lat, s.cache_row(), a.w.uk, s.rankp(), a.kv_max, s.heads * s.dimp(), s.rankp(), ko)) != AGPU_OK) return rc;
        DenseOut vo;  // transposed: one row per head and value dimension
        vo.n_plain = a.kv_max;
        vo.out_bf16 = a.vx + (size_t)b * s.heads * s.vdimp() * kvs;
        vo.ldo = kvs;
        if ((rc = dense_gemm_bf16_launch(ctx, a.w.uv, s.rankp(), lat, s.cache_row(), s.heads * s.vdimp(), a.kv_max, s.rankp(), vo)) != AGPU_OK) return rc;
    }
    const int dv = s.vdimp() / 32;
    if (dv <= 1) return tiled_run_dq<1>(ctx, a);
    if (dv <= 2) return tiled_run_dq<2>(ctx, a);
    return tiled_run_dq<4>(ctx, a);
}
