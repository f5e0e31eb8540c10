// Dense Linears over bf16 weights (dense_linear.h): the decode GEMV with its row prologue (normed addend, RMS norm), the
// K-split kernel for small batches, the tiled GEMMs, and the C entry points that run them.
//
// The matrix-core kernels use v_mfma_f32_32x32x16_bf16 / 16x16x32_bf16 / 32x32x2_f32.  Operand layout (32x32x16): lane l
// holds row (or column) l % 32, k = 8 (l / 32) .. + 7; result register r of lane l is row 8 (r / 4) + 4 (l / 32) + r % 4,
// column l % 32.
#include "dense_linear.h"

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

__device__ __forceinline__ void store_plain(const DenseOut &o, int m, int n, float v) {
    if (o.bias) v += o.bias[n];
    if (o.tab) {
        const uint32_t tok = min(o.tokens[m], (uint32_t)(o.vocab - 1));
        v = n < o.tab_n ? gelu_tanh_dev(v) * bf16_to_f32(o.tab[(size_t)tok * o.tab_ld + o.tab_off + n]) : 0.0f;
    }
    if (o.residual) v += o.residual[(size_t)m * o.ldr + n];
    if (o.out) o.out[(size_t)m * o.ldo + n] = v;
    if (o.out_bf16) o.out_bf16[(size_t)m * o.ldo + n] = f32_to_bf16(v);
}

__device__ __forceinline__ void store_pair(const DenseOut &o, int m, int j, float gate, float up) {
    float a;
    if (o.act_limit > 0.0f) a = gelu_quick_dev(fminf(gate, o.act_limit)) * (fminf(fmaxf(up, -o.act_limit), o.act_limit) + 1.0f);
    else a = silu_dev(gate) * up;
    if (o.act_bf16) ((uint16_t *)o.act)[(size_t)m * o.ld_act + j] = f32_to_bf16(a);
    else ((float *)o.act)[(size_t)m * o.ld_act + j] = a;
}

// Sum over the workgroup, result in every thread.  `red` holds one float per wave and may be reused after the call.
template <int NW>
__device__ __forceinline__ float block_sum(float v, float *red) {
    v = wave_sum(v);
    if (NW == 1) return v;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.0f;
#pragma unroll
    for (int i = 0; i < NW; ++i) s += red[i];
    return s;
}

// One row of DenseRows: h (and x2 behind it) goes through `put(k, value)`, k = 0 .. K - 1.  The first kRowRegs * NT columns
// of x and y are read once and stay in registers; a wider row reads the rest again in every pass.
constexpr int kRowRegs = 4;
enum RowKind { kRowPlain, kRowAdds, kRowGated };  // which parts of DenseRows a kernel has code for
template <int NW, int KIND, typename Put>
__device__ __forceinline__ void run_row(const DenseRows &in, int m, bool write_x, float *red, Put put) {
    constexpr int NT = NW * 64;
    const int t = threadIdx.x;
    const size_t row = (size_t)(in.map_stride > 0 ? in.map_stride * (m + 1) - 1 : m) * in.ldx;
    const float *x = in.x + row, *y = in.y ? in.y + row : nullptr;
    const float *add = KIND == kRowAdds && in.add ? in.add + row : nullptr, *add_vec = KIND == kRowAdds ? in.add_vec : nullptr;
    auto added = [&](int k) -> float { return (add ? add[k] : 0.0f) + (add_vec ? add_vec[k] : 0.0f); };
    float v[kRowRegs], yv[kRowRegs], yw[kRowRegs], nw[kRowRegs], v2[kRowRegs], av[kRowRegs];
#pragma unroll
    for (int i = 0; i < kRowRegs; ++i) {  // clamped addresses; columns beyond d count as zero
        const int k = t + i * NT, kc = min(k, in.d - 1);
        v[i] = x[kc];
        yv[i] = y ? y[kc] : 0.0f;
        yw[i] = y ? in.y_w[kc] : 0.0f;
        nw[i] = in.norm_w ? in.norm_w[kc] : 0.0f;
        v2[i] = in.x2 ? in.x2[row + min(k, in.dp - 1)] : 0.0f;
        av[i] = KIND == kRowAdds ? added(kc) : 0.0f;
    }
    float rs_y = 0.0f;
    if (y) {
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < kRowRegs; ++i) s += t + i * NT < in.d ? yv[i] * yv[i] : 0.0f;
#pragma unroll 1
        for (int k = t + kRowRegs * NT; k < in.d; k += NT) s += y[k] * y[k];
        s = block_sum<NW>(s, red);
        rs_y = 1.0f / sqrtf(s / (float)in.d + in.eps);
    }
#pragma unroll
    for (int i = 0; i < kRowRegs; ++i) v[i] = t + i * NT < in.d ? v[i] + yv[i] * rs_y * yw[i] + av[i] : 0.0f;
    auto value = [&](int k) -> float { return (y ? x[k] + y[k] * rs_y * in.y_w[k] : x[k]) + (KIND == kRowAdds ? added(k) : 0.0f); };
    float rs_x = 1.0f;
    if (in.norm_w) {
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < kRowRegs; ++i) s += v[i] * v[i];
#pragma unroll 1
        for (int k = t + kRowRegs * NT; k < in.d; k += NT) s += value(k) * value(k);
        s = block_sum<NW>(s, red);
        rs_x = 1.0f / sqrtf(s / (float)in.d + in.eps);
    }
    auto finish = [&](int k, float a, float w, float b) {
        if (write_x) in.x_out[row + k] = a;
        put(k, in.norm_w ? a * rs_x * (in.norm_off + w) : a);
        if (in.x2) put(in.dp + k, b);
    };
#pragma unroll
    for (int i = 0; i < kRowRegs; ++i)
        if (t + i * NT < in.dp) finish(t + i * NT, v[i], nw[i], v2[i]);
#pragma unroll 1
    for (int k = t + kRowRegs * NT; k < in.dp; k += NT)
        finish(k, k < in.d ? value(k) : 0.0f, in.norm_w && k < in.d ? in.norm_w[k] : 0.0f, in.x2 ? in.x2[row + k] : 0.0f);
}

// One gated row of DenseRows, a wave per group.
template <int NW, typename Put>
__device__ __forceinline__ void run_gated_row(const DenseRows &in, int m, Put put) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const size_t r = (size_t)(in.map_stride > 0 ? in.map_stride * (m + 1) - 1 : m);
#pragma unroll 1
    for (int g = wave; g < in.groups; g += NW) {
        const float *x = in.x + r * in.ldx + g * in.group_p, *gate = in.gate + r * in.ld_gate + g * in.group_p, *w = in.norm_w + g * in.group_p;
        float v[kRowRegs], gv[kRowRegs], wv[kRowRegs], s = 0.0f;
#pragma unroll
        for (int i = 0; i < kRowRegs; ++i) {
            const int k = lane + 64 * i, kc = min(k, in.group_p - 1);
            v[i] = k < in.group_p ? x[kc] : 0.0f;
            gv[i] = gate[kc];
            wv[i] = w[kc];
            s = fmaf(v[i], v[i], s);
        }
#pragma unroll 1
        for (int k = lane + 64 * kRowRegs; k < in.group_p; k += 64) s = fmaf(x[k], x[k], s);
        const float rs = 1.0f / sqrtf(wave_sum(s) / (float)in.group_d + in.eps);
#pragma unroll
        for (int i = 0; i < kRowRegs; ++i)
            if (lane + 64 * i < in.group_p) put(g * in.group_p + lane + 64 * i, v[i] * rs * wv[i] * sigmoid_dev(gv[i]));
#pragma unroll 1
        for (int k = lane + 64 * kRowRegs; k < in.group_p; k += 64) put(g * in.group_p + k, x[k] * rs * w[k] * sigmoid_dev(gate[k]));
    }
}

// ---- decode GEMV: a wave takes 4 * RPL weight rows, 16 lanes x 8 values along K per row and chunk of 128; the waves of a
// workgroup split K KS ways.  The first weights are requested before the rows are touched.
constexpr int kGemvWaves = 8;

template <int MT, int RPL, int KIND>
__global__ __launch_bounds__(64 * kGemvWaves) void dense_gemv_kernel(DenseRows in, const uint16_t *__restrict__ w, int M, int N, int K, int KS,
                                                                     DenseOut o) {
    extern __shared__ float lds[];
    constexpr int U = RPL == 1 ? 4 : 2;
    float *xs = lds;                              // [MT][K]
    float *red = lds + (size_t)MT * K;            // [KS][rows of the workgroup][MT]
    float *wred = red + kGemvWaves * 4 * RPL * MT;  // one float per wave
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, sub = lane >> 4, kl = lane & 15;
    const int wk = wave % KS, wr = wave / KS;
    const int rows = 4 * RPL * (kGemvWaves / KS);
    const int n0 = blockIdx.x * rows;
    const int nchunks = (K + 127) >> 7;
    uint4 next[U][RPL];
    auto request = [&](int base) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = (base + u * KS) * 128 + kl * 8;
#pragma unroll
            for (int i = 0; i < RPL; ++i) {
                const int n = n0 + wr * 4 * RPL + i * 4 + sub;
                next[u][i] = (k < K && n < N) ? *(const uint4 *)(w + (size_t)n * K + k) : make_uint4(0, 0, 0, 0);
            }
        }
    };
    request(wk);
#pragma unroll 1
    for (int m = 0; m < MT; ++m) {
        float *xm = xs + (size_t)m * K;
        if (m < M) {
            if (KIND == kRowGated) {
                run_gated_row<kGemvWaves>(in, m, [&](int k, float v) { xm[k] = v; });
            } else if (KIND == kRowAdds || in.y || in.norm_w) {
                run_row<kGemvWaves, KIND>(in, m, in.x_out != nullptr && blockIdx.x == 0, wred, [&](int k, float v) { xm[k] = v; });
            } else {
                const size_t row = (size_t)(in.map_stride > 0 ? in.map_stride * (m + 1) - 1 : m) * in.ldx;
                for (int k = threadIdx.x * 4; k < in.dp; k += 256 * kGemvWaves) {
                    *(float4 *)(xm + k) = *(const float4 *)(in.x + row + k);
                    if (in.x2) *(float4 *)(xm + in.dp + k) = *(const float4 *)(in.x2 + row + k);
                }
            }
        } else {
            for (int k = threadIdx.x; k < K; k += 64 * kGemvWaves) xm[k] = 0.0f;
        }
    }
    __syncthreads();
    float acc[MT][RPL];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int i = 0; i < RPL; ++i) acc[m][i] = 0.0f;
    for (int base = wk; base < nchunks; base += U * KS) {
        uint4 cur[U][RPL];
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int i = 0; i < RPL; ++i) cur[u][i] = next[u][i];
        if (base + U * KS < nchunks) request(base + U * KS);
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = min((base + u * KS) * 128 + kl * 8, K - 8);  // beyond K the weights are zero
            float xv[MT][8];
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                *(float4 *)&xv[m][0] = *(const float4 *)(xs + (size_t)m * K + k);
                *(float4 *)&xv[m][4] = *(const float4 *)(xs + (size_t)m * K + k + 4);
            }
#pragma unroll
            for (int i = 0; i < RPL; ++i) {
                const uint32_t q[4] = {cur[u][i].x, cur[u][i].y, cur[u][i].z, cur[u][i].w};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float lo = __uint_as_float(q[e] << 16), hi = __uint_as_float(q[e] & 0xffff0000u);
#pragma unroll
                    for (int m = 0; m < MT; ++m) {
                        acc[m][i] = fmaf(lo, xv[m][2 * e], acc[m][i]);
                        acc[m][i] = fmaf(hi, xv[m][2 * e + 1], acc[m][i]);
                    }
                }
            }
        }
    }
#pragma unroll
    for (int i = 0; i < RPL; ++i) {
        const int r = wr * 4 * RPL + i * 4 + sub;
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            const float s = row16_sum(acc[m][i]);
            if (kl == 0) red[((size_t)wk * rows + r) * MT + m] = s;
        }
    }
    __syncthreads();
    auto total = [&](int r, int m) {
        float s = 0.0f;
        for (int k = 0; k < KS; ++k) s += red[((size_t)k * rows + r) * MT + m];
        return s;
    };
    for (int t = threadIdx.x; t < rows * MT; t += 64 * kGemvWaves) {
        const int r = t / MT, m = t % MT, n = n0 + r;
        if (m >= M || n >= N) continue;
        if (n < o.n_plain) store_plain(o, m, n, total(r, m));
        else if (((n - o.n_plain) & 1) == 0) store_pair(o, m, (n - o.n_plain) >> 1, total(r, m), total(r + 1, m));
    }
}

template <int NW, int KIND>
__global__ __launch_bounds__(64 * NW) void dense_rows_kernel(DenseRows in, void *h, int ldh, int h_bf16) {
    __shared__ float red[NW];
    const int m = blockIdx.x;
    auto put = [&](int k, float v) {
        if (!h) return;
        if (h_bf16) ((uint16_t *)h)[(size_t)m * ldh + k] = f32_to_bf16(v);
        else ((float *)h)[(size_t)m * ldh + k] = v;
    };
    if (KIND == kRowGated) run_gated_row<NW>(in, m, put);
    else run_row<NW, KIND>(in, m, in.x_out != nullptr, red, put);
}

// ---- few rows or few columns: 16 columns and up to 32 rows per workgroup, the waves split K, operands straight from memory ----
template <int RT, int kSkinnyWaves>  // row tiles of 16, waves
__global__ __launch_bounds__(64 * kSkinnyWaves) void dense_skinny_kernel(const uint16_t *__restrict__ a, int lda, const uint16_t *__restrict__ w,
                                                                         int ldw, int M, int N, int K, DenseOut o) {
    __shared__ float red[kSkinnyWaves][RT][16][17];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, rc = lane & 15, kq = lane >> 4;
    const int n0 = blockIdx.x * 16, m0 = blockIdx.y * 16 * RT;
    const uint16_t *wp = w + (size_t)min(n0 + rc, N - 1) * ldw;
    const uint16_t *ap[RT];
#pragma unroll
    for (int t = 0; t < RT; ++t) ap[t] = a + (size_t)min(m0 + t * 16 + rc, M - 1) * lda;
    f32x4 acc[RT];
#pragma unroll
    for (int t = 0; t < RT; ++t) acc[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    const int steps = K >> 5;
    constexpr int U = 4;
    for (int s0 = wave; s0 < steps; s0 += U * kSkinnyWaves) {
        uint4 bw[U], aw[U][RT];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int s = s0 + u * kSkinnyWaves, k = s * 32 + kq * 8;
            const bool on = s < steps;
            bw[u] = on ? *(const uint4 *)(wp + k) : make_uint4(0, 0, 0, 0);
#pragma unroll
            for (int t = 0; t < RT; ++t) aw[u][t] = on ? *(const uint4 *)(ap[t] + k) : make_uint4(0, 0, 0, 0);
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int t = 0; t < RT; ++t)
                acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, aw[u][t]), __builtin_bit_cast(bf16x8, bw[u]), acc[t], 0, 0, 0);
    }
    // 16x16 result: register r of lane l is row 4 (l / 16) + r, column l % 16
#pragma unroll
    for (int t = 0; t < RT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) red[wave][t][kq * 4 + r][rc] = acc[t][r];
    __syncthreads();
    for (int i = threadIdx.x; i < RT * 256; i += 64 * kSkinnyWaves) {
        const int t = i >> 8, r = (i >> 4) & 15, c = i & 15, m = m0 + t * 16 + r, n = n0 + c;
        if (m >= M || n >= N) continue;
        auto total = [&](int col) {
            float s = 0.0f;
#pragma unroll
            for (int k = 0; k < kSkinnyWaves; ++k) s += red[k][t][r][col];
            return s;
        };
        if (n < o.n_plain) store_plain(o, m, n, total(c));
        else if (((n - o.n_plain) & 1) == 0) store_pair(o, m, (n - o.n_plain) >> 1, total(c), total(c + 1));
    }
}

// Results of one 32 x 32 tile (rows m0.., columns n0..) of a wave: through the wave's own piece of LDS, so that a store
// covers two whole rows of the tile and a gate meets its up.
constexpr int kTileLd = 33;
__device__ __forceinline__ void store_tile(const DenseOut &o, const f32x16 &c, float *tile, int m0, int n0, int M, int N, int lane) {
    const int lr = lane & 31, lh = lane >> 5;
#pragma unroll
    for (int r = 0; r < 16; ++r) tile[(8 * (r >> 2) + 4 * lh + (r & 3)) * kTileLd + lr] = c[r];
    __builtin_amdgcn_wave_barrier();  // LDS operations of one wave complete in order
    if (n0 + 31 < o.n_plain) {
        const int n = n0 + lr;
#pragma unroll 1
        for (int r = lh; r < 32; r += 2)
            if (m0 + r < M && n < N) store_plain(o, m0 + r, n, tile[r * kTileLd + lr]);
    } else {
        const int n = n0 + 2 * (lane & 15);  // a pair of columns per lane, four rows at a time
#pragma unroll 1
        for (int r = lane >> 4; r < 32; r += 4) {
            if (m0 + r >= M || n >= N) continue;
            const float u = tile[r * kTileLd + 2 * (lane & 15)], v = tile[r * kTileLd + 2 * (lane & 15) + 1];
            if (n >= o.n_plain) {
                store_pair(o, m0 + r, (n - o.n_plain) >> 1, u, v);
            } else {
                store_plain(o, m0 + r, n, u);
                if (n + 1 < N && n + 1 < o.n_plain) store_plain(o, m0 + r, n + 1, v);
            }
        }
    }
    __builtin_amdgcn_wave_barrier();
}

// ---- tiled bf16 GEMM: BM x BN per workgroup of WM x WN waves, 64 k per step, two LDS buffers, 16-byte chunks of a row
// rotated by row % 8 against bank conflicts.  With KG > 1 there are KG such groups of waves, which take the K steps in turn
// (each with its own buffers) and add their results up in LDS at the end ----
template <int BM, int BN, int WM, int WN, int KG>
__global__ __launch_bounds__(64 * WM * WN * KG) void dense_gemm_bf16_kernel(const uint16_t *__restrict__ a, int lda, const uint16_t *__restrict__ w,
                                                                      int ldw, int M, int N, int K, int tiles_n, DenseOut o) {
    constexpr int NT = 64 * WM * WN, TM = BM / WM / 32, TN = BN / WN / 32;
    constexpr int CA = BM * 8 / NT, CB = BN * 8 / NT;  // 16-byte chunks per thread and step
    extern __shared__ uint4 shm[];  // per group both operands twice; then the groups' results and the waves' result tiles
    constexpr int GROUP = 2 * (BM + BN) * 8;
    static_assert(GROUP * 16 >= 4 * WM * WN * 32 * kTileLd && GROUP * 16 >= 4 * BM * BN, "the results fit the operand buffers");
    const int lane = threadIdx.x & 63, wave = (threadIdx.x % NT) >> 6, wm = wave / WN, wn = wave % WN;
    const int tid = threadIdx.x % NT, group = threadIdx.x / NT;
    uint4 *sab = shm + group * GROUP;
    // workgroups b, b + 8, ... share an XCD: give each XCD a contiguous run of row tiles so that W tiles stay in its L2
    const int nb = gridDim.x;
    int b = blockIdx.x;
    if (nb >= 64) {
        const int per = nb / 8, rem = nb % 8, x = b % 8, i = b / 8;
        b = x * per + min(x, rem) + i;
    }
    const int m0 = (b / tiles_n) * BM, n0 = (b % tiles_n) * BN;
    uint4 ra[CA], rb[CB];
    auto request = [&](int k0) {
#pragma unroll
        for (int i = 0; i < CA; ++i) {
            const int c = tid + i * NT, r = c >> 3, k = k0 + (c & 7) * 8;
            ra[i] = k < K ? *(const uint4 *)(a + (size_t)min(m0 + r, M - 1) * lda + k) : make_uint4(0, 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < CB; ++i) {
            const int c = tid + i * NT, r = c >> 3, k = k0 + (c & 7) * 8;
            rb[i] = k < K ? *(const uint4 *)(w + (size_t)min(n0 + r, N - 1) * ldw + k) : make_uint4(0, 0, 0, 0);
        }
    };
    auto stage = [&](int buf) {
#pragma unroll
        for (int i = 0; i < CA; ++i) {
            const int c = tid + i * NT, r = c >> 3;
            sab[buf * BM * 8 + r * 8 + ((c & 7) ^ (r & 7))] = ra[i];
        }
#pragma unroll
        for (int i = 0; i < CB; ++i) {
            const int c = tid + i * NT, r = c >> 3;
            sab[2 * BM * 8 + buf * BN * 8 + r * 8 + ((c & 7) ^ (r & 7))] = rb[i];
        }
    };
    f32x16 acc[TM][TN];
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int j = 0; j < TN; ++j)
#pragma unroll
            for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.0f;
    request(group * 64);
    stage(0);
    __syncthreads();
    const int lr = lane & 31, lh = lane >> 5;
    int buf = 0;
    for (int k0 = 0; k0 < K; k0 += 64 * KG, buf ^= 1) {  // a group past K works on zeros
        const bool more = k0 + 64 * KG < K;
        if (more) request(k0 + (KG + group) * 64);
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            bf16x8 av[TM], bv[TN];
#pragma unroll
            for (int i = 0; i < TM; ++i) {
                const int r = wm * (BM / WM) + i * 32 + lr;
                av[i] = __builtin_bit_cast(bf16x8, sab[buf * BM * 8 + r * 8 + ((s * 2 + lh) ^ (r & 7))]);
            }
#pragma unroll
            for (int j = 0; j < TN; ++j) {
                const int r = wn * (BN / WN) + j * 32 + lr;
                bv[j] = __builtin_bit_cast(bf16x8, sab[2 * BM * 8 + buf * BN * 8 + r * 8 + ((s * 2 + lh) ^ (r & 7))]);
            }
#pragma unroll
            for (int i = 0; i < TM; ++i)
#pragma unroll
                for (int j = 0; j < TN; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(av[i], bv[j], acc[i][j], 0, 0, 0);
        }
        if (more) stage(buf ^ 1);
        __syncthreads();
    }
    if (KG > 1) {
        float *mine = (float *)sab + wave * TM * TN * 1024 + lane;
        if (group > 0) {
#pragma unroll
            for (int i = 0; i < TM; ++i)
#pragma unroll
                for (int j = 0; j < TN; ++j)
#pragma unroll
                    for (int r = 0; r < 16; ++r) mine[((i * TN + j) * 16 + r) * 64] = acc[i][j][r];
        }
        __syncthreads();
        if (group > 0) return;
        for (int g = 1; g < KG; ++g) {
            const float *other = mine + (size_t)g * GROUP * 4;
#pragma unroll
            for (int i = 0; i < TM; ++i)
#pragma unroll
                for (int j = 0; j < TN; ++j)
#pragma unroll
                    for (int r = 0; r < 16; ++r) acc[i][j][r] += other[((i * TN + j) * 16 + r) * 64];
        }
    }
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int j = 0; j < TN; ++j)
            store_tile(o, acc[i][j], (float *)sab + wave * 32 * kTileLd, m0 + wm * (BM / WM) + i * 32, n0 + wn * (BN / WN) + j * 32, M, N, lane);
}

// ---- fp32 rows: 64 x 64 per workgroup of 2 x 2 waves, 32 k per step; the halves of a wave take k 0 .. 15 and 16 .. 31 ----
__global__ __launch_bounds__(256) void dense_gemm_f32_kernel(const float *__restrict__ a, int lda, const uint16_t *__restrict__ w, int ldw, int M,
                                                             int N, int K, int tiles_n, DenseOut o) {
    constexpr int LD = 36;  // floats per staged row: 144 bytes
    __shared__ float sab[2 * 64 * LD];  // the operands, then the waves' result tiles
    float *sa = sab, *sb = sab + 64 * LD;
    static_assert(2 * 64 * LD >= 4 * 32 * kTileLd, "the result tiles fit the operand buffers");
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, wm = wave >> 1, wn = wave & 1;
    const int m0 = (blockIdx.x / tiles_n) * 64, n0 = (blockIdx.x % tiles_n) * 64;
    if (blockIdx.y > 0) {  // block of a block-diagonal Linear: plain outputs only
        a += (size_t)blockIdx.y * K;
        w += (size_t)blockIdx.y * N * ldw;
        if (o.out) o.out += (size_t)blockIdx.y * N;
        if (o.out_bf16) o.out_bf16 += (size_t)blockIdx.y * N;
        if (o.bias) o.bias += (size_t)blockIdx.y * N;
        if (o.residual) o.residual += (size_t)blockIdx.y * N;
    }
    f32x16 acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.0f;
    const int row = threadIdx.x >> 2, q = (threadIdx.x & 3) * 8;
    const float *ap = a + (size_t)min(m0 + row, M - 1) * lda + q;
    const uint16_t *wp = w + (size_t)min(n0 + row, N - 1) * ldw + q;
    for (int k0 = 0; k0 < K; k0 += 32) {
        const float4 a0 = *(const float4 *)(ap + k0), a1 = *(const float4 *)(ap + k0 + 4);
        const uint4 wv = *(const uint4 *)(wp + k0);
        __syncthreads();
        *(float4 *)(sa + row * LD + q) = a0;
        *(float4 *)(sa + row * LD + q + 4) = a1;
        const uint32_t u[4] = {wv.x, wv.y, wv.z, wv.w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            sb[row * LD + q + 2 * e] = __uint_as_float(u[e] << 16);
            sb[row * LD + q + 2 * e + 1] = __uint_as_float(u[e] & 0xffff0000u);
        }
        __syncthreads();
        const float *ar = sa + (wm * 32 + (lane & 31)) * LD + (lane >> 5) * 16;
        const float *br = sb + (wn * 32 + (lane & 31)) * LD + (lane >> 5) * 16;
#pragma unroll
        for (int s = 0; s < 16; s += 4) {
            const float4 av = *(const float4 *)(ar + s), bv = *(const float4 *)(br + s);
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av.x, bv.x, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av.y, bv.y, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av.z, bv.z, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av.w, bv.w, acc, 0, 0, 0);
        }
    }
    __syncthreads();
    store_tile(o, acc, sab + wave * 32 * kTileLd, m0 + wm * 32, n0 + wn * 32, M, N, lane);
}

size_t gemv_lds_bytes(int MT, int RPL, int K) { return ((size_t)MT * K + (size_t)kGemvWaves * 4 * RPL * MT + kGemvWaves) * sizeof(float); }

template <int MT, int RPL, int KIND>
int32_t gemv_run(agpu_ctx *ctx, const DenseRows &in, const uint16_t *w, int M, int N, int K, int KS, const DenseOut &o) {
    const int rows = 4 * RPL * (kGemvWaves / KS);
    const size_t lds = gemv_lds_bytes(MT, RPL, K);
    if (lds > 64 * 1024) {
        static bool raised = false;  // per instantiation; setting it twice is harmless
        if (!raised) {
            (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&dense_gemv_kernel<MT, RPL, KIND>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                      160 * 1024);
            raised = true;
        }
    }
    hipLaunchKernelGGL((dense_gemv_kernel<MT, RPL, KIND>), dim3((unsigned)ceil_div(N, rows)), dim3(64 * kGemvWaves), lds, ctx->stream, in, w, M, N, K, KS, o);
    return AGPU_LAUNCH_CHECK(ctx, "dense_gemv_kernel");
}

RowKind row_kind(const DenseRows &in) { return in.gate ? kRowGated : (in.add || in.add_vec ? kRowAdds : kRowPlain); }

template <int MT, int RPL>
int32_t gemv_run_kind(agpu_ctx *ctx, const DenseRows &in, const uint16_t *w, int M, int N, int K, int KS, const DenseOut &o) {
    switch (row_kind(in)) {
        case kRowGated: return gemv_run<MT, RPL, kRowGated>(ctx, in, w, M, N, K, KS, o);
        case kRowAdds: return gemv_run<MT, RPL, kRowAdds>(ctx, in, w, M, N, K, KS, o);
        default: return gemv_run<MT, RPL, kRowPlain>(ctx, in, w, M, N, K, KS, o);
    }
}

template <int KIND>
void rows_run(agpu_ctx *ctx, const DenseRows &in, int M, void *h, int ldh, int h_bf16) {
    const dim3 grid((unsigned)M);
    if (in.dp <= 256) hipLaunchKernelGGL((dense_rows_kernel<1, KIND>), grid, dim3(64), 0, ctx->stream, in, h, ldh, h_bf16);
    else if (in.dp <= 1024) hipLaunchKernelGGL((dense_rows_kernel<4, KIND>), grid, dim3(256), 0, ctx->stream, in, h, ldh, h_bf16);
    else hipLaunchKernelGGL((dense_rows_kernel<8, KIND>), grid, dim3(512), 0, ctx->stream, in, h, ldh, h_bf16);
}

template <int BM, int BN, int WM, int WN, int KG>
void gemm_run(agpu_ctx *ctx, const uint16_t *a, int lda, const uint16_t *w, int ldw, int M, int N, int K, const DenseOut &o) {
    constexpr size_t lds = (size_t)KG * 2 * (BM + BN) * 8 * 16;
    if (lds > 64 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void *>(&dense_gemm_bf16_kernel<BM, BN, WM, WN, KG>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                  (int)lds);
    const int tn = ceil_div(N, BN);
    hipLaunchKernelGGL((dense_gemm_bf16_kernel<BM, BN, WM, WN, KG>), dim3((unsigned)(ceil_div(M, BM) * tn)), dim3(64 * WM * WN * KG), lds, ctx->stream, a,
                       lda, w, ldw, M, N, K, tn, o);
}

}  // namespace

bool dense_gemv_supported(int M, int K) {
    const int MT = M <= 1 ? 1 : (M <= 2 ? 2 : 4);
    return M >= 1 && M <= kDenseGemvRows && gemv_lds_bytes(MT, 2, K) <= 150 * 1024;
}

int32_t dense_gemv_launch(agpu_ctx *ctx, const DenseRows &in, const uint16_t *w, int M, int N, int K, const DenseOut &o) {
    if (!dense_gemv_supported(M, K) || K % 32 != 0 || in.dp % 32 != 0 || K != in.dp * (in.x2 ? 2 : 1) || (in.x_out && in.x_out == in.x) ||
        (in.gate && (in.groups * in.group_p != K || !in.norm_w)))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "dense_gemv: M %d, N %d, K %d, dp %d not supported", M, N, K, in.dp);
    // K is split over the waves until the workgroups roughly fill the chip twice or a wave's share is one request
    const int nchunks = (K + 127) / 128;
    const bool wide = N >= 16384;
    const int rpl = wide ? 2 : 1;
    int KS = 8;
    while (KS > 1 && (ceil_div(N, 4 * rpl * (kGemvWaves / KS)) > 1024 || nchunks < KS)) KS /= 2;
    if (M == 1) return wide ? gemv_run_kind<1, 2>(ctx, in, w, M, N, K, KS, o) : gemv_run_kind<1, 1>(ctx, in, w, M, N, K, KS, o);
    if (M == 2) return wide ? gemv_run_kind<2, 2>(ctx, in, w, M, N, K, KS, o) : gemv_run_kind<2, 1>(ctx, in, w, M, N, K, KS, o);
    return wide ? gemv_run_kind<4, 2>(ctx, in, w, M, N, K, KS, o) : gemv_run_kind<4, 1>(ctx, in, w, M, N, K, KS, o);
}

int32_t dense_rows_launch(agpu_ctx *ctx, const DenseRows &in, int M, void *h, int ldh, int h_bf16) {
    if (in.gate && (in.groups * in.group_p != in.dp || !in.norm_w)) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "dense_rows: bad groups");
    switch (row_kind(in)) {
        case kRowGated: rows_run<kRowGated>(ctx, in, M, h, ldh, h_bf16); break;
        case kRowAdds: rows_run<kRowAdds>(ctx, in, M, h, ldh, h_bf16); break;
        default: rows_run<kRowPlain>(ctx, in, M, h, ldh, h_bf16);
    }
    return AGPU_LAUNCH_CHECK(ctx, "dense_rows_kernel");
}

int32_t dense_gemm_bf16_launch(agpu_ctx *ctx, const uint16_t *a, int lda, const uint16_t *w, int ldw, int M, int N, int K, const DenseOut &o) {
    if (M <= 0 || N <= 0 || K <= 0 || K % 32 != 0 || lda % 8 != 0 || ldw % 8 != 0 || (o.n_plain < N && (o.n_plain % 2 != 0 || N % 2 != 0)))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "dense_gemm: M %d, N %d, K %d, lda %d, ldw %d not supported", M, N, K, lda, ldw);
    auto tiles = [&](int bm, int bn) { return ceil_div(M, bm) * ceil_div(N, bn); };
    if (M <= kDenseSkinnyRows || 2 * tiles(32, 64) < ctx->num_cus) {
        const dim3 grid((unsigned)ceil_div(N, 16), (unsigned)ceil_div(M, 32));
        // fewer workgroups than CUs and a long K: more waves each, for more requests in flight per CU
        const bool deep = (int)(grid.x * grid.y) <= ctx->num_cus && K >= 2048;
#define AGPU_SKINNY(RT, NW) hipLaunchKernelGGL((dense_skinny_kernel<RT, NW>), grid, dim3(64 * NW), 0, ctx->stream, a, lda, w, ldw, M, N, K, o)
        if (M <= 16) {
            if (deep) AGPU_SKINNY(1, 16);
            else AGPU_SKINNY(1, 8);
        } else {
            if (deep) AGPU_SKINNY(2, 16);
            else AGPU_SKINNY(2, 8);
        }
#undef AGPU_SKINNY
        return AGPU_LAUNCH_CHECK(ctx, "dense_skinny_kernel");
    }
    if (tiles(128, 128) >= ctx->num_cus) gemm_run<128, 128, 2, 2, 1>(ctx, a, lda, w, ldw, M, N, K, o);
    else if (M > 256 && tiles(128, 64) >= ctx->num_cus) gemm_run<128, 64, 2, 2, 2>(ctx, a, lda, w, ldw, M, N, K, o);
    else if (tiles(64, 64) >= ctx->num_cus) gemm_run<64, 64, 2, 2, 2>(ctx, a, lda, w, ldw, M, N, K, o);
    else gemm_run<32, 64, 1, 2, 4>(ctx, a, lda, w, ldw, M, N, K, o);
    return AGPU_LAUNCH_CHECK(ctx, "dense_gemm_bf16_kernel");
}

int32_t dense_gemm_f32_launch(agpu_ctx *ctx, const float *a, int lda, const uint16_t *w, int ldw, int M, int N, int K, const DenseOut &o, int blocks) {
    if (blocks < 1 || (blocks > 1 && (o.n_plain < N || o.tab)) || M <= 0 || N <= 0 || K <= 0 || K % 32 != 0 || lda % 4 != 0 || ldw % 8 != 0 || (o.n_plain < N && (o.n_plain % 2 != 0 || N % 2 != 0)))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "dense_gemm_f32: M %d, N %d, K %d, lda %d, ldw %d not supported", M, N, K, lda, ldw);
    const int tn = ceil_div(N, 64);
    hipLaunchKernelGGL(dense_gemm_f32_kernel, dim3((unsigned)(ceil_div(M, 64) * tn), (unsigned)blocks), dim3(256), 0, ctx->stream, a, lda, w, ldw, M, N,
                       K, tn, o);
    return AGPU_LAUNCH_CHECK(ctx, "dense_gemm_f32_kernel");
}
