// Gated delta rule (gated_delta.h).  The columns of a head's state evolve independently given q, k, g and beta, so the
// recurrence over a prompt runs token by token with the state in registers: a column is spread over 32 lanes, a wave
// holds two, and the token vectors come through LDS in chunks.  With S the state before the token,
//   S^T diag(g) k and S^T diag(g) q are summed together, u = beta (v - S^T diag(g) k),
//   o = S^T diag(g) q + (k . q) u      (the read-out of the updated state), S <- diag(g) S + k u^T,
// so only one reduction over lanes sits between a token and the next.
#include "gated_delta.h"
#include "short_conv.h"

namespace {

constexpr int kMaxDim = 256;
constexpr int kChunk = 16;  // tokens staged at a time
constexpr int kRecWaves = 4;

__device__ __forceinline__ float softplus_dev(float v) { return fmaxf(v, 0.0f) + log1pf(expf(-fabsf(v))); }
__device__ __forceinline__ float decay_dev(float a_log, float step) { return expf(-expf(a_log) * softplus_dev(step)); }

__device__ __forceinline__ ShortConv conv_of(const DeltaArgs &a, int channels) {
    return ShortConv{a.proj, a.ld, a.ring, a.w.conv, channels, a.s.taps, a.new_len};
}

constexpr int kPrepareWidth = 256;  // channels of v or g per workgroup

// grid (groups of kConvTokens tokens, parts, batch): the first parts take two heads of q and k each (convolution, unit vectors), then
// come parts of v (convolution), then parts of g (decays; the first of them also the step sizes).  q, k and g of a head leave
// side by side, in padded rows.
__global__ __launch_bounds__(256) void delta_prepare_kernel(DeltaArgs a, int channels, int head_row, int qk_parts, int v_parts) {
    extern __shared__ float sx[];  // [2 heads][q, k][kConvTokens][head_row]
    const DeltaShape &s = a.s;
    const int b = blockIdx.z, T = a.new_len, t0 = blockIdx.x * kConvTokens, nt = min(kConvTokens, T - t0), pos = *a.pos_dev, pos_slot = pos % s.taps;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int nk = s.kv_heads * s.dim, nv = s.heads * s.vdim, nb = s.heads + s.kv_heads;
    const size_t row0 = (size_t)b * T + t0;
    const ShortConv conv = conv_of(a, channels);
    int part = blockIdx.y;
    if (part < qk_parts) {
        const int per = kConvTokens * head_row;
#pragma unroll 1
        for (int i = t; i < 4 * head_row; i += 256) {
            const int w = i / head_row, d = i % head_row, h = min(part * 2 + (w >> 1), s.kv_heads - 1), c = h * s.dim + min(d, s.dim - 1);
            short_conv_run(conv, b, pos, pos_slot, t0, (w & 1) * nk + c, ((w & 1) ? a.col_k : a.col_q) + c,
                          [&](int e, float v) { sx[w * per + e * head_row + d] = d < s.dim ? silu_dev(v) : 0.0f; });
        }
        __syncthreads();
        const int group = s.heads / s.kv_heads;
#pragma unroll 1
        for (int i = wave; i < 2 * nt; i += 4) {  // one (head, token) per wave
            const int h = part * 2 + (i & 1), e = i >> 1;
            if (h >= s.kv_heads) continue;
            const float *sq = sx + (size_t)(i & 1) * 2 * per + e * head_row, *sk = sq + per;
            float qq = 0.0f, kk = 0.0f, dot = 0.0f;
            for (int d = lane; d < head_row; d += 64) {
                const float q = sq[d], k = sk[d];
                qq = fmaf(q, q, qq);
                kk = fmaf(k, k, kk);
                dot = fmaf(q, k, dot);
            }
            const float rq = 1.0f / sqrtf(wave_sum(qq) + 1e-6f) / sqrtf((float)s.dim), rk = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
            dot = wave_sum(dot);
            float *out = a.qkg + ((row0 + e) * s.heads + h * group) * 3 * head_row;
            for (int g = 0; g < group; ++g)
                for (int d = lane; d < head_row; d += 64) {
                    out[g * 3 * head_row + d] = sq[d] * rq;
                    out[(g * 3 + 1) * head_row + d] = sk[d] * rk;
                }
            if (lane == 0) a.bkq[(row0 + e) * nb + s.heads + h] = dot * rq * rk;
        }
        return;
    }
    part -= qk_parts;
    if (part < v_parts) {
        const int c = part * kPrepareWidth + t;
        if (c < nv)
            short_conv_run(conv, b, pos, pos_slot, t0, 2 * nk + c, a.col_v + c, [&](int e, float v) {
                if (e < nt) a.v[(row0 + e) * nv + c] = silu_dev(v);
            });
        return;
    }
    part -= v_parts;
    if (part == 0)
        for (int i = t; i < s.heads * nt; i += 256) {
            const int e = i / s.heads, h = i % s.heads;
            a.bkq[(row0 + e) * nb + h] = sigmoid_dev(a.proj[(row0 + e) * a.ld + a.col_b + h]);
        }
    const int c = part * kPrepareWidth + t;
    if (c >= s.heads * head_row) return;
    const int h = c / head_row, d = c % head_row;
    const float a_log = a.w.a_log[h], bias = d < s.dim ? a.w.dt_bias[h * s.dim + d] : 0.0f;
    const float *step = a.step + row0 * s.heads * head_row + c;
    float *g = a.qkg + (row0 * s.heads + h) * 3 * head_row + 2 * head_row + d;
    float x[kConvTokens];
#pragma unroll
    for (int e = 0; e < kConvTokens; ++e) x[e] = step[(size_t)min(e, nt - 1) * s.heads * head_row];
#pragma unroll 1
    for (int e = 0; e < nt; ++e) {
        float v = x[0];
#pragma unroll
        for (int i = 1; i < kConvTokens; ++i) v = e == i ? x[i] : v;
        g[(size_t)e * s.heads * 3 * head_row] = d < s.dim ? decay_dev(a_log, v + bias) : 1.0f;
    }
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
    const int nv = s.heads * s.vdim, T = a.new_len;
    const size_t row0 = (size_t)b * T;
    float *st = a.state + (((size_t)b * s.heads + h) * s.vdim + min(j, s.vdim - 1)) * DP + l32 * DR;
    float S[DR];
#pragma unroll
    for (int r = 0; r < DR; ++r) S[r] = st[r];
    // The vectors of a chunk: requested into registers before the chunk in front of it is worked on, put into LDS after.
    constexpr int QUADS = kChunk * 3 * DP / 4, QN = (QUADS + NT - 1) / NT;
    static_assert(kChunk * (COLS + 2) <= NT, "one scalar per thread");
    const float *vec = a.qkg + (row0 * s.heads + h) * 3 * DP;
    const int token = s.heads * 3 * DP;  // floats from a token to the next
    // this thread's scalar: a value of v, beta or k . q of token t / (COLS + 2)
    const int sct = t / (COLS + 2), scc = t % (COLS + 2), nb = s.heads + s.kv_heads;
    const float *scp = scc < COLS ? a.v + row0 * nv + h * s.vdim + min(j0 + scc, s.vdim - 1)
                                  : a.bkq + row0 * nb + (scc == COLS ? h : s.heads + h / (s.heads / s.kv_heads));
    const int scs = scc < COLS ? nv : nb;
    float4 rq[QN];
    float rs = 0.0f;
    auto request = [&](int t0) {
#pragma unroll
        for (int n = 0; n < QN; ++n) {
            const int i = t + n * NT, tok = min(t0 + i / (3 * DP / 4), T - 1);
            rq[n] = *(const float4 *)(vec + (size_t)tok * token + 4 * (i % (3 * DP / 4)));
        }
        rs = scp[(size_t)min(t0 + min(sct, kChunk - 1), T - 1) * scs];
    };
    auto stage = [&](int buf, int t0) {
        if (t0 + kChunk > T) {  // behind the last token nothing moves
#pragma unroll
            for (int n = 0; n < QN; ++n) {
                const int i = t + n * NT;
                if (t0 + i / (3 * DP / 4) < T) continue;
                const float f = i % (3 * DP / 4) >= 2 * DP / 4 ? 1.0f : 0.0f;
                rq[n] = make_float4(f, f, f, f);
            }
        }
#pragma unroll
        for (int n = 0; n < QN; ++n)
            if (t + n * NT < QUADS) *(float4 *)(&sv[buf][0][0][0] + 4 * (t + n * NT)) = rq[n];
        if (t < kChunk * (COLS + 2)) sc[buf][sct][scc] = rs;
    };
    request(0);
    stage(0, 0);
    __syncthreads();
    int buf = 0;
    for (int t0 = 0; t0 < T; t0 += kChunk, buf ^= 1) {
        const bool more = t0 + kChunk < T;
        if (more) request(t0 + kChunk);
        // two sets of registers: the vectors of the next token are on their way while this one is worked on
        struct Token {
            float q[DR], k[DR], g[DR], v, beta, kq;
        } even, odd;
        constexpr int AL = DR % 4 == 0 ? 16 : (DR % 2 == 0 ? 8 : 4);
        auto fetch = [&](Token &x, int i) {
            __builtin_memcpy(x.q, __builtin_assume_aligned(&sv[buf][i][0][l32 * DR], AL), 4 * DR);
            __builtin_memcpy(x.k, __builtin_assume_aligned(&sv[buf][i][1][l32 * DR], AL), 4 * DR);
            __builtin_memcpy(x.g, __builtin_assume_aligned(&sv[buf][i][2][l32 * DR], AL), 4 * DR);
            x.v = sc[buf][i][wave * 2 + half];
            x.beta = sc[buf][i][COLS];
            x.kq = sc[buf][i][COLS + 1];
        };
        float out = 0.0f;
        auto work = [&](const Token &x, int i) {
            float ks = 0.0f, qs = 0.0f;
#pragma unroll
            for (int r = 0; r < DR; ++r) {
                S[r] *= x.g[r];
                ks = fmaf(S[r], x.k[r], ks);
                qs = fmaf(S[r], x.q[r], qs);
            }
            ks = half_sum(ks);
            qs = half_sum(qs);
            const float u = x.beta * (x.v - ks);
#pragma unroll
            for (int r = 0; r < DR; ++r) S[r] = fmaf(x.k[r], u, S[r]);
            out = l32 == i ? fmaf(x.kq, u, qs) : out;  // lane i keeps the output of token i
        };
        fetch(even, 0);
#pragma unroll 1
        for (int i = 0; i < kChunk; i += 2) {
            fetch(odd, i + 1);
            __builtin_amdgcn_sched_barrier(0);
            work(even, i);
            __builtin_amdgcn_sched_barrier(0);
            fetch(even, min(i + 2, kChunk - 1));
            __builtin_amdgcn_sched_barrier(0);
            work(odd, i + 1);
            __builtin_amdgcn_sched_barrier(0);
        }
        if (l32 < kChunk && j < s.vdim && t0 + l32 < T) a.o[(row0 + t0 + l32) * nv + h * s.vdim + j] = out;
        if (more) stage(buf ^ 1, t0 + kChunk);
        __syncthreads();
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

constexpr int kStepThreads = 512, kStepGroups = kStepThreads / 16;

// Eight values of a bf16 row against eight floats.
__device__ __forceinline__ float dot8(const uint4 &v, const float *x, float acc) {
    const uint32_t u[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        acc = fmaf(__uint_as_float(u[e] << 16), x[2 * e], acc);
        acc = fmaf(__uint_as_float(u[e] & 0xffff0000u), x[2 * e + 1], acc);
    }
    return acc;
}

// One token of one sequence and head: grid (heads, batch).  NF float4 of a state column per lane of 16, CI columns per group.
// The state and the first rows of the low-rank factors are requested before anything else.  The code is kept short: at
// this size a launch waits for its instructions as much as for its data.
template <int NF, int CI>
__global__ __launch_bounds__(kStepThreads) void delta_step_kernel(DeltaArgs a, int channels, int rank_ap, int rank_gp, int state_row) {
    extern __shared__ float low[];  // a1 [rank_ap], g1 [rank_gp]
    __shared__ __align__(16) float sx[4][kMaxDim];  // q, k, g, v
    __shared__ float sgate[kMaxDim], so[kMaxDim];
    __shared__ float red[4];
    const DeltaShape &s = a.s;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int h = blockIdx.x, b = blockIdx.y, group = s.heads / s.kv_heads, hk = h / group, pos = *a.pos_dev, pos_slot = pos % s.taps;
    const int nk = s.kv_heads * s.dim;
    const float *p = a.proj + (size_t)b * a.ld;
    float *state = a.state + ((size_t)b * s.heads + h) * s.vdim * state_row;
    const int kl = lane & 15, col0 = t >> 4;
    float4 S[CI][NF];
#pragma unroll
    for (int i = 0; i < CI; ++i)
#pragma unroll
        for (int f = 0; f < NF; ++f)  // clamped addresses; what lies outside is never used
            S[i][f] = *(const float4 *)(state + (size_t)min(col0 + i * kStepGroups, s.vdim - 1) * state_row + min(kl * 4 + 64 * f, state_row - 4));
    // rows of W_a2 and W_g2 of this head, 4 lanes per row: r = t / 4, + 128, ...
    const uint16_t *wa = a.w.a2 + (size_t)h * state_row * rank_ap, *wg = a.w.g2 + (size_t)h * s.vdim * rank_gp;
    const int rows = s.dim + s.vdim, part = t & 3;
    uint4 wp[2][4];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int r = min((t >> 2) + 128 * i, rows - 1), rank = r < s.dim ? rank_ap : rank_gp;
            wp[i][j] = *(const uint4 *)((r < s.dim ? wa + (size_t)r * rank_ap : wg + (size_t)(r - s.dim) * rank_gp) + min(part * 8 + 32 * j, rank - 8));
        }
    for (int k = t; k < rank_ap + rank_gp; k += kStepThreads) low[k] = p[k < rank_ap ? a.col_a1 + k : a.col_g1 + k - rank_ap];
    // convolution of the head's q, k and v; the new inputs go into a ring slot that no tap of this token reads (q and k by
    // the first head of a group)
    float *slot = a.ring + ((size_t)b * s.taps + pos_slot) * channels;
    const ShortConv conv = conv_of(a, channels);
#pragma unroll 1
    for (int i = t; i < 2 * state_row + s.vdim; i += kStepThreads) {
        const int w = i < state_row ? 0 : (i < 2 * state_row ? 1 : 3), d = i - min(w, 2) * state_row;
        const bool on = w == 3 || d < s.dim;
        const int c = w == 3 ? h * s.vdim + d : hk * s.dim + min(d, s.dim - 1);
        const int ch = min(w, 2) * nk + c, col = (w == 0 ? a.col_q : (w == 1 ? a.col_k : a.col_v)) + c;
        const float v = silu_dev(short_conv(conv, b, pos, pos_slot, 0, ch, col));
        sx[w][d] = on ? v : 0.0f;
        if (on && (w == 3 || h % group == 0)) slot[ch] = p[col];
    }
    __syncthreads();
    // raw low-rank products to sx[2] and sgate
    auto put = [&](int r, float acc) {
        acc += dpp_move<0xb1, 0xf>(0.0f, acc);
        acc += dpp_move<0x4e, 0xf>(0.0f, acc);
        if (part == 0 && r < rows) (r < s.dim ? sx[2][r] : sgate[r - s.dim]) = acc;
    };
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int r = (t >> 2) + 128 * i, rank = r < s.dim ? rank_ap : rank_gp;
        const float *x = low + (r < s.dim ? 0 : rank_ap);
        float acc = 0.0f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int k = part * 8 + 32 * j;
            const float v = dot8(wp[i][j], x + min(k, rank - 8), acc);
            acc = k < rank ? v : acc;
        }
#pragma unroll 1
        for (int k = part * 8 + 128; k < rank; k += 32)
            acc = dot8(*(const uint4 *)((r < s.dim ? wa + (size_t)r * rank_ap : wg + (size_t)min(r - s.dim, s.vdim - 1) * rank_gp) + k), x + k, acc);
        put(r, acc);
    }
#pragma unroll 1
    for (int r = (t >> 2) + 256; r < (rows + 127) / 128 * 128; r += 128) {
        const int rr = min(r, rows - 1), rank = rr < s.dim ? rank_ap : rank_gp;
        const uint16_t *w = rr < s.dim ? wa + (size_t)rr * rank_ap : wg + (size_t)(rr - s.dim) * rank_gp;
        const float *x = low + (rr < s.dim ? 0 : rank_ap);
        float acc = 0.0f;
#pragma unroll 1
        for (int k = part * 8; k < rank; k += 32) acc = dot8(*(const uint4 *)(w + k), x + k, acc);
        put(r, acc);
    }
    if (wave < 3) {  // |q|^2, |k|^2, q . k
        float v = 0.0f;
        for (int d = lane; d < state_row; d += 64) v += sx[wave == 1][d] * sx[wave != 0][d];
        v = wave_sum(v);
        if (lane == 0) red[wave] = v;
    }
    __syncthreads();
    const float rq = 1.0f / sqrtf(red[0] + 1e-6f) / sqrtf((float)s.dim), rk = 1.0f / sqrtf(red[1] + 1e-6f);
    const float kq = red[2] * rq * rk, beta = sigmoid_dev(p[a.col_b + h]);
    if (t < state_row) sx[2][t] = t < s.dim ? decay_dev(a.w.a_log[h], sx[2][t] + a.w.dt_bias[h * s.dim + t]) : 0.0f;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < CI; ++i) {
        const int j = col0 + i * kStepGroups;
        float ks = 0.0f, qs = 0.0f;
#pragma unroll
        for (int f = 0; f < NF; ++f) {
            const int d = kl * 4 + 64 * f;
            if (d >= state_row) continue;
            const float4 g4 = *(const float4 *)&sx[2][d], q4 = *(const float4 *)&sx[0][d], k4 = *(const float4 *)&sx[1][d];
            float4 &v = S[i][f];
            v.x *= g4.x; v.y *= g4.y; v.z *= g4.z; v.w *= g4.w;
            ks += v.x * k4.x + v.y * k4.y + v.z * k4.z + v.w * k4.w;
            qs += v.x * q4.x + v.y * q4.y + v.z * q4.z + v.w * q4.w;
        }
        ks = row16_sum(ks) * rk;
        qs = row16_sum(qs) * rq;
        if (j >= s.vdim) continue;
        const float u = beta * (sx[3][j] - ks), uk = u * rk;
#pragma unroll
        for (int f = 0; f < NF; ++f) {
            const int d = kl * 4 + 64 * f;
            if (d >= state_row) continue;
            const float4 k4 = *(const float4 *)&sx[1][d];
            float4 &v = S[i][f];
            v.x = fmaf(k4.x, uk, v.x);
            v.y = fmaf(k4.y, uk, v.y);
            v.z = fmaf(k4.z, uk, v.z);
            v.w = fmaf(k4.w, uk, v.w);
            *(float4 *)(state + (size_t)j * state_row + d) = v;
        }
        if (kl == 0) so[j] = fmaf(kq, u, qs);
    }
    __syncthreads();
    float sum = 0.0f;  // every wave for itself
    for (int d = lane; d < s.vdim; d += 64) sum = fmaf(so[d], so[d], sum);
    const float rs = 1.0f / sqrtf(wave_sum(sum) / (float)s.vdim + s.eps);
    if (t < s.vdim) {
        const float v = so[t] * rs * a.w.norm[t] * sigmoid_dev(sgate[t]);
        const size_t at = (size_t)b * a.ldo + h * s.vdim + t;
        if (a.out_bf16) ((uint16_t *)a.out)[at] = f32_to_bf16(v);
        else ((float *)a.out)[at] = v;
    }
}

template <int NF>
void step_run(agpu_ctx *ctx, const DeltaArgs &a) {
    const DeltaShape &s = a.s;
    const dim3 grid((unsigned)s.heads, (unsigned)a.batch), block(kStepThreads);
    const size_t lds = (size_t)(s.rank_ap() + s.rank_gp()) * sizeof(float);
    const int ci = ceil_div(s.vdim, kStepGroups);
#define AGPU_DELTA_STEP(CI) \
    hipLaunchKernelGGL((delta_step_kernel<NF, CI>), grid, block, lds, ctx->stream, a, s.channels(), s.rank_ap(), s.rank_gp(), s.state_row())
    if (ci <= 1) AGPU_DELTA_STEP(1);
    else if (ci <= 2) AGPU_DELTA_STEP(2);
    else if (ci <= 4) AGPU_DELTA_STEP(4);
    else AGPU_DELTA_STEP(8);
#undef AGPU_DELTA_STEP
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
    const int nf = ceil_div(a.s.state_row(), 64);
    if (nf <= 1) step_run<1>(ctx, a);
    else if (nf <= 2) step_run<2>(ctx, a);
    else step_run<4>(ctx, a);
    return AGPU_LAUNCH_CHECK(ctx, "delta_step_kernel");
}

int32_t delta_prefill_launch(agpu_ctx *ctx, const DeltaArgs &a) {
    int32_t rc = check(ctx, a);
    if (rc != AGPU_OK) return rc;
    const DeltaShape &s = a.s;
    const unsigned rows = (unsigned)(a.batch * a.new_len);
    // the low-rank products in fp32: they feed decays and gates
    DenseOut step, gate;
    step.n_plain = step.ldo = s.heads * s.state_row();
    step.out = a.step;
    rc = dense_gemm_f32_launch(ctx, a.proj + a.col_a1, a.ld, a.w.a2, s.rank_ap(), (int)rows, step.n_plain, s.rank_ap(), step);
    if (rc != AGPU_OK) return rc;
    gate.n_plain = gate.ldo = s.heads * s.vdim;
    gate.out = a.gate;
    rc = dense_gemm_f32_launch(ctx, a.proj + a.col_g1, a.ld, a.w.g2, s.rank_gp(), (int)rows, gate.n_plain, s.rank_gp(), gate);
    if (rc != AGPU_OK) return rc;
    const int qk_parts = ceil_div(s.kv_heads, 2), v_parts = ceil_div(s.heads * s.vdim, kPrepareWidth), g_parts = ceil_div(s.heads * s.state_row(), kPrepareWidth);
    hipLaunchKernelGGL(delta_prepare_kernel, dim3((unsigned)ceil_div(a.new_len, kConvTokens), (unsigned)(qk_parts + v_parts + g_parts), (unsigned)a.batch),
                       dim3(256), (size_t)4 * kConvTokens * s.state_row() * sizeof(float), ctx->stream, a, s.channels(), s.state_row(), qk_parts, v_parts);
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
