// Real-gated linear recurrent unit (gated_lru.h).
//
// One token: a workgroup takes 32 channels of a block; it needs the whole block's convolution (a few values per channel) for its
// rows of the block-diagonal maps, and then finishes its channels.
//
// Many tokens: convolution -> block-diagonal Linear (fp32 matrix cores) -> per chunk of 32 tokens the recurrence from zero, which
// leaves every token's decay and input and the chunk's total decay and state -> per chunk the state in front of it, folded
// from the chunks before, and the tokens again.
#include "gated_lru.h"
#include "short_conv.h"

namespace {

constexpr int kChunk = 32;    // tokens per chunk of the scan
constexpr int kStepRows = 32; // channels per workgroup of the step

__device__ __forceinline__ float softplus_dev(float v) { return fmaxf(v, 0.0f) + log1pf(expf(-fabsf(v))); }

// Decay and input of one channel and token from the gates in front of their sigmoid.
__device__ __forceinline__ void lru_terms(float r, float i, float u, float sp, float &decay, float &input) {
    const float log_a = -8.0f * sigmoid_dev(r) * sp;
    decay = expf(log_a);
    input = sqrtf(-expm1f(2.0f * log_a)) * sigmoid_dev(i) * u;
}

__device__ __forceinline__ ShortConv conv_of(const LruArgs &a, int widthp) {
    return ShortConv{a.proj, a.ld, a.ring, a.w.conv, widthp, a.s.taps, a.new_len};
}

__device__ __forceinline__ void put_out(const LruArgs &a, size_t row, int c, float v) {
    if (a.out_bf16) ((uint16_t *)a.out)[row * a.ldo + c] = f32_to_bf16(v);
    else ((float *)a.out)[row * a.ldo + c] = v;
}

// grid (blocks * ceil(blockp / 32), batch)
__global__ __launch_bounds__(256) void lru_step_kernel(LruArgs a, int blockp, int widthp) {
    extern __shared__ __align__(16) float su[];  // [blockp]
    __shared__ float sg[2][kStepRows];
    const LruShape &s = a.s;
    const int t = threadIdx.x, kl = t & 15, parts = blockp / kStepRows, blk = blockIdx.x / parts, r0 = blockIdx.x % parts * kStepRows, b = blockIdx.y;
    const int pos = *a.pos_dev, pos_slot = pos % s.taps, c0 = blk * blockp;
    const uint16_t *w = a.w.gates + (size_t)blk * 2 * blockp * blockp;
    // 64 rows (R, then I, of the 32 channels), 16 lanes each, 16 at a time; the first 128 columns are requested before the convolution
    uint4 first[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int row = i * 16 + (t >> 4), r = (row >> 5) * blockp + r0 + (row & 31);
        first[i] = *(const uint4 *)(w + (size_t)r * blockp + min(kl * 8, blockp - 8));
    }
    const ShortConv conv = conv_of(a, widthp);
    for (int c = t; c < blockp; c += 256) su[c] = short_conv(conv, b, pos, pos_slot, 0, c0 + c, a.col_x + c0 + c) + a.w.conv_bias[c0 + c];
    __syncthreads();
    auto dot = [&](const uint4 &v, int k, float acc) {
        const uint32_t u[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            acc = fmaf(__uint_as_float(u[e] << 16), su[k + 2 * e], acc);
            acc = fmaf(__uint_as_float(u[e] & 0xffff0000u), su[k + 2 * e + 1], acc);
        }
        return acc;
    };
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int row = i * 16 + (t >> 4), r = (row >> 5) * blockp + r0 + (row & 31);
        float acc = kl * 8 < blockp ? dot(first[i], kl * 8, 0.0f) : 0.0f;
#pragma unroll 2
        for (int k = kl * 8 + 128; k < blockp; k += 128) acc = dot(*(const uint4 *)(w + (size_t)r * blockp + k), k, acc);
        acc = row16_sum(acc);
        if (kl == 0) sg[row >> 5][row & 31] = acc + a.w.gate_bias[(size_t)blk * 2 * blockp + r];
    }
    __syncthreads();
    if (t >= kStepRows) return;
    const int c = c0 + r0 + t;
    float decay, input;
    lru_terms(sg[0][t], sg[1][t], su[r0 + t], softplus_dev(a.w.lam[c]), decay, input);
    float *state = a.state + (size_t)b * widthp + c;
    const float S = fmaf(decay, *state, input);
    *state = S;
    const float *p = a.proj + (size_t)b * a.ld;
    a.ring[((size_t)b * s.taps + pos_slot) * widthp + c] = p[a.col_x + c];
    put_out(a, b, c, S * gelu_tanh_dev(p[a.col_y + c]));
}

// grid (groups of 256 channels, groups of kConvTokens tokens, batch)
__global__ __launch_bounds__(256) void lru_conv_kernel(LruArgs a, int widthp) {
    const int c = blockIdx.x * 256 + threadIdx.x, t0 = blockIdx.y * kConvTokens, b = blockIdx.z, T = a.new_len, pos = *a.pos_dev;
    if (c >= widthp) return;
    const float bias = a.w.conv_bias[c];
    float *u = a.u + ((size_t)b * T + t0) * widthp + c;
    short_conv_run(conv_of(a, widthp), b, pos, pos % a.s.taps, t0, c, a.col_x + c, [&](int e, float v) {
        if (t0 + e < T) u[(size_t)e * widthp] = v + bias;
    });
}

// Carries: slot 0 the state in front of the portion, slot 1 + c the total decay and the state of chunk c from zero.
__device__ __forceinline__ float2 *carry_of(const LruArgs &a, int chunks, int widthp, int b, int c) {
    return (float2 *)a.carries + (size_t)b * (chunks + 1) * widthp + c;
}

// grid (groups of 256 channels, chunks, batch): the gates give way to decay and input.
__global__ __launch_bounds__(256) void lru_chunk_kernel(LruArgs a, int blockp, int widthp) {
    const int c = blockIdx.x * 256 + threadIdx.x, t0 = blockIdx.y * kChunk, b = blockIdx.z, T = a.new_len, nt = min(kChunk, T - t0);
    if (c >= widthp) return;
    const float sp = softplus_dev(a.w.lam[c]);
    const size_t row0 = (size_t)b * T + t0;
    float *g = a.gates + row0 * 2 * widthp + c / blockp * 2 * blockp + c % blockp;
    const float *u = a.u + row0 * widthp + c;
    float total = 1.0f, S = 0.0f;
    constexpr int U = 8;
#pragma unroll 1
    for (int t = 0; t < nt; t += U) {
        float r[U], i[U], x[U];
#pragma unroll
        for (int e = 0; e < U; ++e) {
            const size_t at = (size_t)min(t + e, nt - 1);
            r[e] = g[at * 2 * widthp];
            i[e] = g[at * 2 * widthp + blockp];
            x[e] = u[at * widthp];
        }
#pragma unroll
        for (int e = 0; e < U; ++e) {
            if (t + e >= nt) break;
            float decay, input;
            lru_terms(r[e], i[e], x[e], sp, decay, input);
            total *= decay;
            S = fmaf(decay, S, input);
            g[(size_t)(t + e) * 2 * widthp] = decay;
            g[(size_t)(t + e) * 2 * widthp + blockp] = input;
        }
    }
    float2 *carry = carry_of(a, gridDim.y, widthp, b, c);
    carry[(size_t)(1 + blockIdx.y) * widthp] = make_float2(total, S);
    if (blockIdx.y == 0) carry[0] = make_float2(0.0f, a.state[(size_t)b * widthp + c]);
}

// grid as above; the last chunk keeps the state and the ring's new inputs.
__global__ __launch_bounds__(256) void lru_output_kernel(LruArgs a, int blockp, int widthp) {
    const int c = blockIdx.x * 256 + threadIdx.x, chunk = blockIdx.y, t0 = chunk * kChunk, b = blockIdx.z, T = a.new_len, nt = min(kChunk, T - t0);
    if (c >= widthp) return;
    const float2 *carry = carry_of(a, gridDim.y, widthp, b, c);
    float S = carry[0].y;
#pragma unroll 8
    for (int i = 0; i < chunk; ++i) {
        const float2 v = carry[(size_t)(1 + i) * widthp];
        S = fmaf(v.x, S, v.y);
    }
    const size_t row0 = (size_t)b * T + t0;
    const float *g = a.gates + row0 * 2 * widthp + c / blockp * 2 * blockp + c % blockp, *y = a.proj + row0 * a.ld + a.col_y + c;
    constexpr int U = 8;
#pragma unroll 1
    for (int t = 0; t < nt; t += U) {
        float decay[U], input[U], x[U];
#pragma unroll
        for (int e = 0; e < U; ++e) {
            const size_t at = (size_t)min(t + e, nt - 1);
            decay[e] = g[at * 2 * widthp];
            input[e] = g[at * 2 * widthp + blockp];
            x[e] = y[at * a.ld];
        }
#pragma unroll
        for (int e = 0; e < U; ++e) {
            if (t + e >= nt) break;
            S = fmaf(decay[e], S, input[e]);
            put_out(a, row0 + t + e, c, S * gelu_tanh_dev(x[e]));
        }
    }
    if (chunk + 1 < (int)gridDim.y) return;
    a.state[(size_t)b * widthp + c] = S;
    const int taps = a.s.taps, pos = *a.pos_dev;
    for (int t = max(T - taps, 0); t < T; ++t)
        a.ring[((size_t)b * taps + (pos + t) % taps) * widthp + c] = a.proj[((size_t)b * T + t) * a.ld + a.col_x + c];
}

}  // namespace

bool lru_supported(const LruShape &s) { return s.width > 0 && s.blocks > 0 && s.width % s.blocks == 0 && s.taps >= 1 && s.blockp() <= 8192; }

size_t lru_carry_floats(const LruShape &s, int batch, int new_len) { return (size_t)batch * (ceil_div(new_len, kChunk) + 1) * s.widthp() * 2; }

int32_t lru_launch(agpu_ctx *ctx, const LruArgs &a) {
    const LruShape &s = a.s;
    if (!lru_supported(s) || a.batch <= 0 || a.new_len <= 0 || (int64_t)a.batch * a.new_len > 65535)
        return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "gated_lru: width %d, blocks %d, taps %d, %d new tokens not supported", s.width, s.blocks, s.taps, a.new_len);
    const int blockp = s.blockp(), widthp = s.widthp();
    if (a.new_len == 1) {
        hipLaunchKernelGGL(lru_step_kernel, dim3((unsigned)(s.blocks * (blockp / kStepRows)), (unsigned)a.batch), dim3(256), blockp * sizeof(float), ctx->stream, a,
                           blockp, widthp);
        return AGPU_LAUNCH_CHECK(ctx, "lru_step_kernel");
    }
    const unsigned groups = (unsigned)ceil_div(widthp, 256), batch = (unsigned)a.batch;
    int32_t rc;
    hipLaunchKernelGGL(lru_conv_kernel, dim3(groups, (unsigned)ceil_div(a.new_len, kConvTokens), batch), dim3(256), 0, ctx->stream, a, widthp);
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "lru_conv_kernel")) != AGPU_OK) return rc;
    DenseOut o;
    o.n_plain = 2 * blockp;
    o.ldo = 2 * widthp;
    o.out = a.gates;
    o.bias = a.w.gate_bias;
    rc = dense_gemm_f32_launch(ctx, a.u, widthp, a.w.gates, blockp, a.batch * a.new_len, 2 * blockp, blockp, o, s.blocks);
    if (rc != AGPU_OK) return rc;
    const dim3 grid(groups, (unsigned)ceil_div(a.new_len, kChunk), batch);
    hipLaunchKernelGGL(lru_chunk_kernel, grid, dim3(256), 0, ctx->stream, a, blockp, widthp);
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "lru_chunk_kernel")) != AGPU_OK) return rc;
    hipLaunchKernelGGL(lru_output_kernel, grid, dim3(256), 0, ctx->stream, a, blockp, widthp);
    return AGPU_LAUNCH_CHECK(ctx, "lru_output_kernel");
}
