// Short causal convolution over time, one filter per channel, on columns of projection rows.  The inputs of earlier tokens are
// kept in a ring [batch][taps][channels], slot = position % taps: a token's own slot is one that none of its taps reads.
#pragma once
#include "agpu_internal.h"

struct ShortConv {
    const float *proj;  // rows [batch * new_len], stride ld
    int ld;
    const float *ring, *w;  // w: [channels][taps], the last tap is the current token's
    int channels, taps, new_len;
};

// Channel c (source column `col` of the projection) at token `t` of the portion.  Inputs before the portion come from the ring,
// before the sequence they are zero.  pos_slot = pos % taps.  Loads go four taps at a time and without branches.
__device__ __forceinline__ float short_conv(const ShortConv &a, int b, int pos, int pos_slot, int t, int c, int col) {
    const int n = a.taps;
    const float *cur = a.proj + (size_t)(b * a.new_len + t) * a.ld + col;
    const float *ring = a.ring + (size_t)b * n * a.channels + c, *w = a.w + (size_t)c * n;
    float v = w[n - 1] * cur[0];
#pragma unroll 1
    for (int k0 = 1; k0 < n; k0 += 4) {
        float x[4], f[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int k = k0 + e;
            const bool on = k < n && pos + t >= k;
            int slot = pos_slot + t - k;
            slot = slot < 0 ? slot + n : slot;
            const float *p = t >= k ? cur - (size_t)k * a.ld : ring + (size_t)slot * a.channels;
            x[e] = *(on ? p : cur);
            f[e] = on ? w[n - 1 - min(k, n - 1)] : 0.0f;
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) v = fmaf(f[e], x[e], v);
    }
    return v;
}

// The same for up to kConvTokens tokens from t0 on, each input loaded once; put(i, value of token t0 + i).
constexpr int kConvTokens = 8, kConvWindow = 4;
template <typename Put>
__device__ __forceinline__ void short_conv_run(const ShortConv &a, int b, int pos, int pos_slot, int t0, int c, int col, Put put) {
    const int n = a.taps, T = a.new_len;
    if (n > kConvWindow) {
#pragma unroll 1
        for (int i = 0; i < kConvTokens && t0 + i < T; ++i) put(i, short_conv(a, b, pos, pos_slot, t0 + i, c, col));
        return;
    }
    const float *base = a.proj + (size_t)b * T * a.ld + col, *ring = a.ring + (size_t)b * n * a.channels + c, *w = a.w + (size_t)c * n;
    float f[kConvWindow], x[kConvTokens + kConvWindow - 1];
#pragma unroll
    for (int e = 0; e < kConvWindow; ++e) f[e] = e >= kConvWindow - n ? w[max(e - (kConvWindow - n), 0)] : 0.0f;
#pragma unroll
    for (int e = 0; e < kConvWindow - 1; ++e) {  // the tokens in front of t0
        const int k = kConvWindow - 1 - e, t = t0 - k;
        int slot = pos_slot + t;
        slot = slot < 0 ? slot + n : slot;
        const bool on = k < n && pos + t >= 0;
        const float *p = t >= 0 ? base + (size_t)t * a.ld : ring + (size_t)slot * a.channels;
        const float v = *(on ? p : base);
        x[e] = on ? v : 0.0f;
    }
#pragma unroll
    for (int i = 0; i < kConvTokens; ++i) x[kConvWindow - 1 + i] = base[(size_t)min(t0 + i, T - 1) * a.ld];
#pragma unroll
    for (int i = 0; i < kConvTokens; ++i) {
        float v = 0.0f;
#pragma unroll
        for (int e = 0; e < kConvWindow; ++e) v = fmaf(f[e], x[i + e], v);
        put(i, v);
    }
}
