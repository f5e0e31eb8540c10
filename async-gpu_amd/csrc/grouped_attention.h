// Causal attention with grouped heads over cached keys and values: H query heads share G key/value heads, H / G each.  Pairs
// of neighbouring dimensions turn with the position (the first rot_dims of every head), scores may be soft-capped, a learned
// sink per head may stand in the softmax denominator, and the output may be gated.
#pragma once
#include "agpu_internal.h"
#include "dense_linear.h"
#include "rope.h"

struct GroupedShape {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, rot_dims = 0;
    float scale = 1.0f, softcap = 0.0f;  // softcap 0: none
    // storage widths of a head, in projections, cache and output
    int dimp() const { return (dim + 31) / 32 * 32; }
    int vdimp() const { return (vdim + 31) / 32 * 32; }
    int group() const { return heads / kv_heads; }
};

// One call appends new_len tokens of each of `batch` sequences to the cache and attends from them.  Padding columns of q, k, v
// are zero.
struct GroupedArgs {
    GroupedShape s;
    const float2 *rope = nullptr;  // [positions][rot_dims / 2]: cos, sin; never null
    const float *sink = nullptr;   // [heads] or null
    // rows [batch * new_len], stride ld: heads x dimp, kv_heads x dimp, kv_heads x vdimp, heads x vdimp (gate before its sigmoid, or null)
    const float *q = nullptr, *k = nullptr, *v = nullptr, *gate = nullptr;
    int ld = 0;
    void *kcache = nullptr;  // [batch][kv_heads][positions][dimp], bf16 or fp32
    void *vcache = nullptr;  // [batch][kv_heads][vdimp][kv_stride], transposed; kv_stride = grouped_kv_stride(positions)
    int cache_bf16 = 0, positions = 0;
    int batch = 1, new_len = 1;
    const int *pos_dev = nullptr;  // positions cached before this call
    int kv_max = 0;                // bound of *pos_dev + new_len
    void *out = nullptr;           // rows, stride ldo: heads x vdimp, bf16 or fp32
    int ldo = 0, out_bf16 = 0;
    float *partial = nullptr;      // grouped_partial_floats
};

bool grouped_supported(const GroupedShape &s);
inline int grouped_kv_stride(int positions) { return (positions + 31) / 32 * 32; }
// Scratch of a call of this shape, for any number of cached positions up to kv_max.
size_t grouped_partial_floats(const agpu_ctx *ctx, const GroupedShape &s, int batch, int new_len, int kv_max);
int32_t grouped_attention_launch(agpu_ctx *ctx, const GroupedArgs &a);
