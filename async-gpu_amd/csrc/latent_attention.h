// Latent attention: keys and values of every head are linear maps of one cached latent per token (RMS-normed, `rank`
// wide), plus one rotated key part of `rot` dimensions that all heads share.  Optionally a learned sink per head in the
// softmax denominator.
#pragma once
#include "agpu_internal.h"
#include "dense_linear.h"
#include "rope.h"

struct LatentShape {
    int heads = 0, dim = 0, rot = 0, rot_dims = 0, vdim = 0, rank = 0;  // rot_dims of the rot dimensions turn
    float scale = 1.0f, eps = 0.0f;
    // storage widths
    int dimp() const { return (dim + 7) / 8 * 8; }
    int rotp() const { return (rot + 7) / 8 * 8; }
    int vdimp() const { return (vdim + 31) / 32 * 32; }
    int rankp() const { return (rank + 31) / 32 * 32; }
    int cache_row() const { return rankp() + (rot + 31) / 32 * 32; }  // [latent | rotated key part], zero padded
    int query_row() const { return (dimp() + rotp() + 15) / 16 * 16; }  // one head's bf16 query in the tiled kernel
};

struct LatentWeights {
    const float *norm = nullptr;    // [rank], plain
    const uint16_t *uk = nullptr;   // [heads * dimp][rankp], zero padded
    const uint16_t *uv = nullptr;   // [heads * vdimp][rankp], zero padded
    const float *sink = nullptr;    // [heads] or null
    const float2 *rope = nullptr;   // [positions][rot_dims / 2]: cos, sin
};

// One call appends new_len tokens of each of `batch` sequences to the cache and attends from them.
struct LatentArgs {
    LatentShape s;
    LatentWeights w;
    const float *q = nullptr;     // rows [batch * new_len], stride ld: heads x [dim | rot]
    const float *down = nullptr;  // same rows and stride: [rank | rot]
    int ld = 0;
    void *cache = nullptr;        // [batch][positions][cache_row], bf16 or fp32
    int cache_bf16 = 0, positions = 0;
    int batch = 1, new_len = 1;
    const int *pos_dev = nullptr; // positions cached before this call
    int kv_max = 0;               // bound of *pos_dev + new_len; exact for the tiled kernel
    void *out = nullptr;          // [rows], stride ldo: heads x vdim, bf16 or fp32
    int ldo = 0, out_bf16 = 0;
    // scratch
    void *qlat = nullptr;       // absorbed: rows * heads * cache_row floats
    float *partial = nullptr;   // absorbed: latent_partial_floats
    uint16_t *qb = nullptr;     // tiled: rows * heads * query_row
    uint16_t *kx = nullptr;     // tiled: [batch][kv_max][heads * dimp]
    uint16_t *vx = nullptr;     // tiled: [batch][heads * vdimp][kv_stride], transposed
};

// Keys split over this many workgroups in the absorbed form.
int latent_splits(const agpu_ctx *ctx, const LatentShape &s, int rows, int kv_max);
size_t latent_partial_floats(const LatentShape &s, int rows, int splits);
inline int latent_kv_stride(int kv_max) { return (kv_max + 31) / 32 * 32; }
// Absorbed form: W_uk is folded into the query and W_uv applied to the attended latent; fp32 arithmetic.  Any row count.
int32_t latent_absorbed_launch(agpu_ctx *ctx, const LatentArgs &a);
// Tiled form for prompts: expands the cached latents into keys and values of every head and runs a flash-style kernel
// on the bf16 matrix cores (fp32 scores and softmax).  bf16 cache only.
bool latent_tiled_supported(const LatentShape &s);
int32_t latent_tiled_launch(agpu_ctx *ctx, const LatentArgs &a);
