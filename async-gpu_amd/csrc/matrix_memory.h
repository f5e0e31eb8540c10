// Matrix memory with exponential gates (the mLSTM of xLSTM): per head a state S [dim, vdim], a normaliser n [dim] and a running
// maximum m of the log gates, all fp32.  Per token, with i = cap tanh(i' / cap) and f = log sigmoid(cap tanh(f' / cap)):
// m' = max(f + m, i), S <- exp(f + m - m') S + exp(i - m') k v^T, n likewise with k alone,
// o = S^T q / (max(|n . q|, exp(-m')) + 1e-6).  Everything here is fp32; the head norm and the gate behind it are DenseRows'.
#pragma once
#include "agpu_internal.h"
#include "dense_linear.h"

struct MemoryShape {
    int heads = 0, dim = 0, vdim = 0;
    float cap = 0.0f;
    // storage widths of a head, in projections, state and output
    int dimp() const { return (dim + 31) / 32 * 32; }
    int vdimp() const { return (vdim + 31) / 32 * 32; }
    size_t state_floats() const { return (size_t)heads * vdimp() * dimp(); }      // per sequence: [heads][vdimp][dimp]
    size_t norm_floats() const { return (size_t)heads * 2 * (dimp() + 4); }       // per sequence: [heads][2][n | m, 3 unused]
};

constexpr int kMemoryChunk = 64;  // tokens that the many-token form takes at once

struct MemoryArgs {
    MemoryShape s;
    // rows [batch * new_len], stride ld: heads x dimp, heads x dimp, heads x vdimp, heads, heads; padding columns are zero
    const float *q = nullptr, *k = nullptr, *v = nullptr, *i = nullptr, *f = nullptr;
    int ld = 0;
    float *state = nullptr;  // [batch] x state_floats
    float *norm = nullptr;   // [batch] x norm_floats; the slot of a position is its parity, so a token never overwrites what it reads
    int batch = 1, new_len = 1;
    const int *pos_dev = nullptr;
    float *out = nullptr;    // rows, stride ldo: heads x vdimp
    int ldo = 0;
    // scratch of the many-token form, per sequence, head and chunk: memory_scratch_bytes
    void *scratch = nullptr;
};

bool memory_supported(const MemoryShape &s);
size_t memory_scratch_bytes(const MemoryShape &s, int batch, int new_len);
// One new token per sequence in one launch, more in chunks of kMemoryChunk.
int32_t memory_launch(agpu_ctx *ctx, const MemoryArgs &a);
