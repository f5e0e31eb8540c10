// Gated delta rule with one decay per head and key channel: a linear-attention layer whose state per head is a matrix
// S [dim, vdim] in fp32.  Per token: S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  q, k, v pass a short
// causal convolution and silu, q and k become unit vectors; the output is RMS-normed per head and gated.
#pragma once
#include "agpu_internal.h"
#include "dense_linear.h"

struct DeltaShape {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 0;
    int rank_a = 0, rank_g = 0;  // low-rank sizes of the decay and of the output gate
    float eps = 0.0f;
    int channels() const { return 2 * kv_heads * dim + heads * vdim; }  // q | k | v of the convolution
    int state_row() const { return (dim + 31) / 32 * 32; }              // state layout: [heads][vdim][state_row], zero padded
    int rank_ap() const { return (rank_a + 31) / 32 * 32; }
    int rank_gp() const { return (rank_g + 31) / 32 * 32; }
};

struct DeltaWeights {
    const float *conv = nullptr;    // [channels][taps], last tap is the current token's
    const float *a_log = nullptr;   // [heads]
    const float *dt_bias = nullptr; // [heads * dim]
    const uint16_t *a2 = nullptr;   // [heads * state_row][rank_ap], zero padded per head
    const uint16_t *g2 = nullptr;   // [heads * vdim][rank_gp]
    const float *norm = nullptr;    // [vdim], plain
};

struct DeltaArgs {
    DeltaShape s;
    DeltaWeights w;
    const float *proj = nullptr;  // rows [batch * new_len], stride ld, with q, k, v, b, a1, g1 at these columns
    int ld = 0, col_q = 0, col_k = 0, col_v = 0, col_b = 0, col_a1 = 0, col_g1 = 0;
    float *state = nullptr;  // [batch][heads][vdim][state_row]
    float *ring = nullptr;   // [batch][taps][channels]: convolution inputs of the last tokens, slot = position % taps
    int batch = 1, new_len = 1;
    const int *pos_dev = nullptr;
    void *out = nullptr;  // rows, stride ldo: heads x vdim, bf16 or fp32
    int ldo = 0, out_bf16 = 0;
    // scratch of the many-token form, fp32 rows
    float *qkg = nullptr;   // [rows][heads][3][state_row]: unit vectors q and k, decays g
    float *v = nullptr;     // [rows][heads * vdim]
    float *step = nullptr;  // [rows][heads * state_row]: W_a2 a1
    float *bkq = nullptr;   // [rows][heads + kv_heads]: beta | k . q
    float *gate = nullptr;  // [rows][heads * vdim]: W_g2 g1
    float *o = nullptr;     // [rows][heads * vdim]
};

bool delta_supported(const DeltaShape &s);
// One new token per sequence, everything after the projections in one launch.
int32_t delta_step_launch(agpu_ctx *ctx, const DeltaArgs &a);
// Any number of tokens.
int32_t delta_prefill_launch(agpu_ctx *ctx, const DeltaArgs &a);
