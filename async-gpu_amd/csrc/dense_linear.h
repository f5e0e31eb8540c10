// Dense Linear layers with bf16 weights W [N, K] (rows contiguous along K, y = x W^T), for models whose weights stay in
// bf16.  Decode rows (up to kDenseGemvRows) are fp32 and multiplied with fp32 FMAs; more rows go to the matrix cores,
// as bf16 rows (v_mfma_f32_*_bf16) or as fp32 rows (v_mfma_f32_32x32x2_f32, every product exact to fp32).
#pragma once
#include "agpu_internal.h"

constexpr int kDenseGemvRows = 4;    // rows the fp32 GEMV takes
constexpr int kDenseSkinnyRows = 32; // rows the K-split bf16 kernel takes

__device__ __forceinline__ float bf16_to_f32(uint16_t v) { return __uint_as_float((uint32_t)v << 16); }
// Round to nearest even; NaN stays NaN.
__device__ __forceinline__ uint16_t f32_to_bf16(float v) {
    const uint32_t u = __float_as_uint(v);
    if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x40u);
    return (uint16_t)((u + 0x7fffu + ((u >> 16) & 1u)) >> 16);
}
__device__ __forceinline__ float silu_dev(float v) { return v / (1.0f + expf(-v)); }
__device__ __forceinline__ float sigmoid_dev(float v) { return 1.0f / (1.0f + expf(-v)); }

// Where the outputs of a dense Linear go.  Columns [0, n_plain) are plain; the columns behind them are pairs (gate, up)
// of a gated feed-forward, column n_plain + 2 j and n_plain + 2 j + 1, and leave as act[m][j] = silu(gate) * up, or with
// act_limit > 0 as g sigmoid(1.702 g) (u + 1) with g = min(gate, act_limit), u = up clamped to +- act_limit.
struct DenseOut {
    int n_plain = 0;
    float *out = nullptr;         // fp32, row stride ldo
    uint16_t *out_bf16 = nullptr; // bf16 instead, row stride ldo
    int ldo = 0;
    const float *bias = nullptr;      // [n_plain]
    const float *residual = nullptr;  // row stride ldr; may alias out
    int ldr = 0;
    // per-token table: out = gelu_tanh(v) * table[token of row m][tab_off + n] for n < tab_n, 0 beyond
    const uint16_t *tab = nullptr;
    const uint32_t *tokens = nullptr;
    int tab_ld = 0, tab_off = 0, tab_n = 0, vocab = 0;
    void *act = nullptr;  // bf16 or fp32, row stride ld_act
    int ld_act = 0, act_bf16 = 0;
    float act_limit = 0.0f;
};

// What happens to the fp32 input rows in front of a Linear (and, in dense_rows_launch, on their own):
//   x <- x + y / rms(y) * y_w                 (y != null: an RMS-normed addend with a plain weight)
//   x <- x + add + add_vec                    (add, add_vec: each if not null; a row per row, one vector for all)
//   h  = x / rms(x) * (norm_off + norm_w)     (norm_w != null)
//   the Linear's input is [h | x2]            (x2 != null)
// or, with gate: h = x / rms(x) * norm_w * sigmoid(gate), where the row is `groups` groups of group_p columns, of which the
// first group_d count for the group's own rms (the rest is zero); nothing else applies then.
// rms(z) = sqrt(mean(z^2) + eps) over the first d columns; columns d .. dp - 1 are zero everywhere.
struct DenseRows {
    const float *x = nullptr;
    int ldx = 0;
    int d = 0, dp = 0;
    const float *y = nullptr, *y_w = nullptr;  // row stride ldx
    float *x_out = nullptr;                    // the updated x (may not alias x in a GEMV: other workgroups still read x)
    const float *norm_w = nullptr;
    float norm_off = 0.0f, eps = 0.0f;
    const float *x2 = nullptr;                 // row stride ldx, dp columns
    const float *add = nullptr, *add_vec = nullptr;  // row stride ldx; [d]
    const float *gate = nullptr;               // row stride ld_gate, same columns as x
    int ld_gate = 0, groups = 0, group_d = 0, group_p = 0;
    // Row m of the input is row map_stride * (m + 1) - 1 of x and y when map_stride > 0 (the last token of each sequence).
    int map_stride = 0;
};

// M <= kDenseGemvRows rows.  K = dp (+ dp with x2), a multiple of 32.
int32_t dense_gemv_launch(agpu_ctx *ctx, const DenseRows &in, const uint16_t *w, int M, int N, int K, const DenseOut &o);
bool dense_gemv_supported(int M, int K);
// The rows on their own: h as fp32 or bf16 [M, ldh] (h [.., x2] as above), for the matrix-core kernels.
int32_t dense_rows_launch(agpu_ctx *ctx, const DenseRows &in, int M, void *h, int ldh, int h_bf16);
// y = A W^T on the matrix cores, A [M, K] with row stride lda, W with row stride ldw.  K % 32 == 0, lda % 8 == 0,
// ldw % 8 == 0, 16-byte aligned.  bf16 A:
int32_t dense_gemm_bf16_launch(agpu_ctx *ctx, const uint16_t *a, int lda, const uint16_t *w, int ldw, int M, int N, int K, const DenseOut &o);
// fp32 A; with `blocks` > 1 a block-diagonal Linear: block b reads columns b K .. of A and rows b N .. of W, and its outputs
// (plain only) are columns b N ...
int32_t dense_gemm_f32_launch(agpu_ctx *ctx, const float *a, int lda, const uint16_t *w, int ldw, int M, int N, int K, const DenseOut &o, int blocks = 1);
