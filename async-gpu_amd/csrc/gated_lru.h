// Real-gated linear recurrent unit (the recurrent block of Griffin).  Two branches of `width` channels: y, which gates the output
// through gelu, and x, which passes a short causal convolution.  With u the convolution's output, block-diagonal maps give
// r = sigmoid(R u + b_r) and i = sigmoid(I u + b_i); per channel log a = -8 r softplus(lam), S <- a S + sqrt(1 - a^2) i u, and
// the output is S gelu(y).  Everything behind the projections is fp32.
#pragma once
#include "agpu_internal.h"
#include "dense_linear.h"

struct LruShape {
    int width = 0, blocks = 0, taps = 0;
    int block() const { return width / blocks; }
    int blockp() const { return (block() + 31) / 32 * 32; }  // storage width of a block, in projections, weights, state and output
    int widthp() const { return blocks * blockp(); }
};

struct LruWeights {
    const float *conv = nullptr, *conv_bias = nullptr;  // [widthp][taps], last tap is the current token's; [widthp]
    const uint16_t *gates = nullptr;                    // [blocks][R | I][blockp][blockp], zero padded
    const float *gate_bias = nullptr;                   // [blocks][2][blockp]
    const float *lam = nullptr;                         // [widthp]
};

struct LruArgs {
    LruShape s;
    LruWeights w;
    const float *proj = nullptr;  // rows [batch * new_len], stride ld, with y and x (biases added) at these columns
    int ld = 0, col_y = 0, col_x = 0;
    float *state = nullptr;  // [batch][widthp]
    float *ring = nullptr;   // [batch][taps][widthp]: convolution inputs of the last tokens
    int batch = 1, new_len = 1;
    const int *pos_dev = nullptr;
    void *out = nullptr;  // rows, stride ldo: widthp, bf16 or fp32
    int ldo = 0, out_bf16 = 0;
    // scratch of the many-token form
    float *u = nullptr;        // [rows][widthp]
    float *gates = nullptr;    // [rows][2 widthp]
    float *carries = nullptr;  // lru_carry_floats
};

bool lru_supported(const LruShape &s);
size_t lru_carry_floats(const LruShape &s, int batch, int new_len);
// One new token per sequence in one launch, or any number.
int32_t lru_launch(agpu_ctx *ctx, const LruArgs &a);
