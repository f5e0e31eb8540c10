/*
 * agpu_ritevik.h — C ABI of the Ritevik model driver in libagpu_hip.so.
 *
 * Ritevik is a decoder-only language model that no library of the reference has: a stack of parallel blocks (one RMS
 * norm, mixer and gated feed-forward side by side), mixers of two kinds (latent attention with a learned sink, a gated
 * delta rule with one decay per key channel), an optional loop that runs a part of the stack several times with a step
 * vector and the embedding output mixed in, and an optional per-layer token input behind every block.
 *
 * The driver shares the generation runtime of agpu_gpt2.h: device-resident cache, one forward over cached positions for
 * prompts, portions of prompts and decode steps, decode steps replayed as HIP graphs with arg-max and token feed on the
 * device, greedy generation and top-k sampling.  `batch` sequences of equal length advance together.  What a sequence
 * holds: per run of an attention layer the latents and rotated key parts of its positions, per run of a delta layer one
 * fp32 state and the last inputs of its short convolution.  A layer inside the loop has one of these per pass.
 *
 * Weights are bf16 on the device.  With AGPU_DTYPE_BF16 prompts run on the bf16 matrix cores (fp32 accumulation) and
 * the latent cache is bf16; with AGPU_DTYPE_F32 activations, products and cache are fp32.  In both, the residual stream,
 * norms, angles, attention scores and softmax, recurrent state, decays and gates of the recurrence are fp32.
 *
 * Same conventions as agpu.h.  One model is used by one thread at a time.
 */
#ifndef AGPU_RITEVIK_H
#define AGPU_RITEVIK_H

#include "agpu_gpt2.h"

#ifdef __cplusplus
extern "C" {
#endif

typedef struct agpu_ritevik agpu_ritevik;

#define AGPU_MIXER_LATENT_ATTENTION 0
#define AGPU_MIXER_CHANNEL_DELTA 1

typedef struct agpu_ritevik_config {
    int32_t n_layer, width, vocab_size, n_positions, max_batch;
    float norm_eps;
    int32_t loop_start, loop_stop, loop_times; /* layers [start, stop) run `times` times; times 0: no loop */
    int32_t side_dim;                          /* size of the per-layer token input; 0: none */
    int32_t dtype;                             /* AGPU_DTYPE_* */
    int32_t argmax_last;                       /* tie rule of greedy decoding, as in agpu_gpt2_config */
} agpu_ritevik_config;

typedef struct agpu_ritevik_layer {
    int32_t mixer; /* AGPU_MIXER_* */
    int32_t heads, dim, vdim;
    int32_t ff; /* 0: no feed-forward */
    /* latent attention */
    int32_t kv_rank, rot_dim, rot_dims;
    float scale;
    double rot_base;
    /* channel delta */
    int32_t kv_heads, conv, decay_rank, gate_rank;
} agpu_ritevik_layer;

/* layers: HOST array of cfg->n_layer entries. */
int32_t agpu_ritevik_create(agpu_ctx *ctx, const agpu_ritevik_config *cfg, const agpu_ritevik_layer *layers, agpu_ritevik **out);
int32_t agpu_ritevik_destroy(agpu_ritevik *m);

/* One weight tensor by its name in the model file ("embed", "l0.mix.q", ...), HOST data, dtype AGPU_DTYPE_* (an fp32 matrix
 * is rounded to bf16).  rows x cols as in the file; a vector has rows = 1.  AGPU_ERR_KERNEL_NOT_FOUND for a name the
 * configuration does not have, AGPU_ERR_SHAPE_MISMATCH for another shape. */
int32_t agpu_ritevik_set_tensor(agpu_ritevik *m, const char *name, const void *data_host, int32_t dtype, int64_t rows, int64_t cols);
/* The i-th tensor the configuration needs: its name (valid as long as the model) and shape; AGPU_ERR_DIM_OUT_OF_RANGE past
 * the last one.  *is_set_out: whether it has been set. */
int32_t agpu_ritevik_tensor_info(const agpu_ritevik *m, int32_t i, const char **name_out, int64_t *rows_out, int64_t *cols_out, int32_t *is_set_out);

/* Device bytes of the weights / of cache and state. */
int64_t agpu_ritevik_weight_bytes(const agpu_ritevik *m);
int64_t agpu_ritevik_cache_bytes(const agpu_ritevik *m);
/* Layer runs of one forward: a looped layer counts once per pass. */
int32_t agpu_ritevik_layer_runs(const agpu_ritevik *m);

/* The calls below behave as their namesakes in agpu_gpt2.h. */
int32_t agpu_ritevik_reset_cache(agpu_ritevik *m);
int32_t agpu_ritevik_cache_len(const agpu_ritevik *m);
int32_t agpu_ritevik_forward_cached(agpu_ritevik *m, const uint32_t *tokens, int32_t batch, int32_t new_len, float *logits, int32_t all_rows);
int32_t agpu_ritevik_generate_cached(agpu_ritevik *m, const uint32_t *prompt_host, int32_t batch, int32_t prompt_len, int32_t max_new_tokens,
                                     int32_t eos, uint32_t *tokens_out_host, int32_t *lengths_out_host, float *timing_ms_out_host);
int32_t agpu_ritevik_generate(agpu_ritevik *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens, int32_t eos,
                              uint32_t *tokens_out_host, int32_t *length_out_host);
int32_t agpu_ritevik_generate_cached_sampling(agpu_ritevik *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens,
                                              int32_t top_k, float temperature, uint64_t *rng_state, int32_t eos, uint32_t *tokens_out_host,
                                              int32_t *length_out_host);
/* AGPU_DECODE_AUTO and AGPU_DECODE_PER_STAGE are the same here: one launch per stage, replayed as a HIP graph. */
int32_t agpu_ritevik_set_decode_mode(agpu_ritevik *m, int32_t mode);
int32_t agpu_ritevik_decode_steps(agpu_ritevik *m, int32_t batch, int32_t steps, float *ms_total_out_host);
int32_t agpu_ritevik_last_logits(agpu_ritevik *m, int32_t batch, float *logits_out_host);
/* forward_cached over one sequence's new tokens (DEVICE pointer) that also returns the residual stream after every layer
 * run: streams_out_host [layer runs][new_len][width]. */
int32_t agpu_ritevik_layer_streams(agpu_ritevik *m, const uint32_t *tokens, int32_t new_len, float *streams_out_host);

#ifdef __cplusplus
}
#endif
#endif /* AGPU_RITEVIK_H */
