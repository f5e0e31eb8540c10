/*
 * agpu_piralix.h — C ABI of the Piralix model driver in libagpu_hip.so.
 *
 * Piralix is a decoder-only language model that no library of the reference has: a stack of layers with an RMS norm before
 * and after each sublayer, mixers of three kinds (a matrix memory with exponential gates, grouped attention with capped
 * scores, a sink and an output gate, a real-gated linear recurrent unit), an optional clipped feed-forward per layer, and an
 * optional loop that runs a part of the stack several times, with a step vector and the embedding output added in front of a
 * pass.  The output reuses the embedding table.
 *
 * The driver shares the generation runtime of agpu_gpt2.h, as agpu_ritevik.h does.  `batch` sequences of equal length advance
 * together.  What a sequence holds, per layer run (a layer inside the loop has one of these per pass): keys and values of its
 * positions, or the memory's state, normaliser and running maximum, or the recurrent state and the last inputs of the short
 * convolution.
 *
 * Weights are bf16 on the device.  With AGPU_DTYPE_BF16 prompts run on the bf16 matrix cores (fp32 accumulation) and keys and
 * values are cached in bf16; with AGPU_DTYPE_F32 activations, products and cache are fp32.  In both, the residual stream,
 * norms, angles, attention scores and softmax, recurrent state, and all gates, decays and products of the recurrences are fp32.
 *
 * Same conventions as agpu.h.  One model is used by one thread at a time.
 */
#ifndef AGPU_PIRALIX_H
#define AGPU_PIRALIX_H

#include "agpu_gpt2.h"

#ifdef __cplusplus
extern "C" {
#endif

typedef struct agpu_piralix agpu_piralix;

#define AGPU_MIXER_MATRIX_MEMORY 2
#define AGPU_MIXER_GROUPED_ATTENTION 3
#define AGPU_MIXER_GATED_LRU 4

typedef struct agpu_piralix_config {
    int32_t n_layer, width, vocab_size, n_positions, max_batch;
    float norm_eps;
    int32_t loop_start, loop_stop, loop_times; /* layers [start, stop) run `times` times; times 0: no loop */
    int32_t dtype;                             /* AGPU_DTYPE_* */
    int32_t argmax_last;                       /* tie rule of greedy decoding, as in agpu_gpt2_config */
} agpu_piralix_config;

typedef struct agpu_piralix_layer {
    int32_t mixer;            /* AGPU_MIXER_* */
    int32_t heads, dim, vdim; /* matrix memory and attention; at most 256 dimensions a head (vdim of a matrix memory: any) */
    int32_t ff;               /* 0: no feed-forward */
    float ff_limit;           /* > 0: clip of the feed-forward */
    /* matrix memory */
    float gate_cap;
    /* grouped attention; softcap 0: none; rot_factor 0: plain rotation, else stretched by that factor */
    float scale, softcap;
    int32_t kv_heads, rot_dims;
    double rot_base, rot_factor, rot_original, rot_fast, rot_slow;
    /* gated linear recurrent unit */
    int32_t lru_width, blocks, conv;
} agpu_piralix_layer;

/* layers: HOST array of cfg->n_layer entries. */
int32_t agpu_piralix_create(agpu_ctx *ctx, const agpu_piralix_config *cfg, const agpu_piralix_layer *layers, agpu_piralix **out);
int32_t agpu_piralix_destroy(agpu_piralix *m);

/* One weight tensor by its name in the model file, as agpu_ritevik_set_tensor; a tensor of three dimensions has the first two
 * as its rows. */
int32_t agpu_piralix_set_tensor(agpu_piralix *m, const char *name, const void *data_host, int32_t dtype, int64_t rows, int64_t cols);
int32_t agpu_piralix_tensor_info(const agpu_piralix *m, int32_t i, const char **name_out, int64_t *rows_out, int64_t *cols_out, int32_t *is_set_out);

/* Device bytes of the weights / of cache and state. */
int64_t agpu_piralix_weight_bytes(const agpu_piralix *m);
int64_t agpu_piralix_cache_bytes(const agpu_piralix *m);
/* Layer runs of one forward: a looped layer counts once per pass. */
int32_t agpu_piralix_layer_runs(const agpu_piralix *m);

/* The calls below behave as their namesakes in agpu_gpt2.h and agpu_ritevik.h. */
int32_t agpu_piralix_reset_cache(agpu_piralix *m);
int32_t agpu_piralix_cache_len(const agpu_piralix *m);
int32_t agpu_piralix_forward_cached(agpu_piralix *m, const uint32_t *tokens, int32_t batch, int32_t new_len, float *logits, int32_t all_rows);
int32_t agpu_piralix_generate_cached(agpu_piralix *m, const uint32_t *prompt_host, int32_t batch, int32_t prompt_len, int32_t max_new_tokens,
                                     int32_t eos, uint32_t *tokens_out_host, int32_t *lengths_out_host, float *timing_ms_out_host);
int32_t agpu_piralix_generate(agpu_piralix *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens, int32_t eos,
                              uint32_t *tokens_out_host, int32_t *length_out_host);
int32_t agpu_piralix_generate_cached_sampling(agpu_piralix *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens,
                                              int32_t top_k, float temperature, uint64_t *rng_state, int32_t eos, uint32_t *tokens_out_host,
                                              int32_t *length_out_host);
int32_t agpu_piralix_set_decode_mode(agpu_piralix *m, int32_t mode);
int32_t agpu_piralix_decode_steps(agpu_piralix *m, int32_t batch, int32_t steps, float *ms_total_out_host);
int32_t agpu_piralix_last_logits(agpu_piralix *m, int32_t batch, float *logits_out_host);
int32_t agpu_piralix_layer_streams(agpu_piralix *m, const uint32_t *tokens, int32_t new_len, float *streams_out_host);

#ifdef __cplusplus
}
#endif
#endif /* AGPU_PIRALIX_H */
