// What every language model of this library shares around its own forward: device-side generation state (current
// token, positions, recorded tokens), the decode loop as replayed HIP graphs, greedy generation and sampling, and the
// owned buffers.  A model derives from LmRuntime, supplies its forward over cached positions, and its C entry points
// call the lm_* functions.  A cache or a recurrent state belongs to the model; `cache_len` positions of it are filled.
#pragma once
#include <map>
#include <vector>

#include "agpu_internal.h"
#include "elementwise.h"

struct DevBuf {
    void *p = nullptr;
    size_t bytes = 0;
};

// Folds device addresses into one word (see LmRuntime::mix_addresses).
struct AddrHash {
    unsigned long long h = 1469598103934665603ull;
    void mix(const void *p) { h = (h ^ (unsigned long long)(uintptr_t)p) * 1099511628211ull; }
};

struct LmRuntime {
    explicit LmRuntime(const char *model_name) : name(model_name) {}
    LmRuntime(const LmRuntime &) = delete;
    virtual ~LmRuntime() {}

    const char *name;
    agpu_ctx *ctx = nullptr;
    int V = 0, P = 0;  // vocabulary, positions the cache holds
    int max_batch = 1, argmax_last = 0;
    int cache_len = 0;
    DevBuf logits, tok_in;
    uint32_t *cur_tok = nullptr, *next_tok = nullptr, *out_tok = nullptr;
    int out_capacity = 0;  // steps recorded in out_tok
    int *pos_dev = nullptr, *step_dev = nullptr;
    std::map<long long, hipGraphExec_t> graphs;          // key: batch << 32 | kv bucket
    std::map<long long, unsigned long long> graph_addr;  // per graph: fingerprint of the device addresses it was captured with
    unsigned long long ws_epoch = 0;                     // the context's scratch the graphs were captured with
    hipEvent_t ev0 = nullptr, ev1 = nullptr, ev2 = nullptr;
    int decode_mode = 0;                        // AGPU_DECODE_*
    long long n_one_launch = 0, n_per_stage = 0;  // decode steps by the way they went

    // ---- what a model supplies ----
    virtual int32_t check_ready() = 0;  // every weight is set
    virtual int32_t ensure_buffers(int B, int new_len, bool all_rows_logits) = 0;
    virtual int logits_stride() const = 0;
    // One forward over `new_len` tokens per sequence at positions *pos_dev ..., logits into `logits`; max_kv bounds the
    // cached length afterwards.  With `feed` (single row only) the launch may also pick the arg-max and feed it back.
    virtual int32_t launch_forward(const uint32_t *tokens, int B, int new_len, int max_kv, bool all_rows_logits, const ArgmaxAdvance *feed,
                                   bool *fed) = 0;
    // Every device address a decode step refers to.
    virtual void mix_addresses(AddrHash &h, bool one_launch) const = 0;
    virtual int32_t reset_state() { return AGPU_OK; }     // recurrent state back to the start of a sequence
    virtual void graphs_dropped() {}                      // the captured graphs are gone: so is whatever shares their addresses
    virtual int32_t prepare_steps(int) { return AGPU_OK; }  // before decode steps of that batch are launched or captured
    // A decode step as one launch, where a model has one.
    virtual bool one_launch_ready() { return false; }
    virtual bool one_launch_planned() const { return false; }
    virtual int32_t launch_one_step() { return AGPU_ERR_UNSUPPORTED; }
    virtual int32_t check_waits() { return AGPU_OK; }  // after a synchronisation: did a bounded wait give up
};

// ---- owned memory ----
int32_t dev_alloc(agpu_ctx *ctx, void **p, size_t bytes);
int32_t upload(agpu_ctx *ctx, void *dst, const void *src, size_t bytes, int on_device);
int32_t fill_u32(agpu_ctx *ctx, void *p, uint32_t v, size_t words);  // capturable, unlike a memset node
int32_t ensure(LmRuntime *m, DevBuf &b, size_t bytes);  // grows a buffer; graphs that hold the old address are dropped
void drop_graphs(LmRuntime *m);

// ---- generation state and loop ----
int32_t lm_init(LmRuntime *m, agpu_ctx *ctx, int vocab, int positions, int max_batch, int argmax_last);
void lm_release(LmRuntime *m);  // frees the runtime's own memory, graphs and events, and the reference on the context
int32_t check_token_ids(LmRuntime *m, const uint32_t *ids_host, size_t n, const char *who);
int32_t set_counters(LmRuntime *m, int pos, int step);
ArgmaxAdvance token_feed(const LmRuntime *m, int B, int delta);
int32_t launch_argmax_advance(LmRuntime *m, int B, int delta);
int kv_bucket(const LmRuntime *m, int kv_len);
int32_t ensure_out_tokens(LmRuntime *m, int steps);
int32_t run_decode_steps(LmRuntime *m, int B, int steps);

// ---- bodies of the models' entry points ----
int32_t lm_reset_cache(LmRuntime *m);
int32_t lm_forward_cached(LmRuntime *m, const uint32_t *tokens, int32_t batch, int32_t new_len, float *logits, int32_t all_rows);
int32_t lm_decode_steps(LmRuntime *m, int32_t batch, int32_t steps, float *ms_total_out_host);
int32_t lm_last_logits(LmRuntime *m, int32_t batch, float *logits_out_host);
int32_t lm_set_decode_mode(LmRuntime *m, int32_t mode);
int32_t lm_generate_cached(LmRuntime *m, const uint32_t *prompt_host, int32_t batch, int32_t prompt_len, int32_t max_new_tokens, int32_t eos,
                           uint32_t *tokens_out_host, int32_t *lengths_out_host, float *timing_ms_out_host);
int32_t lm_generate_cached_sampling(LmRuntime *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens, int32_t top_k,
                                    float temperature, uint64_t *rng_state, int32_t eos, uint32_t *tokens_out_host, int32_t *length_out_host);
int32_t lm_generate(LmRuntime *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens, int32_t eos,
                    uint32_t *tokens_out_host, int32_t *length_out_host);
