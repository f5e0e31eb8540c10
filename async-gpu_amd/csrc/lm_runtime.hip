// The generation runtime shared by the models: device-side generation state, the decode step replayed as a HIP graph
// (arg-max and token feed stay on the device, so a step needs no host round trip), greedy generation and sampling.
// Control flow: forward_cached / generate_cached / generate_cached_sampling (nn/models/gpt2.rs:712-783, 931-977) and
// generate (gpt2.rs:1536-1560).
#include <algorithm>
#include <cstring>

#include "../../include/agpu_gpt2.h"
#include "lm_runtime.h"

namespace {

__global__ void advance_counters_kernel(int *pos_dev, int *step_dev, int delta) {
    *pos_dev += delta;
    *step_dev += 1;
}

__global__ void set_counters_kernel(int *pos_dev, int pos, int *step_dev, int step) {
    *pos_dev = pos;
    if (step >= 0) *step_dev = step;
}

__global__ __launch_bounds__(256) void fill_u32_kernel(uint32_t *p, uint32_t v, size_t n) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i < n) p[i] = v;
}

// Every device address a decode step refers to, folded into one word.  A captured graph holds these addresses; a
// replay is only right while they are still the model's.  Every path that frees or moves one of them drops the graphs
// (ensure, ensure_out_tokens, the weight setters, a new scratch); this is the check behind that rule.
unsigned long long step_addresses(const LmRuntime *m, bool one_launch) {
    AddrHash h;
    for (const void *p : {(const void *)m->cur_tok, (const void *)m->next_tok, (const void *)m->out_tok, (const void *)m->pos_dev,
                          (const void *)m->step_dev, (const void *)m->ctx->workspace, (const void *)m->ctx->counters,
                          (const void *)m->logits.p, (const void *)m->tok_in.p})
        h.mix(p);
    m->mix_addresses(h, one_launch);
    return h.h;
}

// One decode step as one launch per stage; the LM head picks and feeds the next token itself where it can.
int32_t launch_step_per_stage(LmRuntime *m, int B, int bucket) {
    const ArgmaxAdvance feed = token_feed(m, B, 1);
    bool fed = false;
    int32_t rc = m->launch_forward(m->cur_tok, B, 1, bucket, false, &feed, &fed);
    if (rc == AGPU_OK && !fed) rc = launch_argmax_advance(m, B, 1);
    return rc;
}

// The captured decode step for (batch, kv bucket); captured on first use.
// The one-launch step reads the position on the device and does not depend on the bucket: `reps` > 1 captures that many
// of its launches in a row (one graph launch then costs its overhead once for `reps` tokens).
int32_t decode_graph(LmRuntime *m, int B, int bucket, hipGraphExec_t *out, int reps = 1) {
    const long long key = reps > 1 ? ((1ll << 62) | reps) : (((long long)B << 32) | (unsigned)bucket);
    if (m->ws_epoch != m->ctx->ws_epoch) {  // the scratch moved: captured launches point at the old one
        drop_graphs(m);
        m->ws_epoch = m->ctx->ws_epoch;
    }
    auto it = m->graphs.find(key);
    if (it != m->graphs.end()) {
        if (m->graph_addr[key] == step_addresses(m, reps > 1 || (B == 1 && m->one_launch_planned()))) {
            *out = it->second;
            return AGPU_OK;
        }
        // an address changed under a cached graph: never replay it; every graph goes and this one is captured anew
        drop_graphs(m);
    }
    agpu_ctx *ctx = m->ctx;
    if (ctx->stream == nullptr)
        return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "%s: graph capture needs a context with its own stream (agpu_ctx_create)", m->name);
    const bool one_launch = B == 1 && m->one_launch_ready();  // builds the plan: before the capture begins
    hipError_t e = hipStreamBeginCapture(ctx->stream, hipStreamCaptureModeThreadLocal);
    if (e != hipSuccess) return agpu_hip(ctx, e, "hipStreamBeginCapture");
    int32_t rc;
    if (one_launch) {
        // one sequence: the whole step, arg-max and token feed included, is one launch
        rc = AGPU_OK;
        for (int r = 0; r < reps && rc == AGPU_OK; ++r) rc = m->launch_one_step();
    } else if (reps > 1) {
        rc = agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "%s: several steps per graph need the one-launch step", m->name);
    } else {
        rc = launch_step_per_stage(m, B, bucket);
    }
    hipGraph_t graph = nullptr;
    e = hipStreamEndCapture(ctx->stream, &graph);
    if (rc != AGPU_OK) {
        if (graph) (void)hipGraphDestroy(graph);
        return rc;
    }
    if (e != hipSuccess) return agpu_hip(ctx, e, "hipStreamEndCapture");
    hipGraphExec_t exec = nullptr;
    e = hipGraphInstantiate(&exec, graph, nullptr, nullptr, 0);
    (void)hipGraphDestroy(graph);
    if (e != hipSuccess) return agpu_hip(ctx, e, "hipGraphInstantiate");
    m->graphs[key] = exec;
    m->graph_addr[key] = step_addresses(m, one_launch);
    *out = exec;
    return AGPU_OK;
}

}  // namespace

int32_t dev_alloc(agpu_ctx *ctx, void **p, size_t bytes) {
    hipError_t e = hipMalloc(p, bytes);
    if (e != hipSuccess) return agpu_hip(ctx, e, "hipMalloc");
    return AGPU_OK;
}

int32_t upload(agpu_ctx *ctx, void *dst, const void *src, size_t bytes, int on_device) {
    hipError_t e = hipMemcpyAsync(dst, src, bytes, on_device ? hipMemcpyDeviceToDevice : hipMemcpyHostToDevice, ctx->stream);
    if (e != hipSuccess) return agpu_hip(ctx, e, "hipMemcpyAsync");
    // host sources may be freed by the caller right after the call returns
    if (!on_device) return agpu_hip(ctx, hipStreamSynchronize(ctx->stream), "hipStreamSynchronize");
    return AGPU_OK;
}

int32_t fill_u32(agpu_ctx *ctx, void *p, uint32_t v, size_t words) {
    if (words == 0) return AGPU_OK;
    hipLaunchKernelGGL(fill_u32_kernel, dim3((unsigned)((words + 255) / 256)), dim3(256), 0, ctx->stream, (uint32_t *)p, v, words);
    return AGPU_LAUNCH_CHECK(ctx, "fill_u32_kernel");
}

void drop_graphs(LmRuntime *m) {
    // a replay still on the stream must not lose its graph, nor the plan its arena
    if (m->ctx && !m->graphs.empty()) (void)hipStreamSynchronize(m->ctx->stream);
    for (auto &kv : m->graphs) (void)hipGraphExecDestroy(kv.second);
    m->graphs.clear();
    m->graph_addr.clear();
    m->graphs_dropped();
}

// Grow a buffer; existing graphs hold the old address, so they are dropped.
int32_t ensure(LmRuntime *m, DevBuf &b, size_t bytes) {
    if (b.bytes >= bytes) return AGPU_OK;
    (void)hipStreamSynchronize(m->ctx->stream);
    drop_graphs(m);
    if (b.p) (void)hipFree(b.p);
    b.p = nullptr;
    b.bytes = 0;
    int32_t rc = dev_alloc(m->ctx, &b.p, bytes);
    if (rc != AGPU_OK) return rc;
    b.bytes = bytes;
    return AGPU_OK;
}

int32_t lm_init(LmRuntime *m, agpu_ctx *ctx, int vocab, int positions, int max_batch, int argmax_last) {
    m->ctx = ctx;
    ctx->refs.fetch_add(1);
    m->V = vocab;
    m->P = positions;
    m->max_batch = max_batch;
    m->argmax_last = argmax_last;
    int32_t rc = dev_alloc(ctx, (void **)&m->cur_tok, (size_t)max_batch * 4);
    if (rc == AGPU_OK) rc = dev_alloc(ctx, (void **)&m->next_tok, (size_t)max_batch * 4);
    if (rc == AGPU_OK) rc = dev_alloc(ctx, (void **)&m->pos_dev, 2 * sizeof(int));
    if (rc == AGPU_OK) {
        m->step_dev = m->pos_dev + 1;
        rc = agpu_hip(ctx, hipMemset(m->pos_dev, 0, 2 * sizeof(int)), "hipMemset");
    }
    for (hipEvent_t *e : {&m->ev0, &m->ev1, &m->ev2})
        if (rc == AGPU_OK) rc = agpu_hip(ctx, hipEventCreate(e), "hipEventCreate");
    return rc;
}

void lm_release(LmRuntime *m) {
    drop_graphs(m);
    for (void *p : {(void *)m->cur_tok, (void *)m->next_tok, (void *)m->out_tok, (void *)m->pos_dev, m->logits.p, m->tok_in.p})
        if (p) (void)hipFree(p);
    for (hipEvent_t e : {m->ev0, m->ev1, m->ev2})
        if (e) (void)hipEventDestroy(e);
    agpu_ctx_release(m->ctx);
}

// Token ids the host can see are checked before anything is launched.
int32_t check_token_ids(LmRuntime *m, const uint32_t *ids_host, size_t n, const char *who) {
    for (size_t i = 0; i < n; ++i)
        if (ids_host[i] >= (uint32_t)m->V)
            return agpu_fail(m->ctx, AGPU_ERR_DIM_OUT_OF_RANGE, "%s: token id %u at index %zu is outside the vocabulary of %d", who,
                             ids_host[i], i, m->V);
    return AGPU_OK;
}

int32_t set_counters(LmRuntime *m, int pos, int step) {
    hipLaunchKernelGGL(set_counters_kernel, dim3(1), dim3(1), 0, m->ctx->stream, m->pos_dev, pos, m->step_dev, step);
    return AGPU_LAUNCH_CHECK(m->ctx, "set_counters_kernel");
}

ArgmaxAdvance token_feed(const LmRuntime *m, int B, int delta) {
    ArgmaxAdvance adv{};
    adv.cur_tok = m->cur_tok; adv.out_tok = m->out_tok; adv.pos_dev = m->pos_dev; adv.step_dev = m->step_dev;
    adv.delta = delta; adv.out_capacity = m->out_capacity; adv.bump_counters = (B == 1);
    return adv;
}

int32_t launch_argmax_advance(LmRuntime *m, int B, int delta) {
    const ArgmaxAdvance adv = token_feed(m, B, delta);
    int32_t rc = agpu_argmax_rows_strided(m->ctx, (float *)m->logits.p, m->next_tok, B, m->V, m->logits_stride(),
                                          m->argmax_last, &adv);
    if (rc != AGPU_OK || B == 1) return rc;
    // several rows: the counters advance once every row has read them
    hipLaunchKernelGGL(advance_counters_kernel, dim3(1), dim3(1), 0, m->ctx->stream, m->pos_dev, m->step_dev, delta);
    return AGPU_LAUNCH_CHECK(m->ctx, "advance_counters_kernel");
}

int kv_bucket(const LmRuntime *m, int kv_len) {
    int b = 128;
    while (b < kv_len) b *= 2;
    return b < m->P ? b : m->P;
}

int32_t ensure_out_tokens(LmRuntime *m, int steps) {
    if (m->out_capacity >= steps && m->out_tok) return AGPU_OK;
    (void)hipStreamSynchronize(m->ctx->stream);
    drop_graphs(m);
    if (m->out_tok) (void)hipFree(m->out_tok);
    m->out_tok = nullptr;
    const int cap = steps > m->P ? steps : m->P;
    int32_t rc = dev_alloc(m->ctx, (void **)&m->out_tok, (size_t)cap * m->max_batch * sizeof(uint32_t));
    if (rc != AGPU_OK) return rc;
    m->out_capacity = cap;
    return AGPU_OK;
}

// Replays `steps` decode steps; the host only tracks the position to pick the graph.
int32_t run_decode_steps(LmRuntime *m, int B, int steps) {
    constexpr int kStepsPerGraph = 16;  // lm_decode_steps captures the same number ahead of its timed region
    // what a step of this batch needs must exist before it is launched or captured
    const int32_t prc = m->prepare_steps(B);
    if (prc != AGPU_OK) return prc;
    int s = 0;
    if (B == 1 && steps >= 2 && m->one_launch_ready()) {
        // graphs of sixteen launches, then one graph of what is left (a graph launch costs 5.5 us, a node inside one 1.5)
        while (s < steps) {
            const int n = std::min(kStepsPerGraph, steps - s);
            if (n < 2) break;
            hipGraphExec_t exec;
            const int32_t rc = decode_graph(m, 1, 0, &exec, n);
            if (rc != AGPU_OK) return rc;
            const hipError_t e = hipGraphLaunch(exec, m->ctx->stream);
            if (e != hipSuccess) return agpu_hip(m->ctx, e, "hipGraphLaunch");
            m->cache_len += n;
            m->n_one_launch += n;
            s += n;
        }
    }
    for (; s < steps; ++s) {
        const int bucket = kv_bucket(m, m->cache_len + 1);
        if (B == 1 && m->one_launch_ready()) ++m->n_one_launch;
        else ++m->n_per_stage;
        if (m->decode_mode == AGPU_DECODE_EAGER) {
            const int32_t rc = launch_step_per_stage(m, B, bucket);
            if (rc != AGPU_OK) return rc;
        } else {
            hipGraphExec_t exec;
            const int32_t rc = decode_graph(m, B, bucket, &exec);
            if (rc != AGPU_OK) return rc;
            const hipError_t e = hipGraphLaunch(exec, m->ctx->stream);
            if (e != hipSuccess) return agpu_hip(m->ctx, e, "hipGraphLaunch");
        }
        m->cache_len += 1;
    }
    return AGPU_OK;
}

int32_t lm_reset_cache(LmRuntime *m) {
    m->cache_len = 0;
    const int32_t rc = m->reset_state();
    return rc == AGPU_OK ? set_counters(m, 0, 0) : rc;
}

int32_t lm_set_decode_mode(LmRuntime *m, int32_t mode) {
    if (mode != AGPU_DECODE_AUTO && mode != AGPU_DECODE_PER_STAGE && mode != AGPU_DECODE_EAGER)
        return agpu_fail(m->ctx, AGPU_ERR_DIM_OUT_OF_RANGE, "%s_set_decode_mode: unknown mode %d", m->name, mode);
    if (mode != m->decode_mode) {
        (void)hipStreamSynchronize(m->ctx->stream);
        drop_graphs(m);
        m->decode_mode = mode;
    }
    return AGPU_OK;
}

int32_t lm_forward_cached(LmRuntime *m, const uint32_t *tokens, int32_t batch, int32_t new_len,
                                             float *logits, int32_t all_rows) {
    agpu_ctx *ctx = m->ctx;
    AGPU_REQUIRE_CTX(ctx);
    if (!tokens) return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "%s_forward_cached: null tokens", m->name);
    if (batch <= 0 || batch > m->max_batch)
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "%s_forward_cached: batch %d not in 1..%d", m->name, batch, m->max_batch);
    if (new_len <= 0) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "%s_forward_cached: new_len must be positive", m->name);
    if (m->cache_len + new_len > m->P)
        return agpu_fail(ctx, AGPU_ERR_DIM_OUT_OF_RANGE, "%s_forward_cached: %d cached + %d new positions exceed n_positions %d", m->name,
                         m->cache_len, new_len, m->P);
    int32_t rc = m->check_ready();
    if (rc != AGPU_OK) return rc;
    if ((rc = m->ensure_buffers(batch, new_len, all_rows != 0)) != AGPU_OK) return rc;
    if ((rc = ensure_out_tokens(m, m->P)) != AGPU_OK) return rc;
    if ((rc = set_counters(m, m->cache_len, -1)) != AGPU_OK) return rc;
    if ((rc = m->launch_forward(tokens, batch, new_len, m->cache_len + new_len, all_rows != 0, nullptr, nullptr)) != AGPU_OK) return rc;
    // keep the device-side generation state usable: next token = arg-max of the last rows
    if (!all_rows) {
        if ((rc = launch_argmax_advance(m, batch, new_len)) != AGPU_OK) return rc;
    } else {
        if ((rc = set_counters(m, m->cache_len + new_len, -1)) != AGPU_OK) return rc;
    }
    m->cache_len += new_len;
    if (logits) {
        const size_t rows = all_rows ? (size_t)batch * new_len : (size_t)batch;
        hipError_t e = hipMemcpy2DAsync(logits, (size_t)m->V * 4, m->logits.p, (size_t)m->logits_stride() * 4, (size_t)m->V * 4,
                                        rows, hipMemcpyDeviceToDevice, ctx->stream);
        if (e != hipSuccess) return agpu_hip(ctx, e, "hipMemcpy2DAsync(logits)");
    }
    return AGPU_OK;
}

int32_t lm_decode_steps(LmRuntime *m, int32_t batch, int32_t steps, float *ms_total_out_host) {
    agpu_ctx *ctx = m->ctx;
    AGPU_REQUIRE_CTX(ctx);
    if (batch <= 0 || batch > m->max_batch || steps < 0)
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "%s_decode_steps: bad batch/steps", m->name);
    if (m->cache_len == 0) return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "%s_decode_steps: run a prefill first", m->name);
    if (m->cache_len + steps > m->P)
        return agpu_fail(ctx, AGPU_ERR_DIM_OUT_OF_RANGE, "%s_decode_steps: %d cached + %d steps exceed n_positions %d", m->name,
                         m->cache_len, steps, m->P);
    int32_t rc = m->ensure_buffers(batch, 1, false);
    if (rc != AGPU_OK) return rc;
    // capture outside the timed region
    hipGraphExec_t exec;
    if (batch == 1 && steps >= 2 && m->one_launch_ready()) {
        if (steps >= 16 && (rc = decode_graph(m, 1, 0, &exec, 16)) != AGPU_OK) return rc;
        if (steps % 16 >= 2 && (rc = decode_graph(m, 1, 0, &exec, steps % 16)) != AGPU_OK) return rc;
    }
    for (int s = 0; s < steps && m->decode_mode != AGPU_DECODE_EAGER; ++s)
        if ((rc = decode_graph(m, batch, kv_bucket(m, m->cache_len + 1 + s), &exec)) != AGPU_OK) return rc;
    if ((rc = agpu_hip(ctx, hipEventRecord(m->ev0, ctx->stream), "hipEventRecord")) != AGPU_OK) return rc;
    if ((rc = run_decode_steps(m, batch, steps)) != AGPU_OK) return rc;
    if ((rc = agpu_hip(ctx, hipEventRecord(m->ev1, ctx->stream), "hipEventRecord")) != AGPU_OK) return rc;
    if ((rc = agpu_hip(ctx, hipEventSynchronize(m->ev1), "hipEventSynchronize")) != AGPU_OK) return rc;
    if (ms_total_out_host) (void)hipEventElapsedTime(ms_total_out_host, m->ev0, m->ev1);
    return m->check_waits();
}

int32_t lm_last_logits(LmRuntime *m, int32_t batch, float *logits_out_host) {
    agpu_ctx *ctx = m->ctx;
    if (!logits_out_host) return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "%s_last_logits: null pointer", m->name);
    if (batch <= 0 || batch > m->max_batch) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "%s_last_logits: bad batch", m->name);
    const size_t stride = m->logits_stride();
    if (!m->logits.p || m->logits.bytes < (size_t)batch * stride * 4)
        return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "%s_last_logits: no forward has run for this batch", m->name);
    hipError_t e = hipMemcpy2DAsync(logits_out_host, (size_t)m->V * 4, m->logits.p, stride * 4, (size_t)m->V * 4, (size_t)batch,
                                    hipMemcpyDeviceToHost, ctx->stream);
    if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
    return agpu_hip(ctx, e, "last_logits");
}

int32_t lm_generate_cached(LmRuntime *m, const uint32_t *prompt_host, int32_t batch, int32_t prompt_len,
                                              int32_t max_new_tokens, int32_t eos, uint32_t *tokens_out_host,
                                              int32_t *lengths_out_host, float *timing_ms_out_host) {
    agpu_ctx *ctx = m->ctx;
    AGPU_REQUIRE_CTX(ctx);
    if (!prompt_host || !tokens_out_host || !lengths_out_host)
        return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "%s_generate_cached: null pointer", m->name);
    if (batch <= 0 || batch > m->max_batch || prompt_len <= 0 || max_new_tokens < 0)
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "%s_generate_cached: bad batch/prompt_len/max_new_tokens", m->name);
    // the last generated token is never fed back, so prompt_len + max_new_tokens - 1 positions are cached
    if (prompt_len + (max_new_tokens > 0 ? max_new_tokens - 1 : 0) > m->P)
        return agpu_fail(ctx, AGPU_ERR_DIM_OUT_OF_RANGE, "%s_generate_cached: prompt %d + %d new tokens exceed n_positions %d", m->name,
                         prompt_len, max_new_tokens, m->P);
    int32_t rc = check_token_ids(m, prompt_host, (size_t)batch * prompt_len, "generate_cached");
    if (rc != AGPU_OK) return rc;
    const int total = prompt_len + max_new_tokens;
    for (int b = 0; b < batch; ++b) {
        std::memcpy(tokens_out_host + (size_t)b * total, prompt_host + (size_t)b * prompt_len, (size_t)prompt_len * 4);
        lengths_out_host[b] = prompt_len;
    }
    if (max_new_tokens == 0) return AGPU_OK;
    if ((rc = m->check_ready()) != AGPU_OK) return rc;
    if ((rc = ensure(m, m->tok_in, (size_t)batch * prompt_len * 4)) != AGPU_OK) return rc;
    if ((rc = m->ensure_buffers(batch, prompt_len, false)) != AGPU_OK) return rc;
    if ((rc = ensure_out_tokens(m, max_new_tokens)) != AGPU_OK) return rc;
    if ((rc = upload(ctx, m->tok_in.p, prompt_host, (size_t)batch * prompt_len * 4, 0)) != AGPU_OK) return rc;
    if ((rc = lm_reset_cache(m)) != AGPU_OK) return rc;

    (void)hipEventRecord(m->ev0, ctx->stream);
    if ((rc = lm_forward_cached(m, (const uint32_t *)m->tok_in.p, batch, prompt_len, nullptr, 0)) != AGPU_OK) return rc;
    (void)hipEventRecord(m->ev1, ctx->stream);
    if ((rc = run_decode_steps(m, batch, max_new_tokens - 1)) != AGPU_OK) return rc;
    (void)hipEventRecord(m->ev2, ctx->stream);

    std::vector<uint32_t> gen((size_t)max_new_tokens * batch);
    rc = agpu_memcpy_d2h(ctx, gen.data(), m->out_tok, gen.size() * 4);
    if (rc != AGPU_OK) return rc;
    if ((rc = m->check_waits()) != AGPU_OK) return rc;
    if (timing_ms_out_host) {
        (void)hipEventElapsedTime(&timing_ms_out_host[0], m->ev0, m->ev1);
        (void)hipEventElapsedTime(&timing_ms_out_host[1], m->ev1, m->ev2);
    }
    for (int b = 0; b < batch; ++b) {
        int len = prompt_len;
        for (int s = 0; s < max_new_tokens; ++s) {
            const uint32_t t = gen[(size_t)s * batch + b];
            if (eos >= 0 && t == (uint32_t)eos) break;  // stop before appending (gpt2.rs:762,776)
            tokens_out_host[(size_t)b * total + len++] = t;
        }
        lengths_out_host[b] = len;
    }
    return AGPU_OK;
}

// sampling.hip
int32_t agpu_top_k_launch(agpu_ctx *ctx, const float *logits, int rows, int n, int stride, int k, float temperature,
                          uint32_t *idx_out, float *val_out);
extern "C" uint32_t agpu_top_k_draw_host(const float *ranked_vals, const uint32_t *ranked_idx, int32_t k, float r);
extern "C" float agpu_simple_rng_next_f32(uint64_t *state);

int32_t lm_generate_cached_sampling(LmRuntime *m, const uint32_t *prompt_host, int32_t prompt_len,
                                                       int32_t max_new_tokens, int32_t top_k, float temperature,
                                                       uint64_t *rng_state, int32_t eos, uint32_t *tokens_out_host,
                                                       int32_t *length_out_host) {
    agpu_ctx *ctx = m->ctx;
    AGPU_REQUIRE_CTX(ctx);
    if (!prompt_host || !tokens_out_host || !length_out_host || !rng_state)
        return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "%s_generate_cached_sampling: null pointer", m->name);
    if (prompt_len <= 0 || max_new_tokens < 0 || top_k <= 0)
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "%s_generate_cached_sampling: bad prompt_len/max_new_tokens/top_k", m->name);
    if (prompt_len + (max_new_tokens > 0 ? max_new_tokens - 1 : 0) > m->P)
        return agpu_fail(ctx, AGPU_ERR_DIM_OUT_OF_RANGE,
                         "%s_generate_cached_sampling: prompt %d + %d new tokens exceed n_positions %d", m->name, prompt_len,
                         max_new_tokens, m->P);
    int32_t rc = check_token_ids(m, prompt_host, (size_t)prompt_len, "generate_cached_sampling");
    if (rc != AGPU_OK) return rc;
    std::memcpy(tokens_out_host, prompt_host, (size_t)prompt_len * 4);
    int len = prompt_len;
    *length_out_host = len;
    if (max_new_tokens == 0) return AGPU_OK;
    if ((rc = m->check_ready()) != AGPU_OK) return rc;
    const int k = top_k < m->V ? top_k : m->V;
    if (k > 1024) return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "%s_generate_cached_sampling: top_k = %d exceeds 1024", m->name, top_k);
    uint32_t *idx_dev = nullptr;
    float *val_dev = nullptr;
    if ((rc = dev_alloc(ctx, (void **)&idx_dev, (size_t)k * 4)) != AGPU_OK) return rc;
    if ((rc = dev_alloc(ctx, (void **)&val_dev, (size_t)k * 4)) != AGPU_OK) {
        (void)hipFree(idx_dev);
        return rc;
    }
    std::vector<uint32_t> idx((size_t)k);
    std::vector<float> val((size_t)k);
    if ((rc = ensure(m, m->tok_in, (size_t)prompt_len * 4)) == AGPU_OK) rc = m->ensure_buffers(1, prompt_len, false);
    if (rc == AGPU_OK) rc = ensure_out_tokens(m, max_new_tokens);
    if (rc == AGPU_OK) rc = upload(ctx, m->tok_in.p, prompt_host, (size_t)prompt_len * 4, 0);
    if (rc == AGPU_OK) rc = lm_reset_cache(m);
    for (int step = 0; rc == AGPU_OK && step < max_new_tokens; ++step) {
        // logits of the last position: the prefill first, then one replayed decode step per token.  The
        // replayed graph also runs the arg-max feed; its token is overwritten by the sampled one below.
        if (step == 0) rc = lm_forward_cached(m, (const uint32_t *)m->tok_in.p, 1, prompt_len, nullptr, 0);
        else rc = run_decode_steps(m, 1, 1);
        if (rc != AGPU_OK) break;
        rc = agpu_top_k_launch(ctx, (const float *)m->logits.p, 1, m->V, m->logits_stride(), k, temperature, idx_dev, val_dev);
        if (rc == AGPU_OK) rc = agpu_memcpy_d2h(ctx, idx.data(), idx_dev, (size_t)k * 4);
        if (rc == AGPU_OK) rc = agpu_memcpy_d2h(ctx, val.data(), val_dev, (size_t)k * 4);
        if (rc != AGPU_OK) break;
        const uint32_t next = agpu_top_k_draw_host(val.data(), idx.data(), k, agpu_simple_rng_next_f32(rng_state));
        if (eos >= 0 && next == (uint32_t)eos) break;  // gpt2.rs:956-958, 970-972
        tokens_out_host[len++] = next;
        if (step + 1 < max_new_tokens) rc = upload(ctx, m->cur_tok, &next, 4, 0);
    }
    (void)hipFree(idx_dev);
    (void)hipFree(val_dev);
    *length_out_host = len;
    if (rc == AGPU_OK) rc = m->check_waits();
    return rc;
}

int32_t lm_generate(LmRuntime *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens,
                                       int32_t eos, uint32_t *tokens_out_host, int32_t *length_out_host) {
    agpu_ctx *ctx = m->ctx;
    AGPU_REQUIRE_CTX(ctx);
    if (!prompt_host || !tokens_out_host || !length_out_host)
        return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "%s_generate: null pointer", m->name);
    if (prompt_len <= 0 || max_new_tokens < 0)
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "%s_generate: bad prompt_len/max_new_tokens", m->name);
    int32_t rc = check_token_ids(m, prompt_host, (size_t)prompt_len, "generate");
    if (rc != AGPU_OK) return rc;
    std::memcpy(tokens_out_host, prompt_host, (size_t)prompt_len * 4);
    int len = prompt_len;
    if ((rc = m->check_ready()) != AGPU_OK) return rc;
    for (int step = 0; step < max_new_tokens; ++step) {
        if (len > m->P) {
            rc = agpu_fail(ctx, AGPU_ERR_DIM_OUT_OF_RANGE, "%s_generate: sequence length %d exceeds n_positions %d", m->name, len, m->P);
            break;
        }
        if ((rc = ensure(m, m->tok_in, (size_t)len * 4)) != AGPU_OK) break;
        if ((rc = upload(ctx, m->tok_in.p, tokens_out_host, (size_t)len * 4, 0)) != AGPU_OK) break;
        if ((rc = lm_reset_cache(m)) != AGPU_OK) break;
        if ((rc = lm_forward_cached(m, (const uint32_t *)m->tok_in.p, 1, len, nullptr, 0)) != AGPU_OK) break;
        uint32_t next = 0;
        if ((rc = agpu_memcpy_d2h(ctx, &next, m->next_tok, 4)) != AGPU_OK) break;
        if (eos >= 0 && next == (uint32_t)eos) break;
        tokens_out_host[len++] = next;
    }
    *length_out_host = len;
    return rc;
}

