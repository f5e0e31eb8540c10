// Piralix model driver (include/agpu_piralix.h) on the generation runtime of lm_runtime.h.
//
// Per layer run, x the fp32 residual stream:
//   in    [q | k | v | gate | i, f], [q | k | v | gate] or [y | x] = norm1(x) W + bias   one Linear
//   mixer
//   out   y = W_o (mixer's output)                                                       one Linear
//   up    act(norm2(x) W)                                                                one Linear, the activation in its epilogue
//   down  y = W_down act                                                                 one Linear
// The norm behind a sublayer and its addition are left to whatever reads x next (DenseRows::y), as are the additions in front
// of a loop's pass; the matrix memory's head norm and gate are left to its out Linear (DenseRows::gate).  One or two rows run
// as GEMVs that do all this in their prologue; more rows go through dense_rows_launch and the matrix cores.
//
// Heads and blocks are padded to multiples of 32 columns everywhere (projections, cache, state, mixer output, columns of W_o),
// each on its own; the padding is zero.
#include <algorithm>
#include <new>
#include <string>
#include <vector>

#include "../../include/agpu_piralix.h"
#include "gated_lru.h"
#include "grouped_attention.h"
#include "layered_model.h"
#include "matrix_memory.h"

namespace {

struct Layer {
    agpu_piralix_layer c{};
    GroupedShape gs;
    MemoryShape ms;
    LruShape rs;
    LruWeights rw;
    RopeSpec rope_spec;
    float2 *rope = nullptr;
    Mat in, out, gates, up, down;
    float *norm1 = nullptr, *norm1b = nullptr, *norm2 = nullptr, *norm2b = nullptr, *in_bias = nullptr, *sink = nullptr, *mix_norm = nullptr, *conv = nullptr,
          *conv_bias = nullptr, *gate_bias = nullptr, *lam = nullptr;
    int col[5] = {0, 0, 0, 0, 0};  // q, k, v, gate, i (f behind it); or y, x
    int mix_w = 0, ffp = 0;        // padded widths of the mixer's output and of the feed-forward
};

struct Run {
    int layer = 0;
    int loop_step = -1;            // >= 0: the first layer of that pass
    size_t kcache = 0, vcache = 0; // keys and values of this run, elements
    size_t state = 0, extra = 0;   // recurrent state of this run, normaliser or convolution ring, floats
};

}  // namespace

struct agpu_piralix final : LayeredModel {
    agpu_piralix() : LayeredModel("piralix") {}
    int32_t ensure_buffers(int B, int new_len, bool all_rows_logits) override;
    int layer_runs() const override { return (int)runs.size(); }
    int32_t launch_forward(const uint32_t *tokens, int B, int new_len, int max_kv, bool all_rows_logits, const ArgmaxAdvance *feed,
                           bool *fed) override;
    void mix_addresses(AddrHash &h, bool one_launch) const override;
    int32_t reset_state() override { return fill_u32(ctx, state, 0u, state_floats); }
    int32_t mixer(const Run &r, int B, int new_len, int max_kv, bool out_bf16);

    agpu_piralix_config cfg{};
    std::vector<Layer> layers;
    std::vector<Run> runs;
    Mat embed;  // [padded vocabulary][dp]: table and head
    float *final_norm = nullptr, *loop_step = nullptr;
    char *cache = nullptr;   // keys and values of every run
    float *state = nullptr;  // recurrent states, normalisers and rings of every run
    size_t cache_elems = 0, state_floats = 0;
    int max_in = 0, max_mix = 0, max_ff = 0;
    DevBuf xa, xb, x0, y, h, proj, raw, mix, act, partial, memory, lru_u, lru_gates, lru_carries;

    // more rows than these pay more for a prologue per workgroup than for row launches and the matrix cores
    bool small(int rows) const { return rows <= 2 && dense_gemv_supported(rows, std::max({dp, max_mix, max_ff})); }
};

namespace {

int32_t bad_sizes(agpu_piralix *m, int i) { return agpu_fail(m->ctx, AGPU_ERR_SHAPE_MISMATCH, "piralix: sizes of layer %d not supported", i); }

// A matrix of `heads` heads of `per` rows at columns (rows of `in`) `at` ..
void add_in(agpu_piralix *m, Layer &L, const std::string &name, int at, int heads, int per, int per_p) {
    m->add_head_rows(name, L.in, heads, per, per_p, m->d, at);
}

int32_t build_layer(agpu_piralix *m, int i) {
    Layer &L = m->layers[i];
    const agpu_piralix_layer &c = L.c;
    const std::string p = "l" + std::to_string(i) + ".", q = p + "mix.";
    const int d = m->d, dp = m->dp;
    if (c.ff < 0 || (c.ff > 0 && !(c.ff_limit > 0.0f))) return bad_sizes(m, i);
    AGPU_TRY(m->add_vec(p + "norm1", &L.norm1, 1, d));
    AGPU_TRY(m->add_vec(p + "norm1b", &L.norm1b, 1, d));
    if (c.mixer == AGPU_MIXER_MATRIX_MEMORY) {
        MemoryShape &s = L.ms;
        s.heads = c.heads; s.dim = c.dim; s.vdim = c.vdim; s.cap = c.gate_cap;
        if (!memory_supported(s)) return bad_sizes(m, i);
        const int H = c.heads, nk = H * s.dimp(), nv = H * s.vdimp();
        for (int e = 0, at[5] = {0, nk, 2 * nk, 2 * nk + nv, 2 * nk + 2 * nv}; e < 5; ++e) L.col[e] = at[e];
        L.mix_w = nv;
        AGPU_TRY(m->new_mat(L.in, L.col[4] + pad32(2 * H), dp));
        add_in(m, L, q + "q", L.col[0], H, c.dim, s.dimp());
        add_in(m, L, q + "k", L.col[1], H, c.dim, s.dimp());
        add_in(m, L, q + "v", L.col[2], H, c.vdim, s.vdimp());
        add_in(m, L, q + "g", L.col[3], H, c.vdim, s.vdimp());
        AGPU_TRY(m->new_mat(L.out, dp, nv));
        m->add_head_cols(q + "o", L.out, H, c.vdim, s.vdimp(), d);
        AGPU_TRY(m->add_vec(q + "norm", &L.mix_norm, 1, (int64_t)H * c.vdim, (size_t)nv, 0, c.vdim, s.vdimp()));
        add_in(m, L, q + "i", L.col[4], H, 1, 1);
        AGPU_TRY(m->add_vec(q + "i.b", &L.in_bias, 1, H, L.in.N, L.col[4]));
        add_in(m, L, q + "f", L.col[4] + H, H, 1, 1);
        AGPU_TRY(m->add_vec(q + "f.b", &L.in_bias, 1, H, 0, L.col[4] + H));
    } else if (c.mixer == AGPU_MIXER_GROUPED_ATTENTION) {
        GroupedShape &s = L.gs;
        s.heads = c.heads; s.kv_heads = c.kv_heads; s.dim = c.dim; s.vdim = c.vdim; s.rot_dims = c.rot_dims; s.scale = c.scale; s.softcap = c.softcap;
        if (!grouped_supported(s)) return bad_sizes(m, i);
        const int H = c.heads, G = c.kv_heads, nq = H * s.dimp(), nk = G * s.dimp(), nkv = G * s.vdimp(), nv = H * s.vdimp();
        for (int e = 0, at[4] = {0, nq, nq + nk, nq + nk + nkv}; e < 4; ++e) L.col[e] = at[e];
        L.mix_w = nv;
        AGPU_TRY(m->new_mat(L.in, L.col[3] + nv, dp));
        add_in(m, L, q + "q", L.col[0], H, c.dim, s.dimp());
        add_in(m, L, q + "k", L.col[1], G, c.dim, s.dimp());
        add_in(m, L, q + "v", L.col[2], G, c.vdim, s.vdimp());
        add_in(m, L, q + "g", L.col[3], H, c.vdim, s.vdimp());
        AGPU_TRY(m->add_vec(q + "sink", &L.sink, 1, H));
        AGPU_TRY(m->new_mat(L.out, dp, nv));
        m->add_head_cols(q + "o", L.out, H, c.vdim, s.vdimp(), d);
        RopeSpec &rs = L.rope_spec;
        rs.dims = c.rot_dims; rs.base = c.rot_base; rs.factor = c.rot_factor; rs.original = c.rot_original; rs.fast = c.rot_fast; rs.slow = c.rot_slow;
        for (int j = 0; j < i; ++j)  // layers that turn alike share a table
            if (m->layers[j].rope && m->layers[j].rope_spec == rs) L.rope = m->layers[j].rope;
        if (!L.rope) {
            AGPU_TRY(m->own((void **)&L.rope, (size_t)m->P * std::max(c.rot_dims / 2, 1) * sizeof(float2), nullptr));
            AGPU_TRY(rope_table_launch(m->ctx, L.rope, m->P, rs));
        }
    } else if (c.mixer == AGPU_MIXER_GATED_LRU) {
        LruShape &s = L.rs;
        s.width = c.lru_width; s.blocks = c.blocks; s.taps = c.conv;
        if (!lru_supported(s)) return bad_sizes(m, i);
        const int B = s.blocks, bs = s.block(), bp = s.blockp(), wp = s.widthp();
        L.col[1] = wp;
        L.mix_w = wp;
        AGPU_TRY(m->new_mat(L.in, 2 * wp, dp));
        add_in(m, L, q + "y", 0, B, bs, bp);
        AGPU_TRY(m->add_vec(q + "y.b", &L.in_bias, 1, s.width, L.in.N, 0, bs, bp));
        add_in(m, L, q + "x", wp, B, bs, bp);
        AGPU_TRY(m->add_vec(q + "x.b", &L.in_bias, 1, s.width, 0, wp, bs, bp));
        AGPU_TRY(m->add_vec(q + "conv", &L.conv, s.width, s.taps, (size_t)wp * s.taps, 0, (size_t)bs * s.taps, (size_t)bp * s.taps));
        AGPU_TRY(m->add_vec(q + "conv.b", &L.conv_bias, 1, s.width, wp, 0, bs, bp));
        AGPU_TRY(m->new_mat(L.gates, B * 2 * bp, bp));
        m->add_head_rows(q + "ra", L.gates, B, bs, 2 * bp, bs, 0);
        AGPU_TRY(m->add_vec(q + "ra.b", &L.gate_bias, B, bs, (size_t)2 * wp, 0, bs, (size_t)2 * bp));
        m->add_head_rows(q + "ri", L.gates, B, bs, 2 * bp, bs, bp);
        AGPU_TRY(m->add_vec(q + "ri.b", &L.gate_bias, B, bs, 0, bp, bs, (size_t)2 * bp));
        AGPU_TRY(m->add_vec(q + "lam", &L.lam, 1, s.width, wp, 0, bs, bp));
        AGPU_TRY(m->new_mat(L.out, dp, wp));
        m->add_head_cols(q + "o", L.out, B, bs, bp, d);
        L.rw.conv = L.conv; L.rw.conv_bias = L.conv_bias; L.rw.gates = L.gates.w; L.rw.gate_bias = L.gate_bias; L.rw.lam = L.lam;
    } else {
        return agpu_fail(m->ctx, AGPU_ERR_UNSUPPORTED, "piralix: unknown mixer %d of layer %d", c.mixer, i);
    }
    if (c.ff > 0) {
        L.ffp = pad32(c.ff);
        AGPU_TRY(m->add_vec(p + "norm2", &L.norm2, 1, d));
        AGPU_TRY(m->add_vec(p + "norm2b", &L.norm2b, 1, d));
        AGPU_TRY(m->new_mat(L.up, 2 * L.ffp, dp));
        m->add_rows(p + "mlp.gate", L.up, 0, 0, c.ff, d, 2);
        m->add_rows(p + "mlp.up", L.up, 1, 0, c.ff, d, 2);
        AGPU_TRY(m->new_mat(L.down, dp, L.ffp));
        m->add_rows(p + "mlp.down", L.down, 0, 0, d, c.ff);
    }
    m->max_in = std::max(m->max_in, L.in.N);
    m->max_mix = std::max(m->max_mix, L.mix_w);
    m->max_ff = std::max(m->max_ff, L.ffp);
    return AGPU_OK;
}

int32_t build(agpu_piralix *m) {
    const agpu_piralix_config &c = m->cfg;
    AGPU_TRY(m->new_mat(m->embed, pad32(m->V), m->dp));
    m->add_rows("embed", m->embed, 0, 0, m->V, m->d);
    if (c.loop_times > 0) AGPU_TRY(m->add_vec("loop.step", &m->loop_step, c.loop_times, m->d, (size_t)c.loop_times * m->dp, 0, m->d, m->dp));
    for (int i = 0; i < c.n_layer; ++i) AGPU_TRY(build_layer(m, i));
    AGPU_TRY(m->add_vec("final.norm", &m->final_norm, 1, m->d));

    // the layer runs in order, each with a cache or state of its own
    auto push = [&](int layer, int step) {
        Run r;
        r.layer = layer;
        r.loop_step = step;
        const Layer &L = m->layers[layer];
        const size_t B = (size_t)m->max_batch;
        if (L.c.mixer == AGPU_MIXER_GROUPED_ATTENTION) {
            r.kcache = m->cache_elems;
            r.vcache = r.kcache + B * L.gs.kv_heads * m->P * L.gs.dimp();
            m->cache_elems = r.vcache + B * L.gs.kv_heads * L.gs.vdimp() * grouped_kv_stride(m->P);
        } else {
            r.state = m->state_floats;
            r.extra = r.state + B * (L.c.mixer == AGPU_MIXER_MATRIX_MEMORY ? L.ms.state_floats() : (size_t)L.rs.widthp());
            m->state_floats = r.extra + B * (L.c.mixer == AGPU_MIXER_MATRIX_MEMORY ? L.ms.norm_floats() : (size_t)L.rs.taps * L.rs.widthp());
        }
        m->runs.push_back(r);
    };
    const int lo = c.loop_times > 0 ? c.loop_start : c.n_layer, hi = c.loop_times > 0 ? c.loop_stop : c.n_layer;
    for (int i = 0; i < lo; ++i) push(i, -1);
    for (int t = 0; t < c.loop_times; ++t)
        for (int i = lo; i < hi; ++i) push(i, i == lo ? t : -1);
    for (int i = hi; i < c.n_layer; ++i) push(i, -1);
    if (m->cache_elems) AGPU_TRY(m->own((void **)&m->cache, m->cache_elems * (m->f32 ? 4 : 2), &m->cache_bytes));
    if (m->state_floats) AGPU_TRY(m->own((void **)&m->state, m->state_floats * sizeof(float), &m->cache_bytes));
    return AGPU_OK;
}

}  // namespace

// The mixer's output goes to `mix`, of a matrix memory (before head norm and gate) to `raw`.
int32_t agpu_piralix::mixer(const Run &r, int B, int new_len, int max_kv, bool out_bf16) {
    Layer &L = layers[r.layer];
    const float *in = (const float *)proj.p;
    if (L.c.mixer == AGPU_MIXER_GROUPED_ATTENTION) {
        const size_t elem = f32 ? 4 : 2;
        GroupedArgs a;
        a.s = L.gs;
        a.rope = L.rope;
        a.sink = L.sink;
        a.q = in + L.col[0]; a.k = in + L.col[1]; a.v = in + L.col[2]; a.gate = in + L.col[3];
        a.ld = L.in.N;
        a.kcache = cache + r.kcache * elem;
        a.vcache = cache + r.vcache * elem;
        a.cache_bf16 = !f32;
        a.positions = P;
        a.batch = B; a.new_len = new_len; a.pos_dev = pos_dev; a.kv_max = max_kv;
        a.out = mix.p; a.ldo = L.mix_w; a.out_bf16 = out_bf16;
        a.partial = (float *)partial.p;
        return grouped_attention_launch(ctx, a);
    }
    if (L.c.mixer == AGPU_MIXER_MATRIX_MEMORY) {
        MemoryArgs a;
        a.s = L.ms;
        a.q = in + L.col[0]; a.k = in + L.col[1]; a.v = in + L.col[2]; a.i = in + L.col[4]; a.f = in + L.col[4] + L.c.heads;
        a.ld = L.in.N;
        a.state = state + r.state; a.norm = state + r.extra;
        a.batch = B; a.new_len = new_len; a.pos_dev = pos_dev;
        a.out = (float *)raw.p; a.ldo = L.mix_w;
        a.scratch = memory.p;
        return memory_launch(ctx, a);
    }
    LruArgs a;
    a.s = L.rs;
    a.w = L.rw;
    a.proj = in;
    a.ld = L.in.N;
    a.col_y = L.col[0]; a.col_x = L.col[1];
    a.state = state + r.state; a.ring = state + r.extra;
    a.batch = B; a.new_len = new_len; a.pos_dev = pos_dev;
    a.out = mix.p; a.ldo = L.mix_w; a.out_bf16 = out_bf16;
    a.u = (float *)lru_u.p; a.gates = (float *)lru_gates.p; a.carries = (float *)lru_carries.p;
    return lru_launch(ctx, a);
}

int32_t agpu_piralix::launch_forward(const uint32_t *tokens, int B, int new_len, int max_kv, bool all_rows_logits, const ArgmaxAdvance *feed,
                                     bool *fed) {
    (void)feed;
    if (fed) *fed = false;
    const int R = B * new_len;
    const bool gemv = small(R), a16 = !f32 && !gemv;
    float *x = (float *)xa.p, *spare = (float *)xb.p;
    AGPU_TRY(embed_rows_launch(ctx, tokens, embed.w, dp, nullptr, x, cfg.loop_times > 0 ? (float *)x0.p : nullptr, R, V, d, dp, cfg.norm_eps));
    const float *pending = nullptr;  // the norm of a sublayer whose output still waits in `y`
    auto rows_of = [&](const float *norm_w) {
        DenseRows in;
        in.x = x;
        in.ldx = in.dp = dp;
        in.d = d;
        in.eps = cfg.norm_eps;
        in.norm_w = norm_w;
        if (pending) {
            in.y = (const float *)y.p;
            in.y_w = pending;
        }
        return in;
    };
    // a Linear on the residual stream, which takes up what waits for it
    auto linear_of_x = [&](DenseRows in, const Mat &w, const DenseOut &o) -> int32_t {
        const bool changed = in.y || in.add || in.add_vec;
        if (gemv) {
            if (changed) in.x_out = spare;
            AGPU_TRY(dense_gemv_launch(ctx, in, w.w, R, w.N, w.K, o));
            if (changed) std::swap(x, spare);
        } else {
            if (changed) in.x_out = x;
            AGPU_TRY(dense_rows_launch(ctx, in, R, h.p, dp, a16));
            AGPU_TRY(gemm(h.p, dp, w, R, o));
        }
        pending = nullptr;
        return AGPU_OK;
    };
    // a Linear on finished rows of w.K columns
    auto linear_of_rows = [&](const void *rows, const Mat &w, const DenseOut &o) -> int32_t {
        if (!gemv) return gemm(rows, w.K, w, R, o);
        DenseRows in;
        in.x = (const float *)rows;
        in.ldx = in.d = in.dp = w.K;
        return dense_gemv_launch(ctx, in, w.w, R, w.N, w.K, o);
    };
    DenseOut to_y;
    to_y.n_plain = to_y.ldo = dp;
    to_y.out = (float *)y.p;
    for (size_t i = 0; i < runs.size(); ++i) {
        const Run &r = runs[i];
        Layer &L = layers[r.layer];
        DenseRows in = rows_of(L.norm1);
        if (r.loop_step >= 0) {
            if (r.loop_step > 0) in.add = (const float *)x0.p;
            in.add_vec = loop_step + (size_t)r.loop_step * dp;
        }
        DenseOut o;
        o.n_plain = o.ldo = L.in.N;
        o.out = (float *)proj.p;
        o.bias = L.in_bias;
        AGPU_TRY(linear_of_x(in, L.in, o));
        AGPU_TRY(mixer(r, B, new_len, max_kv, a16));
        if (L.c.mixer == AGPU_MIXER_MATRIX_MEMORY) {
            DenseRows g;
            g.x = (const float *)raw.p;
            g.ldx = g.d = g.dp = L.mix_w;
            g.norm_w = L.mix_norm;
            g.eps = cfg.norm_eps;
            g.gate = (const float *)proj.p + L.col[3];
            g.ld_gate = L.in.N;
            g.groups = L.c.heads; g.group_d = L.c.vdim; g.group_p = L.ms.vdimp();
            if (gemv) {
                AGPU_TRY(dense_gemv_launch(ctx, g, L.out.w, R, L.out.N, L.out.K, to_y));
            } else {
                AGPU_TRY(dense_rows_launch(ctx, g, R, mix.p, L.mix_w, a16));
                AGPU_TRY(gemm(mix.p, L.mix_w, L.out, R, to_y));
            }
        } else {
            AGPU_TRY(linear_of_rows(mix.p, L.out, to_y));
        }
        pending = L.norm1b;
        if (L.ffp > 0) {
            DenseOut u;
            u.act = act.p;
            u.ld_act = L.ffp;
            u.act_bf16 = a16;
            u.act_limit = L.c.ff_limit;
            AGPU_TRY(linear_of_x(rows_of(L.norm2), L.up, u));
            AGPU_TRY(linear_of_rows(act.p, L.down, to_y));
            pending = L.norm2b;
        }
        if (tap) {
            DenseRows fi = rows_of(nullptr);
            fi.x_out = x;
            AGPU_TRY(dense_rows_launch(ctx, fi, R, nullptr, 0, 0));
            pending = nullptr;
            AGPU_TRY(save_tap(i, x, R));
        }
    }
    const int rows = all_rows_logits ? R : B;
    DenseRows in = rows_of(final_norm);
    in.map_stride = all_rows_logits ? 0 : new_len;
    DenseOut o;
    o.n_plain = o.ldo = logits_stride();
    o.out = (float *)logits.p;
    if (dense_gemv_supported(rows, dp)) return dense_gemv_launch(ctx, in, embed.w, rows, embed.N, embed.K, o);
    AGPU_TRY(dense_rows_launch(ctx, in, rows, h.p, dp, !f32));
    return gemm(h.p, dp, embed, rows, o);
}

int32_t agpu_piralix::ensure_buffers(int B, int new_len, bool all_rows_logits) {
    const size_t R = (size_t)B * new_len, f = sizeof(float);
    if (R > 65535) return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "piralix: %zu rows in one forward exceed 65535; feed the prompt in portions", R);
    for (DevBuf *b : {&xa, &xb, &y, &h}) AGPU_TRY(ensure(this, *b, R * dp * f));
    if (cfg.loop_times > 0) AGPU_TRY(ensure(this, x0, R * dp * f));
    AGPU_TRY(ensure(this, proj, R * max_in * f));
    AGPU_TRY(ensure(this, mix, R * max_mix * f));
    if (max_ff > 0) AGPU_TRY(ensure(this, act, R * max_ff * f));
    AGPU_TRY(ensure(this, logits, (all_rows_logits ? R : (size_t)B) * logits_stride() * f));
    for (const Layer &L : layers) {
        if (L.c.mixer == AGPU_MIXER_GROUPED_ATTENTION) {
            AGPU_TRY(ensure(this, partial, grouped_partial_floats(ctx, L.gs, B, new_len, P) * f));
        } else if (L.c.mixer == AGPU_MIXER_MATRIX_MEMORY) {
            AGPU_TRY(ensure(this, raw, R * max_mix * f));
            if (new_len > 1) AGPU_TRY(ensure(this, memory, memory_scratch_bytes(L.ms, B, new_len)));
        } else if (new_len > 1) {
            AGPU_TRY(ensure(this, lru_u, R * L.rs.widthp() * f));
            AGPU_TRY(ensure(this, lru_gates, R * 2 * L.rs.widthp() * f));
            AGPU_TRY(ensure(this, lru_carries, lru_carry_floats(L.rs, B, new_len) * f));
        }
    }
    return AGPU_OK;
}

void agpu_piralix::mix_addresses(AddrHash &hash, bool) const {
    for (void *p : owned) hash.mix(p);
    for (const DevBuf *b : {&xa, &xb, &x0, &y, &h, &proj, &raw, &mix, &act, &partial}) hash.mix(b->p);
}

AGPU_EXPORT int32_t agpu_piralix_create(agpu_ctx *ctx, const agpu_piralix_config *cfg, const agpu_piralix_layer *layers, agpu_piralix **out) {
    AGPU_REQUIRE_CTX(ctx);
    if (!cfg || !layers || !out) return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "piralix_create: null pointer");
    *out = nullptr;
    if (cfg->n_layer <= 0 || cfg->width <= 0 || cfg->vocab_size <= 0 || cfg->n_positions <= 0 || cfg->max_batch <= 0 || cfg->max_batch > 1024 ||
        cfg->loop_times < 0 || (cfg->dtype != AGPU_DTYPE_BF16 && cfg->dtype != AGPU_DTYPE_F32))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "piralix_create: bad configuration");
    if (cfg->loop_times > 0 && (cfg->loop_start < 0 || cfg->loop_stop <= cfg->loop_start || cfg->loop_stop > cfg->n_layer))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "piralix_create: loop over layers %d .. %d of %d", cfg->loop_start, cfg->loop_stop, cfg->n_layer);
    agpu_piralix *m = new (std::nothrow) agpu_piralix();
    if (!m) return AGPU_ERR_NULL_POINTER;
    m->cfg = *cfg;
    m->d = cfg->width;
    m->dp = pad32(m->d);
    m->f32 = cfg->dtype == AGPU_DTYPE_F32;
    m->layers.resize((size_t)cfg->n_layer);
    for (int i = 0; i < cfg->n_layer; ++i) m->layers[(size_t)i].c = layers[i];
    int32_t rc = lm_init(m, ctx, cfg->vocab_size, cfg->n_positions, cfg->max_batch, cfg->argmax_last);
    if (rc == AGPU_OK) rc = build(m);
    if (rc == AGPU_OK) rc = agpu_hip(ctx, hipStreamSynchronize(ctx->stream), "hipStreamSynchronize");
    if (rc != AGPU_OK) {
        agpu_piralix_destroy(m);
        return rc;
    }
    *out = m;
    return AGPU_OK;
}

AGPU_EXPORT int32_t agpu_piralix_destroy(agpu_piralix *m) {
    if (!m) return AGPU_OK;
    layered_release(m, {&m->xa, &m->xb, &m->x0, &m->y, &m->h, &m->proj, &m->raw, &m->mix, &m->act, &m->partial, &m->memory, &m->lru_u, &m->lru_gates,
                        &m->lru_carries});
    delete m;
    return AGPU_OK;
}

AGPU_EXPORT int32_t agpu_piralix_set_tensor(agpu_piralix *m, const char *name, const void *data_host, int32_t dtype, int64_t rows, int64_t cols) {
    return m ? lm_set_tensor(m, name, data_host, dtype, rows, cols) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_piralix_tensor_info(const agpu_piralix *m, int32_t i, const char **name_out, int64_t *rows_out, int64_t *cols_out,
                                             int32_t *is_set_out) {
    return m ? lm_tensor_info(m, i, name_out, rows_out, cols_out, is_set_out) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int64_t agpu_piralix_weight_bytes(const agpu_piralix *m) { return m ? m->weight_bytes : 0; }
AGPU_EXPORT int64_t agpu_piralix_cache_bytes(const agpu_piralix *m) { return m ? m->cache_bytes : 0; }
AGPU_EXPORT int32_t agpu_piralix_layer_runs(const agpu_piralix *m) { return m ? (int32_t)m->runs.size() : 0; }

AGPU_EXPORT int32_t agpu_piralix_reset_cache(agpu_piralix *m) { return m ? lm_reset_cache(m) : AGPU_ERR_NULL_POINTER; }
AGPU_EXPORT int32_t agpu_piralix_cache_len(const agpu_piralix *m) { return m ? m->cache_len : 0; }

AGPU_EXPORT int32_t agpu_piralix_forward_cached(agpu_piralix *m, const uint32_t *tokens, int32_t batch, int32_t new_len, float *logits,
                                                int32_t all_rows) {
    return m ? lm_forward_cached(m, tokens, batch, new_len, logits, all_rows) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_piralix_generate_cached(agpu_piralix *m, const uint32_t *prompt_host, int32_t batch, int32_t prompt_len,
                                                 int32_t max_new_tokens, int32_t eos, uint32_t *tokens_out_host, int32_t *lengths_out_host,
                                                 float *timing_ms_out_host) {
    if (!m) return AGPU_ERR_NULL_POINTER;
    return lm_generate_cached(m, prompt_host, batch, prompt_len, max_new_tokens, eos, tokens_out_host, lengths_out_host, timing_ms_out_host);
}

AGPU_EXPORT int32_t agpu_piralix_generate(agpu_piralix *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens, int32_t eos,
                                          uint32_t *tokens_out_host, int32_t *length_out_host) {
    return m ? lm_generate(m, prompt_host, prompt_len, max_new_tokens, eos, tokens_out_host, length_out_host) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_piralix_generate_cached_sampling(agpu_piralix *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens,
                                                          int32_t top_k, float temperature, uint64_t *rng_state, int32_t eos,
                                                          uint32_t *tokens_out_host, int32_t *length_out_host) {
    if (!m) return AGPU_ERR_NULL_POINTER;
    return lm_generate_cached_sampling(m, prompt_host, prompt_len, max_new_tokens, top_k, temperature, rng_state, eos, tokens_out_host, length_out_host);
}

AGPU_EXPORT int32_t agpu_piralix_set_decode_mode(agpu_piralix *m, int32_t mode) { return m ? lm_set_decode_mode(m, mode) : AGPU_ERR_NULL_POINTER; }

AGPU_EXPORT int32_t agpu_piralix_decode_steps(agpu_piralix *m, int32_t batch, int32_t steps, float *ms_total_out_host) {
    return m ? lm_decode_steps(m, batch, steps, ms_total_out_host) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_piralix_last_logits(agpu_piralix *m, int32_t batch, float *logits_out_host) {
    return m ? lm_last_logits(m, batch, logits_out_host) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_piralix_layer_streams(agpu_piralix *m, const uint32_t *tokens, int32_t new_len, float *streams_out_host) {
    return m ? lm_layer_streams(m, tokens, new_len, streams_out_host) : AGPU_ERR_NULL_POINTER;
}
