// Ritevik model driver (include/agpu_ritevik.h) on the generation runtime of lm_runtime.h.
//
// Per layer run, x the fp32 residual stream:
//   in     [q | down | gate, up] or [q | k | v | b | a1 | g1 | gate, up] = norm1(x) W   one Linear, silu(gate) up in its epilogue
//   mixer  -> the front of `cat`, the activation behind it
//   out    x += [W_o | W_down] cat                                                      one Linear
//   side   s = gelu(W_gate x) * table[token], y = W_proj s                              two Linears
// The side input's own norm and addition are left to whatever reads x next (DenseRows::y): the next layer's norm, the
// loop's input or the head.  Up to four rows run as GEMVs that do this in their prologue; more rows go through
// dense_rows_launch and the matrix cores.
#include <algorithm>
#include <new>
#include <string>
#include <vector>

#include "../../include/agpu_ritevik.h"
#include "dense_linear.h"
#include "gated_delta.h"
#include "latent_attention.h"
#include "layered_model.h"

namespace {

constexpr int kTiledFrom = 16;  // new tokens per sequence from which latent attention takes the tiled form

struct Layer {
    agpu_ritevik_layer c{};
    LatentShape ls;
    LatentWeights lw;
    DeltaShape ds;
    DeltaWeights dw;
    Mat in, out, uk, uv, a2, g2, side_gate, side_proj;
    float *norm1 = nullptr, *dkv_norm = nullptr, *sink = nullptr, *conv = nullptr, *a_log = nullptr, *dt_bias = nullptr, *mix_norm = nullptr,
          *side_norm = nullptr;
    int n_plain = 0;                                                  // columns of `in` in front of the gate/up pairs
    int col_q = 0, col_k = 0, col_v = 0, col_b = 0, col_a1 = 0, col_g1 = 0;  // col_k: the latent part of an attention layer
    int mix_w = 0, mix_wp = 0, ffp = 0;                               // mixer output width, padded; feed-forward width, padded
    int cat_k() const { return mix_wp + ffp; }
};

struct Run {
    int layer = 0;
    int loop_step = -1;      // >= 0: the first layer of that pass
    size_t cache = 0;        // latent cache of this run, elements
    size_t state = 0, ring = 0;  // delta state of this run, floats
};

// Columns [lo, hi) of rows [0, rows) to zero.
template <typename T>
__global__ __launch_bounds__(256) void zero_columns_kernel(T *p, int ld, int lo, int hi, int rows) {
    const int n = hi - lo, i = blockIdx.x * 256 + threadIdx.x;
    if (i < n * rows) p[(size_t)(i / n) * ld + lo + i % n] = (T)0;
}

}  // namespace

struct agpu_ritevik final : LayeredModel {
    agpu_ritevik() : LayeredModel("ritevik") {}
    int32_t ensure_buffers(int B, int new_len, bool all_rows_logits) override;
    int layer_runs() const override { return (int)runs.size(); }
    int32_t launch_forward(const uint32_t *tokens, int B, int new_len, int max_kv, bool all_rows_logits, const ArgmaxAdvance *feed,
                           bool *fed) override;
    void mix_addresses(AddrHash &h, bool one_launch) const override;
    int32_t reset_state() override;

    agpu_ritevik_config cfg{};
    int side_p = 0;
    std::vector<Layer> layers;
    std::vector<Run> runs;
    uint16_t *embed = nullptr, *side_embed = nullptr;
    float *embed_norm = nullptr, *final_norm = nullptr, *loop_step = nullptr;
    Mat loop_in, head;
    void *latents = nullptr;
    float *state = nullptr;  // delta states and convolution rings of every run
    size_t latent_elems = 0, state_floats = 0;
    int max_cat = 0, max_in = 0;
    DevBuf xa, xb, x0, y, h, proj, cat, side, qlat, partial, qb, kx, vx, dqkg, dv, dstep, dbkq, dgate, dout;

    bool small(int rows) const { return dense_gemv_supported(rows, std::max(max_cat, loop_in.K)); }
};

namespace {

int32_t build_layer(agpu_ritevik *m, int i) {
    Layer &L = m->layers[i];
    const agpu_ritevik_layer &c = L.c;
    const std::string p = "l" + std::to_string(i) + ".";
    const int d = m->d, dp = m->dp;
    if (c.heads <= 0 || c.dim <= 0 || c.vdim <= 0 || c.ff < 0)
        return agpu_fail(m->ctx, AGPU_ERR_SHAPE_MISMATCH, "ritevik: bad sizes of layer %d", i);
    L.mix_w = c.heads * c.vdim;
    L.mix_wp = pad32(L.mix_w);
    L.ffp = pad32(c.ff);
    AGPU_TRY(m->add_vec(p + "norm1", &L.norm1, 1, d));
    if (c.mixer == AGPU_MIXER_LATENT_ATTENTION) {
        if (c.kv_rank <= 0 || c.rot_dim < 0 || c.rot_dims < 0 || c.rot_dims > c.rot_dim || c.rot_dims % 2 != 0 || c.kv_rank > 1024 || c.dim > 1024)
            return agpu_fail(m->ctx, AGPU_ERR_SHAPE_MISMATCH, "ritevik: bad latent attention sizes of layer %d", i);
        LatentShape &s = L.ls;
        s.heads = c.heads; s.dim = c.dim; s.rot = c.rot_dim; s.rot_dims = c.rot_dims; s.vdim = c.vdim; s.rank = c.kv_rank;
        s.scale = c.scale; s.eps = m->cfg.norm_eps;
        const int nq = c.heads * (c.dim + c.rot_dim), nd = c.kv_rank + c.rot_dim;
        L.col_q = 0;
        L.col_k = pad32(nq);
        L.n_plain = L.col_k + pad32(nd);
        AGPU_TRY(m->new_mat(L.in, L.n_plain + 2 * L.ffp, dp));
        m->add_rows(p + "mix.q", L.in, L.col_q, 0, nq, d);
        m->add_rows(p + "mix.dkv", L.in, L.col_k, 0, nd, d);
        AGPU_TRY(m->add_vec(p + "mix.dkv.norm", &L.dkv_norm, 1, c.kv_rank));
        AGPU_TRY(m->new_mat(L.uk, c.heads * s.dimp(), s.rankp()));
        m->add_head_rows(p + "mix.uk", L.uk, c.heads, c.dim, s.dimp(), c.kv_rank);
        AGPU_TRY(m->new_mat(L.uv, c.heads * s.vdimp(), s.rankp()));
        m->add_head_rows(p + "mix.uv", L.uv, c.heads, c.vdim, s.vdimp(), c.kv_rank);
        AGPU_TRY(m->add_vec(p + "mix.sink", &L.sink, 1, c.heads));
        float2 *rope = nullptr;
        for (int j = 0; j < i; ++j) {  // layers that turn alike share a table
            const Layer &o = m->layers[j];
            if (o.c.mixer == c.mixer && o.c.rot_dims == c.rot_dims && o.c.rot_base == c.rot_base) rope = const_cast<float2 *>(o.lw.rope);
        }
        if (!rope && c.rot_dims > 0) {
            AGPU_TRY(m->own((void **)&rope, (size_t)m->P * (c.rot_dims / 2) * sizeof(float2), nullptr));
            RopeSpec spec;
            spec.dims = c.rot_dims;
            spec.base = c.rot_base;
            AGPU_TRY(rope_table_launch(m->ctx, rope, m->P, spec));
        }
        L.lw.norm = L.dkv_norm; L.lw.uk = L.uk.w; L.lw.uv = L.uv.w; L.lw.sink = L.sink; L.lw.rope = rope;
    } else if (c.mixer == AGPU_MIXER_CHANNEL_DELTA) {
        DeltaShape &s = L.ds;
        s.heads = c.heads; s.kv_heads = c.kv_heads; s.dim = c.dim; s.vdim = c.vdim; s.taps = c.conv; s.rank_a = c.decay_rank; s.rank_g = c.gate_rank;
        s.eps = m->cfg.norm_eps;
        if (!delta_supported(s)) return agpu_fail(m->ctx, AGPU_ERR_SHAPE_MISMATCH, "ritevik: channel delta sizes of layer %d not supported", i);
        const int nk = c.kv_heads * c.dim, nv = c.heads * c.vdim;
        L.col_q = 0;
        L.col_k = L.col_q + pad32(nk);
        L.col_v = L.col_k + pad32(nk);
        L.col_b = L.col_v + pad32(nv);
        L.col_a1 = L.col_b + pad32(c.heads);
        L.col_g1 = L.col_a1 + s.rank_ap();
        L.n_plain = L.col_g1 + s.rank_gp();
        AGPU_TRY(m->new_mat(L.in, L.n_plain + 2 * L.ffp, dp));
        m->add_rows(p + "mix.q", L.in, L.col_q, 0, nk, d);
        m->add_rows(p + "mix.k", L.in, L.col_k, 0, nk, d);
        m->add_rows(p + "mix.v", L.in, L.col_v, 0, nv, d);
        m->add_rows(p + "mix.b", L.in, L.col_b, 0, c.heads, d);
        m->add_rows(p + "mix.a1", L.in, L.col_a1, 0, c.decay_rank, d);
        m->add_rows(p + "mix.g1", L.in, L.col_g1, 0, c.gate_rank, d);
        const size_t conv = (size_t)s.channels() * c.conv;
        AGPU_TRY(m->add_vec(p + "mix.q.conv", &L.conv, nk, c.conv, conv, 0));
        AGPU_TRY(m->add_vec(p + "mix.k.conv", &L.conv, nk, c.conv, conv, (size_t)nk * c.conv));
        AGPU_TRY(m->add_vec(p + "mix.v.conv", &L.conv, nv, c.conv, conv, (size_t)2 * nk * c.conv));
        AGPU_TRY(m->add_vec(p + "mix.A_log", &L.a_log, 1, c.heads));
        AGPU_TRY(m->add_vec(p + "mix.dt_bias", &L.dt_bias, 1, (int64_t)c.heads * c.dim));
        AGPU_TRY(m->add_vec(p + "mix.norm", &L.mix_norm, 1, c.vdim));
        AGPU_TRY(m->new_mat(L.a2, c.heads * s.state_row(), s.rank_ap()));
        m->add_head_rows(p + "mix.a2", L.a2, c.heads, c.dim, s.state_row(), c.decay_rank);
        AGPU_TRY(m->new_mat(L.g2, nv, s.rank_gp()));
        m->add_rows(p + "mix.g2", L.g2, 0, 0, nv, c.gate_rank);
        L.dw.conv = L.conv; L.dw.a_log = L.a_log; L.dw.dt_bias = L.dt_bias; L.dw.a2 = L.a2.w; L.dw.g2 = L.g2.w; L.dw.norm = L.mix_norm;
    } else {
        return agpu_fail(m->ctx, AGPU_ERR_UNSUPPORTED, "ritevik: unknown mixer %d of layer %d", c.mixer, i);
    }
    AGPU_TRY(m->new_mat(L.out, dp, L.cat_k()));
    m->add_rows(p + "mix.o", L.out, 0, 0, d, L.mix_w);
    if (c.ff > 0) {
        m->add_rows(p + "mlp.gate", L.in, L.n_plain, 0, c.ff, d, 2);
        m->add_rows(p + "mlp.up", L.in, L.n_plain + 1, 0, c.ff, d, 2);
        m->add_rows(p + "mlp.down", L.out, 0, L.mix_wp, d, c.ff);
    }
    if (m->cfg.side_dim > 0) {
        AGPU_TRY(m->new_mat(L.side_gate, m->side_p, dp));
        m->add_rows(p + "side.gate", L.side_gate, 0, 0, m->cfg.side_dim, d);
        AGPU_TRY(m->new_mat(L.side_proj, dp, m->side_p));
        m->add_rows(p + "side.proj", L.side_proj, 0, 0, d, m->cfg.side_dim);
        AGPU_TRY(m->add_vec(p + "side.norm", &L.side_norm, 1, d));
    }
    m->max_cat = std::max(m->max_cat, L.cat_k());
    m->max_in = std::max(m->max_in, L.n_plain);
    return AGPU_OK;
}

int32_t build(agpu_ritevik *m) {
    const agpu_ritevik_config &c = m->cfg;
    const int d = m->d, dp = m->dp, V = m->V;
    Mat et;
    et.N = V;
    et.K = d;
    AGPU_TRY(m->own((void **)&m->embed, (size_t)V * d * 2, &m->weight_bytes));
    et.w = m->embed;
    m->add_rows("embed", et, 0, 0, V, d);
    AGPU_TRY(m->add_vec("embed.norm", &m->embed_norm, 1, d));
    if (c.loop_times > 0) {
        AGPU_TRY(m->new_mat(m->loop_in, dp, 2 * dp));
        const Mat t = m->loop_in;
        m->add_mat("loop.in", d, 2 * d, [=](const uint16_t *src) {
            int32_t rc = place_rows(m->ctx, t, 0, 1, 0, src, d, d, 2 * d);
            return rc == AGPU_OK ? place_rows(m->ctx, t, 0, 1, dp, src + d, d, d, 2 * d) : rc;
        });
        // rows of the step table have the padded stride of the residual stream
        AGPU_TRY(m->add_vec("loop.step", &m->loop_step, c.loop_times, d, (size_t)c.loop_times * dp, 0, d, dp));
    }
    if (c.side_dim > 0) {
        Mat st;
        st.N = V;
        st.K = c.n_layer * c.side_dim;
        AGPU_TRY(m->own((void **)&m->side_embed, (size_t)st.N * st.K * 2, &m->weight_bytes));
        st.w = m->side_embed;
        m->add_rows("side.embed", st, 0, 0, V, st.K);
    }
    for (int i = 0; i < c.n_layer; ++i) AGPU_TRY(build_layer(m, i));
    AGPU_TRY(m->add_vec("final.norm", &m->final_norm, 1, d));
    AGPU_TRY(m->new_mat(m->head, pad32(V), dp));
    m->add_rows("head", m->head, 0, 0, V, d);

    // the layer runs in order, each with a cache or state of its own
    auto push = [&](int layer, int step) {
        Run r;
        r.layer = layer;
        r.loop_step = step;
        const Layer &L = m->layers[layer];
        if (L.c.mixer == AGPU_MIXER_LATENT_ATTENTION) {
            r.cache = m->latent_elems;
            m->latent_elems += (size_t)m->max_batch * m->P * L.ls.cache_row();
        } else {
            r.state = m->state_floats;
            m->state_floats += (size_t)m->max_batch * L.ds.heads * L.ds.vdim * L.ds.state_row();
            r.ring = m->state_floats;
            m->state_floats += ((size_t)m->max_batch * L.ds.taps * L.ds.channels() + 3) / 4 * 4;
        }
        m->runs.push_back(r);
    };
    const int lo = c.loop_times > 0 ? c.loop_start : c.n_layer, hi = c.loop_times > 0 ? c.loop_stop : c.n_layer;
    for (int i = 0; i < lo; ++i) push(i, -1);
    for (int t = 0; t < c.loop_times; ++t)
        for (int i = lo; i < hi; ++i) push(i, i == lo ? t : -1);
    for (int i = hi; i < c.n_layer; ++i) push(i, -1);
    if (m->latent_elems) AGPU_TRY(m->own(&m->latents, m->latent_elems * (m->f32 ? 4 : 2), &m->cache_bytes));
    if (m->state_floats) AGPU_TRY(m->own((void **)&m->state, m->state_floats * sizeof(float), &m->cache_bytes));
    return AGPU_OK;
}

int32_t mixer(agpu_ritevik *m, const Run &r, int B, int new_len, int max_kv, void *cat, bool cat_bf16) {
    Layer &L = m->layers[r.layer];
    const int R = B * new_len;
    const float *proj = (const float *)m->proj.p;
    if (L.c.mixer == AGPU_MIXER_LATENT_ATTENTION) {
        LatentArgs a;
        a.s = L.ls;
        a.w = L.lw;
        a.q = proj + L.col_q;
        a.down = proj + L.col_k;
        a.ld = L.n_plain;
        a.cache = (char *)m->latents + r.cache * (m->f32 ? 4 : 2);
        a.cache_bf16 = !m->f32;
        a.positions = m->P;
        a.batch = B;
        a.new_len = new_len;
        a.pos_dev = m->pos_dev;
        a.kv_max = max_kv;
        a.out = cat;
        a.ldo = L.cat_k();
        a.out_bf16 = cat_bf16;
        a.qlat = m->qlat.p;
        a.partial = (float *)m->partial.p;
        a.qb = (uint16_t *)m->qb.p;
        a.kx = (uint16_t *)m->kx.p;
        a.vx = (uint16_t *)m->vx.p;
        if (!m->f32 && new_len >= kTiledFrom && latent_tiled_supported(L.ls)) AGPU_TRY(latent_tiled_launch(m->ctx, a));
        else AGPU_TRY(latent_absorbed_launch(m->ctx, a));
    } else {
        DeltaArgs a;
        a.s = L.ds;
        a.w = L.dw;
        a.proj = proj;
        a.ld = L.n_plain;
        a.col_q = L.col_q; a.col_k = L.col_k; a.col_v = L.col_v; a.col_b = L.col_b; a.col_a1 = L.col_a1; a.col_g1 = L.col_g1;
        a.state = m->state + r.state;
        a.ring = m->state + r.ring;
        a.batch = B;
        a.new_len = new_len;
        a.pos_dev = m->pos_dev;
        a.out = cat;
        a.ldo = L.cat_k();
        a.out_bf16 = cat_bf16;
        if (new_len == 1) {
            AGPU_TRY(delta_step_launch(m->ctx, a));
        } else {
            a.qkg = (float *)m->dqkg.p;
            a.v = (float *)m->dv.p;
            a.step = (float *)m->dstep.p;
            a.bkq = (float *)m->dbkq.p;
            a.gate = (float *)m->dgate.p;
            a.o = (float *)m->dout.p;
            AGPU_TRY(delta_prefill_launch(m->ctx, a));
        }
    }
    if (L.mix_w != L.mix_wp) {
        const unsigned blocks = (unsigned)ceil_div((L.mix_wp - L.mix_w) * R, 256);
        if (cat_bf16)
            hipLaunchKernelGGL(zero_columns_kernel<uint16_t>, dim3(blocks), dim3(256), 0, m->ctx->stream, (uint16_t *)cat, L.cat_k(), L.mix_w, L.mix_wp, R);
        else hipLaunchKernelGGL(zero_columns_kernel<float>, dim3(blocks), dim3(256), 0, m->ctx->stream, (float *)cat, L.cat_k(), L.mix_w, L.mix_wp, R);
        return AGPU_LAUNCH_CHECK(m->ctx, "zero_columns_kernel");
    }
    return AGPU_OK;
}

}  // namespace

int32_t agpu_ritevik::launch_forward(const uint32_t *tokens, int B, int new_len, int max_kv, bool all_rows_logits, const ArgmaxAdvance *feed,
                                     bool *fed) {
    (void)feed;
    if (fed) *fed = false;
    const int R = B * new_len;
    const bool gemv = small(R), a16 = !f32 && !gemv;
    float *x = (float *)xa.p, *spare = (float *)xb.p;
    AGPU_TRY(embed_rows_launch(ctx, tokens, embed, d, embed_norm, x, cfg.loop_times > 0 ? (float *)x0.p : nullptr, R, V, d, dp, cfg.norm_eps));
    const float *pending = nullptr;  // the side norm of a layer whose addend still waits in `y`
    auto rows_of = [&](const float *norm_w) {
        DenseRows in;
        in.x = x;
        in.ldx = in.dp = dp;
        in.d = d;
        in.eps = cfg.norm_eps;
        in.norm_w = norm_w;
        in.norm_off = 1.0f;
        if (pending) {
            in.y = (const float *)y.p;
            in.y_w = pending;
        }
        return in;
    };
    for (size_t i = 0; i < runs.size(); ++i) {
        const Run &r = runs[i];
        Layer &L = layers[r.layer];
        if (r.loop_step >= 0) {
            DenseRows in = rows_of(nullptr);
            in.x2 = (const float *)x0.p;
            DenseOut o;
            o.n_plain = o.ldo = dp;
            o.bias = loop_step + (size_t)r.loop_step * dp;
            o.out = spare;
            if (gemv) {
                AGPU_TRY(dense_gemv_launch(ctx, in, loop_in.w, R, loop_in.N, loop_in.K, o));
            } else {
                AGPU_TRY(dense_rows_launch(ctx, in, R, h.p, 2 * dp, a16));
                AGPU_TRY(gemm(h.p, 2 * dp, loop_in, R, o));
            }
            std::swap(x, spare);
            pending = nullptr;
        }
        DenseRows in = rows_of(L.norm1);
        DenseOut o;
        o.n_plain = o.ldo = L.n_plain;
        o.out = (float *)proj.p;
        o.act = a16 ? (void *)((uint16_t *)cat.p + L.mix_wp) : (void *)((float *)cat.p + L.mix_wp);
        o.ld_act = L.cat_k();
        o.act_bf16 = a16;
        if (gemv) {
            if (pending) in.x_out = spare;
            AGPU_TRY(dense_gemv_launch(ctx, in, L.in.w, R, L.in.N, L.in.K, o));
            if (pending) std::swap(x, spare);
        } else {
            if (pending) in.x_out = x;
            AGPU_TRY(dense_rows_launch(ctx, in, R, h.p, dp, a16));
            AGPU_TRY(gemm(h.p, dp, L.in, R, o));
        }
        pending = nullptr;
        AGPU_TRY(mixer(this, r, B, new_len, max_kv, cat.p, a16));
        DenseOut oo;
        oo.n_plain = oo.ldo = oo.ldr = dp;
        oo.out = x;
        oo.residual = x;
        if (gemv) {
            DenseRows ci;
            ci.x = (const float *)cat.p;
            ci.ldx = ci.d = ci.dp = L.cat_k();
            AGPU_TRY(dense_gemv_launch(ctx, ci, L.out.w, R, L.out.N, L.out.K, oo));
        } else {
            AGPU_TRY(gemm(cat.p, L.cat_k(), L.out, R, oo));
        }
        if (cfg.side_dim > 0) {
            DenseOut og, op;
            og.n_plain = og.ldo = side_p;
            og.tab = side_embed;
            og.tokens = tokens;
            og.vocab = V;
            og.tab_ld = cfg.n_layer * cfg.side_dim;
            og.tab_off = r.layer * cfg.side_dim;
            og.tab_n = cfg.side_dim;
            if (a16) og.out_bf16 = (uint16_t *)side.p;
            else og.out = (float *)side.p;
            op.n_plain = op.ldo = dp;
            op.out = (float *)y.p;
            if (gemv) {
                AGPU_TRY(dense_gemv_launch(ctx, rows_of(nullptr), L.side_gate.w, R, L.side_gate.N, L.side_gate.K, og));
                DenseRows si;
                si.x = (const float *)side.p;
                si.ldx = si.d = si.dp = side_p;
                AGPU_TRY(dense_gemv_launch(ctx, si, L.side_proj.w, R, L.side_proj.N, L.side_proj.K, op));
            } else {
                const void *xin = x;
                if (a16) {
                    AGPU_TRY(dense_rows_launch(ctx, rows_of(nullptr), R, h.p, dp, 1));
                    xin = h.p;
                }
                AGPU_TRY(gemm(xin, dp, L.side_gate, R, og));
                AGPU_TRY(gemm(side.p, side_p, L.side_proj, R, op));
            }
            pending = L.side_norm;
        }
        if (tap) {
            if (pending) {
                DenseRows fi = rows_of(nullptr);
                fi.x_out = x;
                AGPU_TRY(dense_rows_launch(ctx, fi, R, nullptr, 0, 0));
                pending = nullptr;
            }
            AGPU_TRY(save_tap(i, x, R));
        }
    }
    const int rows = all_rows_logits ? R : B;
    DenseRows in = rows_of(final_norm);
    in.map_stride = all_rows_logits ? 0 : new_len;
    DenseOut o;
    o.n_plain = o.ldo = logits_stride();
    o.out = (float *)logits.p;
    if (dense_gemv_supported(rows, dp)) return dense_gemv_launch(ctx, in, head.w, rows, head.N, head.K, o);
    AGPU_TRY(dense_rows_launch(ctx, in, rows, h.p, dp, !f32));
    return gemm(h.p, dp, head, rows, o);
}

int32_t agpu_ritevik::ensure_buffers(int B, int new_len, bool all_rows_logits) {
    const size_t R = (size_t)B * new_len, f = sizeof(float);
    if (R > 65535) return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "ritevik: %zu rows in one forward exceed 65535; feed the prompt in portions", R);
    AGPU_TRY(ensure(this, xa, R * dp * f));
    AGPU_TRY(ensure(this, xb, R * dp * f));
    if (cfg.loop_times > 0) AGPU_TRY(ensure(this, x0, R * dp * f));
    AGPU_TRY(ensure(this, h, R * dp * (cfg.loop_times > 0 ? 2 : 1) * f));
    AGPU_TRY(ensure(this, proj, R * max_in * f));
    AGPU_TRY(ensure(this, cat, R * max_cat * f));
    if (cfg.side_dim > 0) {
        AGPU_TRY(ensure(this, y, R * dp * f));
        AGPU_TRY(ensure(this, side, R * side_p * f));
    }
    AGPU_TRY(ensure(this, logits, (all_rows_logits ? R : (size_t)B) * logits_stride() * f));
    const int kv = std::min(cache_len + new_len, P);
    for (const Layer &L : layers) {
        if (L.c.mixer == AGPU_MIXER_LATENT_ATTENTION) {
            const LatentShape &s = L.ls;
            if (!f32 && new_len >= kTiledFrom && latent_tiled_supported(s)) {
                AGPU_TRY(ensure(this, qb, R * s.heads * s.query_row() * 2));
                AGPU_TRY(ensure(this, kx, (size_t)B * kv * s.heads * s.dimp() * 2));
                AGPU_TRY(ensure(this, vx, (size_t)B * s.heads * s.vdimp() * latent_kv_stride(kv) * 2));
            } else {
                AGPU_TRY(ensure(this, qlat, R * s.heads * s.cache_row() * f));
                AGPU_TRY(ensure(this, partial, latent_partial_floats(s, (int)R, latent_splits(ctx, s, (int)R, P)) * f));
            }
        } else if (new_len > 1) {
            const DeltaShape &s = L.ds;
            AGPU_TRY(ensure(this, dqkg, R * s.heads * 3 * s.state_row() * f));
            AGPU_TRY(ensure(this, dv, R * s.heads * s.vdim * f));
            AGPU_TRY(ensure(this, dstep, R * s.heads * s.state_row() * f));
            AGPU_TRY(ensure(this, dbkq, R * (s.heads + s.kv_heads) * f));
            AGPU_TRY(ensure(this, dgate, R * s.heads * s.vdim * f));
            AGPU_TRY(ensure(this, dout, R * s.heads * s.vdim * f));
        }
    }
    return AGPU_OK;
}

void agpu_ritevik::mix_addresses(AddrHash &hash, bool) const {
    for (void *p : owned) hash.mix(p);
    for (const DevBuf *b : {&xa, &xb, &x0, &y, &h, &proj, &cat, &side, &qlat, &partial}) hash.mix(b->p);
}

int32_t agpu_ritevik::reset_state() { return fill_u32(ctx, state, 0u, state_floats); }

AGPU_EXPORT int32_t agpu_ritevik_create(agpu_ctx *ctx, const agpu_ritevik_config *cfg, const agpu_ritevik_layer *layers, agpu_ritevik **out) {
    AGPU_REQUIRE_CTX(ctx);
    if (!cfg || !layers || !out) return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "ritevik_create: null pointer");
    *out = nullptr;
    if (cfg->n_layer <= 0 || cfg->width <= 0 || cfg->vocab_size <= 0 || cfg->n_positions <= 0 || cfg->max_batch <= 0 || cfg->max_batch > 1024 ||
        cfg->side_dim < 0 || cfg->loop_times < 0 || (cfg->dtype != AGPU_DTYPE_BF16 && cfg->dtype != AGPU_DTYPE_F32))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "ritevik_create: bad configuration");
    if (cfg->loop_times > 0 && (cfg->loop_start < 0 || cfg->loop_stop <= cfg->loop_start || cfg->loop_stop > cfg->n_layer))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "ritevik_create: loop over layers %d .. %d of %d", cfg->loop_start, cfg->loop_stop, cfg->n_layer);
    agpu_ritevik *m = new (std::nothrow) agpu_ritevik();
    if (!m) return AGPU_ERR_NULL_POINTER;
    m->cfg = *cfg;
    m->d = cfg->width;
    m->dp = pad32(m->d);
    m->side_p = pad32(cfg->side_dim);
    m->f32 = cfg->dtype == AGPU_DTYPE_F32;
    m->layers.resize((size_t)cfg->n_layer);
    for (int i = 0; i < cfg->n_layer; ++i) m->layers[(size_t)i].c = layers[i];
    int32_t rc = lm_init(m, ctx, cfg->vocab_size, cfg->n_positions, cfg->max_batch, cfg->argmax_last);
    if (rc == AGPU_OK) rc = build(m);
    if (rc == AGPU_OK) rc = agpu_hip(ctx, hipStreamSynchronize(ctx->stream), "hipStreamSynchronize");
    if (rc != AGPU_OK) {
        agpu_ritevik_destroy(m);
        return rc;
    }
    *out = m;
    return AGPU_OK;
}

AGPU_EXPORT int32_t agpu_ritevik_destroy(agpu_ritevik *m) {
    if (!m) return AGPU_OK;
    layered_release(m, {&m->xa, &m->xb, &m->x0, &m->y, &m->h, &m->proj, &m->cat, &m->side, &m->qlat, &m->partial, &m->qb, &m->kx, &m->vx, &m->dqkg, &m->dv,
                        &m->dstep, &m->dbkq, &m->dgate, &m->dout});
    delete m;
    return AGPU_OK;
}

AGPU_EXPORT int32_t agpu_ritevik_set_tensor(agpu_ritevik *m, const char *name, const void *data_host, int32_t dtype, int64_t rows, int64_t cols) {
    return m ? lm_set_tensor(m, name, data_host, dtype, rows, cols) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_ritevik_tensor_info(const agpu_ritevik *m, int32_t i, const char **name_out, int64_t *rows_out, int64_t *cols_out,
                                             int32_t *is_set_out) {
    return m ? lm_tensor_info(m, i, name_out, rows_out, cols_out, is_set_out) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int64_t agpu_ritevik_weight_bytes(const agpu_ritevik *m) { return m ? m->weight_bytes : 0; }
AGPU_EXPORT int64_t agpu_ritevik_cache_bytes(const agpu_ritevik *m) { return m ? m->cache_bytes : 0; }
AGPU_EXPORT int32_t agpu_ritevik_layer_runs(const agpu_ritevik *m) { return m ? (int32_t)m->runs.size() : 0; }

AGPU_EXPORT int32_t agpu_ritevik_reset_cache(agpu_ritevik *m) { return m ? lm_reset_cache(m) : AGPU_ERR_NULL_POINTER; }
AGPU_EXPORT int32_t agpu_ritevik_cache_len(const agpu_ritevik *m) { return m ? m->cache_len : 0; }

AGPU_EXPORT int32_t agpu_ritevik_forward_cached(agpu_ritevik *m, const uint32_t *tokens, int32_t batch, int32_t new_len, float *logits,
                                                int32_t all_rows) {
    return m ? lm_forward_cached(m, tokens, batch, new_len, logits, all_rows) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_ritevik_generate_cached(agpu_ritevik *m, const uint32_t *prompt_host, int32_t batch, int32_t prompt_len,
                                                 int32_t max_new_tokens, int32_t eos, uint32_t *tokens_out_host, int32_t *lengths_out_host,
                                                 float *timing_ms_out_host) {
    if (!m) return AGPU_ERR_NULL_POINTER;
    return lm_generate_cached(m, prompt_host, batch, prompt_len, max_new_tokens, eos, tokens_out_host, lengths_out_host, timing_ms_out_host);
}

AGPU_EXPORT int32_t agpu_ritevik_generate(agpu_ritevik *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens, int32_t eos,
                                          uint32_t *tokens_out_host, int32_t *length_out_host) {
    return m ? lm_generate(m, prompt_host, prompt_len, max_new_tokens, eos, tokens_out_host, length_out_host) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_ritevik_generate_cached_sampling(agpu_ritevik *m, const uint32_t *prompt_host, int32_t prompt_len, int32_t max_new_tokens,
                                                          int32_t top_k, float temperature, uint64_t *rng_state, int32_t eos,
                                                          uint32_t *tokens_out_host, int32_t *length_out_host) {
    if (!m) return AGPU_ERR_NULL_POINTER;
    return lm_generate_cached_sampling(m, prompt_host, prompt_len, max_new_tokens, top_k, temperature, rng_state, eos, tokens_out_host, length_out_host);
}

AGPU_EXPORT int32_t agpu_ritevik_set_decode_mode(agpu_ritevik *m, int32_t mode) { return m ? lm_set_decode_mode(m, mode) : AGPU_ERR_NULL_POINTER; }

AGPU_EXPORT int32_t agpu_ritevik_decode_steps(agpu_ritevik *m, int32_t batch, int32_t steps, float *ms_total_out_host) {
    return m ? lm_decode_steps(m, batch, steps, ms_total_out_host) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_ritevik_last_logits(agpu_ritevik *m, int32_t batch, float *logits_out_host) {
    return m ? lm_last_logits(m, batch, logits_out_host) : AGPU_ERR_NULL_POINTER;
}

AGPU_EXPORT int32_t agpu_ritevik_layer_streams(agpu_ritevik *m, const uint32_t *tokens, int32_t new_len, float *streams_out_host) {
    return m ? lm_layer_streams(m, tokens, new_len, streams_out_host) : AGPU_ERR_NULL_POINTER;
}
