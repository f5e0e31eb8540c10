// C entry points of the bf16-weight layers (include/agpu.h) over the launchers the model drivers use.
#include <algorithm>

#include "dense_linear.h"
#include "gated_delta.h"
#include "gated_lru.h"
#include "grouped_attention.h"
#include "latent_attention.h"
#include "matrix_memory.h"

namespace {

__global__ void set_position_kernel(int *pos, int value) { *pos = value; }

size_t align256(size_t n) { return (n + 255) / 256 * 256; }

// Cuts a caller's workspace into pieces; with a null base it only counts.
struct Carver {
    char *base;
    size_t at = 0;
    template <typename T>
    T *take(size_t n) {
        T *p = base ? (T *)(base + at) : nullptr;
        at += align256(n * sizeof(T));
        return p;
    }
};

LatentShape latent_shape(const agpu_latent_attention_desc &d) {
    LatentShape s;
    s.heads = d.heads; s.dim = d.dim; s.rot = d.rot_dim; s.rot_dims = d.rot_dims; s.vdim = d.vdim; s.rank = d.rank;
    s.scale = d.scale; s.eps = d.eps;
    return s;
}

bool latent_desc_ok(const agpu_latent_attention_desc &d) {
    return d.heads > 0 && d.dim > 0 && d.dim % 8 == 0 && d.dim <= 1024 && d.rot_dim >= 0 && d.rot_dim % 8 == 0 && d.rot_dims >= 0 && d.rot_dims % 2 == 0 &&
           d.rot_dims <= d.rot_dim && d.vdim > 0 && d.vdim % 32 == 0 && d.rank > 0 && d.rank % 32 == 0 && d.rank <= 1024 && d.positions > 0 && d.batch > 0 &&
           d.new_len > 0 && d.cached >= 0 && (int64_t)d.batch * d.new_len <= 65535 && d.cached <= d.positions - d.new_len && d.ld > 0 &&
           d.ldo >= d.heads * d.vdim && (d.cache_dtype == AGPU_DTYPE_BF16 || d.cache_dtype == AGPU_DTYPE_F32);
}

void latent_carve(const agpu_ctx *ctx, const agpu_latent_attention_desc &d, Carver &c, LatentArgs &a, int **pos) {
    const LatentShape s = latent_shape(d);
    const int rows = d.batch * d.new_len, kv = d.cached + d.new_len;
    *pos = c.take<int>(1);
    if (d.tiled) {
        a.qb = c.take<uint16_t>((size_t)rows * s.heads * s.query_row());
        a.kx = c.take<uint16_t>((size_t)d.batch * kv * s.heads * s.dimp());
        a.vx = c.take<uint16_t>((size_t)d.batch * s.heads * s.vdimp() * latent_kv_stride(kv));
    } else {
        a.qlat = c.take<float>((size_t)rows * s.heads * s.cache_row());
        a.partial = c.take<float>(latent_partial_floats(s, rows, latent_splits(ctx, s, rows, kv)));
    }
}

DeltaShape delta_shape(const agpu_channel_delta_desc &d) {
    DeltaShape s;
    s.heads = d.heads; s.kv_heads = d.kv_heads; s.dim = d.dim; s.vdim = d.vdim; s.taps = d.taps; s.rank_a = d.decay_rank; s.rank_g = d.gate_rank;
    s.eps = d.eps;
    return s;
}

bool delta_desc_ok(const agpu_channel_delta_desc &d) {
    for (int c : {d.col_q, d.col_k, d.col_v, d.col_b, d.col_a1, d.col_g1})
        if (c < 0 || c % 4 != 0) return false;
    return delta_supported(delta_shape(d)) && d.dim % 32 == 0 && d.decay_rank % 32 == 0 && d.gate_rank % 32 == 0 && d.batch > 0 && d.new_len > 0 &&
           d.cached >= 0 && d.ld > 0 && d.ld % 4 == 0 && d.ldo >= d.heads * d.vdim && (int64_t)d.batch * d.new_len <= 65535;
}

void delta_carve(const agpu_channel_delta_desc &d, Carver &c, DeltaArgs &a, int **pos) {
    const DeltaShape s = delta_shape(d);
    const size_t rows = (size_t)d.batch * d.new_len;
    *pos = c.take<int>(1);
    if (d.new_len == 1) return;
    a.qkg = c.take<float>(rows * s.heads * 3 * s.state_row());
    a.v = c.take<float>(rows * s.heads * s.vdim);
    a.step = c.take<float>(rows * s.heads * s.state_row());
    a.bkq = c.take<float>(rows * (s.heads + s.kv_heads));
    a.gate = c.take<float>(rows * s.heads * s.vdim);
    a.o = c.take<float>(rows * s.heads * s.vdim);
}

bool rows_ok(int batch, int new_len, int cached) { return batch > 0 && new_len > 0 && cached >= 0 && (int64_t)batch * new_len <= 65535; }

GroupedShape grouped_shape(const agpu_grouped_attention_desc &d) {
    GroupedShape s;
    s.heads = d.heads; s.kv_heads = d.kv_heads; s.dim = d.dim; s.vdim = d.vdim; s.rot_dims = d.rot_dims; s.scale = d.scale; s.softcap = d.softcap;
    return s;
}

bool grouped_desc_ok(const agpu_grouped_attention_desc &d) {
    return grouped_supported(grouped_shape(d)) && d.dim % 32 == 0 && d.vdim % 32 == 0 && rows_ok(d.batch, d.new_len, d.cached) && d.positions > 0 &&
           d.cached <= d.positions - d.new_len && d.ld > 0 && d.ld % 4 == 0 && d.ldo % 4 == 0 && d.ldo >= d.heads * d.vdim &&
           (d.cache_dtype == AGPU_DTYPE_BF16 || d.cache_dtype == AGPU_DTYPE_F32);
}

void grouped_carve(const agpu_ctx *ctx, const agpu_grouped_attention_desc &d, Carver &c, GroupedArgs &a, int **pos, float2 **no_turn) {
    *pos = c.take<int>(1);
    *no_turn = c.take<float2>(1);
    a.partial = c.take<float>(grouped_partial_floats(ctx, grouped_shape(d), d.batch, d.new_len, d.cached + d.new_len));
}

MemoryShape memory_shape(const agpu_matrix_memory_desc &d) {
    MemoryShape s;
    s.heads = d.heads; s.dim = d.dim; s.vdim = d.vdim; s.cap = d.gate_cap;
    return s;
}

bool memory_desc_ok(const agpu_matrix_memory_desc &d) {
    return memory_supported(memory_shape(d)) && d.dim % 32 == 0 && d.vdim % 32 == 0 && rows_ok(d.batch, d.new_len, d.cached) && d.ld > 0 && d.ld % 4 == 0 &&
           d.ldo % 4 == 0 && d.ldo >= d.heads * d.vdim;
}

void memory_carve(const agpu_matrix_memory_desc &d, Carver &c, MemoryArgs &a, int **pos) {
    *pos = c.take<int>(1);
    if (d.new_len > 1) a.scratch = c.take<char>(memory_scratch_bytes(memory_shape(d), d.batch, d.new_len));
}

LruShape lru_shape(const agpu_gated_lru_desc &d) {
    LruShape s;
    s.width = d.width; s.blocks = d.blocks; s.taps = d.taps;
    return s;
}

bool lru_desc_ok(const agpu_gated_lru_desc &d) {
    return lru_supported(lru_shape(d)) && d.width / d.blocks % 32 == 0 && rows_ok(d.batch, d.new_len, d.cached) && d.ld > 0 && d.ld % 4 == 0 &&
           d.ldo >= d.width && d.col_y >= 0 && d.col_y % 4 == 0 && d.col_x >= 0 && d.col_x % 4 == 0;
}

void lru_carve(const agpu_gated_lru_desc &d, Carver &c, LruArgs &a, int **pos) {
    const LruShape s = lru_shape(d);
    const size_t rows = (size_t)d.batch * d.new_len;
    *pos = c.take<int>(1);
    if (d.new_len == 1) return;
    a.u = c.take<float>(rows * s.widthp());
    a.gates = c.take<float>(rows * 2 * s.widthp());
    a.carries = c.take<float>(lru_carry_floats(s, d.batch, d.new_len));
}

int32_t set_position(agpu_ctx *ctx, int *pos, int value) {
    hipLaunchKernelGGL(set_position_kernel, dim3(1), dim3(1), 0, ctx->stream, pos, value);
    return AGPU_LAUNCH_CHECK(ctx, "set_position_kernel");
}

}  // namespace

AGPU_EXPORT int32_t agpu_rms_norm(agpu_ctx *ctx, const float *x, const float *weight, float weight_offset, float *y, int32_t rows, int32_t d, float eps) {
    AGPU_REQUIRE_CTX(ctx);
    AGPU_REQUIRE_PTR(ctx, x);
    AGPU_REQUIRE_PTR(ctx, weight);
    AGPU_REQUIRE_PTR(ctx, y);
    if (rows <= 0 || d <= 0) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "rms_norm: rows %d, d %d", rows, d);
    DenseRows in;
    in.x = x;
    in.ldx = in.d = in.dp = d;
    in.norm_w = weight;
    in.norm_off = weight_offset;
    in.eps = eps;
    return dense_rows_launch(ctx, in, rows, y, d, 0);
}

AGPU_EXPORT int32_t agpu_dense_linear(agpu_ctx *ctx, const float *x, const uint16_t *w, const float *bias, const float *residual, float *y, int32_t M,
                                      int32_t N, int32_t K, int32_t dtype, uint32_t flags) {
    AGPU_REQUIRE_CTX(ctx);
    AGPU_REQUIRE_PTR(ctx, x);
    AGPU_REQUIRE_PTR(ctx, w);
    AGPU_REQUIRE_PTR(ctx, y);
    const bool gated = (flags & AGPU_DENSE_GATED) != 0;
    if (M <= 0 || N <= 0 || K <= 0 || K % 32 != 0 || (gated && (N % 2 != 0 || bias || residual)) || (dtype != AGPU_DTYPE_BF16 && dtype != AGPU_DTYPE_F32))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "dense_linear: M %d, N %d, K %d, dtype %d, flags 0x%x", M, N, K, dtype, flags);
    DenseOut o;
    if (gated) {
        o.act = y;
        o.ld_act = N / 2;
    } else {
        o.n_plain = N;
        o.out = y;
        o.ldo = o.ldr = N;
        o.bias = bias;
        o.residual = residual;
    }
    DenseRows in;
    in.x = x;
    in.ldx = in.d = in.dp = K;
    if (dense_gemv_supported(M, K)) return dense_gemv_launch(ctx, in, w, M, N, K, o);
    if (dtype == AGPU_DTYPE_F32) return dense_gemm_f32_launch(ctx, x, K, w, K, M, N, K, o);
    if ((size_t)M * K * 2 > ctx->ws_bytes / 2)
        return agpu_fail(ctx, AGPU_ERR_WORKSPACE, "dense_linear: %d x %d rows do not fit the context's scratch", M, K);
    const int32_t rc = dense_rows_launch(ctx, in, M, ctx->workspace, K, 1);
    return rc == AGPU_OK ? dense_gemm_bf16_launch(ctx, (const uint16_t *)ctx->workspace, K, w, K, M, N, K, o) : rc;
}

AGPU_EXPORT int32_t agpu_rope_table(agpu_ctx *ctx, float *table, int32_t positions, int32_t dims, double base) {
    AGPU_REQUIRE_CTX(ctx);
    AGPU_REQUIRE_PTR(ctx, table);
    if (positions <= 0 || dims <= 0 || dims % 2 != 0 || !(base > 0.0)) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "rope_table: positions %d, dims %d", positions, dims);
    RopeSpec spec;
    spec.dims = dims;
    spec.base = base;
    return rope_table_launch(ctx, (float2 *)table, positions, spec);
}

AGPU_EXPORT int32_t agpu_rope_table_stretched(agpu_ctx *ctx, float *table, int32_t positions, int32_t dims, double base, double factor, double original,
                                              double fast, double slow) {
    AGPU_REQUIRE_CTX(ctx);
    AGPU_REQUIRE_PTR(ctx, table);
    if (positions <= 0 || dims <= 0 || dims % 2 != 0 || !(base > 1.0) || !(factor > 0.0) || !(original > 0.0) || !(fast > 0.0) || !(slow > 0.0))
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "rope_table_stretched: positions %d, dims %d, base %g, factor %g", positions, dims, base, factor);
    RopeSpec spec;
    spec.dims = dims; spec.base = base; spec.factor = factor; spec.original = original; spec.fast = fast; spec.slow = slow;
    return rope_table_launch(ctx, (float2 *)table, positions, spec);
}

AGPU_EXPORT int32_t agpu_latent_cache_row(int32_t rank, int32_t rot_dim) {
    LatentShape s;
    s.rank = rank;
    s.rot = rot_dim;
    return s.cache_row();
}

AGPU_EXPORT size_t agpu_latent_attention_workspace_bytes(const agpu_ctx *ctx, const agpu_latent_attention_desc *desc) {
    if (!ctx || !desc || !latent_desc_ok(*desc)) return 0;
    Carver c{nullptr};
    LatentArgs a;
    int *pos;
    latent_carve(ctx, *desc, c, a, &pos);
    return c.at;
}

AGPU_EXPORT int32_t agpu_latent_attention(agpu_ctx *ctx, const agpu_latent_attention_desc *desc, const float *q, const float *down, const float *norm,
                                          const uint16_t *uk, const uint16_t *uv, const float *sink, const float *rope, void *cache, float *out,
                                          void *workspace) {
    AGPU_REQUIRE_CTX(ctx);
    for (const void *p : {(const void *)desc, (const void *)q, (const void *)down, (const void *)norm, (const void *)uk, (const void *)uv, (const void *)cache,
                          (const void *)out, (const void *)workspace})
        AGPU_REQUIRE_PTR(ctx, p);
    if (!latent_desc_ok(*desc)) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "latent_attention: sizes not supported");
    if (desc->rot_dims > 0) AGPU_REQUIRE_PTR(ctx, rope);
    LatentArgs a;
    a.s = latent_shape(*desc);
    a.w.norm = norm; a.w.uk = uk; a.w.uv = uv; a.w.sink = sink; a.w.rope = (const float2 *)rope;
    a.q = q; a.down = down; a.ld = desc->ld;
    a.cache = cache; a.cache_bf16 = desc->cache_dtype == AGPU_DTYPE_BF16; a.positions = desc->positions;
    a.batch = desc->batch; a.new_len = desc->new_len; a.kv_max = desc->cached + desc->new_len;
    a.out = out; a.ldo = desc->ldo;
    Carver c{(char *)workspace};
    int *pos = nullptr;
    latent_carve(ctx, *desc, c, a, &pos);
    a.pos_dev = pos;
    const int32_t rc = set_position(ctx, pos, desc->cached);
    if (rc != AGPU_OK) return rc;
    return desc->tiled ? latent_tiled_launch(ctx, a) : latent_absorbed_launch(ctx, a);
}

AGPU_EXPORT size_t agpu_channel_delta_workspace_bytes(const agpu_ctx *ctx, const agpu_channel_delta_desc *desc) {
    if (!ctx || !desc || !delta_desc_ok(*desc)) return 0;
    Carver c{nullptr};
    DeltaArgs a;
    int *pos;
    delta_carve(*desc, c, a, &pos);
    return c.at;
}

AGPU_EXPORT int32_t agpu_channel_delta(agpu_ctx *ctx, const agpu_channel_delta_desc *desc, const float *proj, const float *conv, const float *a_log,
                                       const float *dt_bias, const uint16_t *a2, const uint16_t *g2, const float *norm, float *state, float *ring,
                                       float *out, void *workspace) {
    AGPU_REQUIRE_CTX(ctx);
    for (const void *p : {(const void *)desc, (const void *)proj, (const void *)conv, (const void *)a_log, (const void *)dt_bias, (const void *)a2,
                          (const void *)g2, (const void *)norm, (const void *)state, (const void *)ring, (const void *)out, (const void *)workspace})
        AGPU_REQUIRE_PTR(ctx, p);
    if (!delta_desc_ok(*desc)) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "channel_delta: sizes not supported");
    const agpu_channel_delta_desc &d = *desc;
    DeltaArgs a;
    a.s = delta_shape(d);
    a.w.conv = conv; a.w.a_log = a_log; a.w.dt_bias = dt_bias; a.w.a2 = a2; a.w.g2 = g2; a.w.norm = norm;
    a.proj = proj; a.ld = d.ld;
    a.col_q = d.col_q; a.col_k = d.col_k; a.col_v = d.col_v; a.col_b = d.col_b; a.col_a1 = d.col_a1; a.col_g1 = d.col_g1;
    a.state = state; a.ring = ring; a.batch = d.batch; a.new_len = d.new_len; a.out = out; a.ldo = d.ldo;
    Carver c{(char *)workspace};
    int *pos = nullptr;
    delta_carve(d, c, a, &pos);
    a.pos_dev = pos;
    const int32_t rc = set_position(ctx, pos, d.cached);
    if (rc != AGPU_OK) return rc;
    return d.new_len == 1 ? delta_step_launch(ctx, a) : delta_prefill_launch(ctx, a);
}

AGPU_EXPORT int32_t agpu_grouped_kv_stride(int32_t positions) { return grouped_kv_stride(positions); }

AGPU_EXPORT size_t agpu_grouped_attention_workspace_bytes(const agpu_ctx *ctx, const agpu_grouped_attention_desc *desc) {
    if (!ctx || !desc || !grouped_desc_ok(*desc)) return 0;
    Carver c{nullptr};
    GroupedArgs a;
    int *pos;
    float2 *no_turn;
    grouped_carve(ctx, *desc, c, a, &pos, &no_turn);
    return c.at;
}

AGPU_EXPORT int32_t agpu_grouped_attention(agpu_ctx *ctx, const agpu_grouped_attention_desc *desc, const float *q, const float *k, const float *v,
                                           const float *gate, const float *sink, const float *rope, void *kcache, void *vcache, float *out,
                                           void *workspace) {
    AGPU_REQUIRE_CTX(ctx);
    for (const void *p : {(const void *)desc, (const void *)q, (const void *)k, (const void *)v, (const void *)kcache, (const void *)vcache, (const void *)out,
                          (const void *)workspace})
        AGPU_REQUIRE_PTR(ctx, p);
    if (!grouped_desc_ok(*desc)) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "grouped_attention: sizes not supported");
    if (desc->rot_dims > 0) AGPU_REQUIRE_PTR(ctx, rope);
    const agpu_grouped_attention_desc &d = *desc;
    GroupedArgs a;
    a.s = grouped_shape(d);
    a.q = q; a.k = k; a.v = v; a.gate = gate; a.sink = sink; a.ld = d.ld;
    a.kcache = kcache; a.vcache = vcache; a.cache_bf16 = d.cache_dtype == AGPU_DTYPE_BF16; a.positions = d.positions;
    a.batch = d.batch; a.new_len = d.new_len; a.kv_max = d.cached + d.new_len;
    a.out = out; a.ldo = d.ldo;
    Carver c{(char *)workspace};
    int *pos = nullptr;
    float2 *no_turn = nullptr;
    grouped_carve(ctx, d, c, a, &pos, &no_turn);
    a.pos_dev = pos;
    a.rope = rope ? (const float2 *)rope : no_turn;
    const int32_t rc = set_position(ctx, pos, d.cached);
    return rc == AGPU_OK ? grouped_attention_launch(ctx, a) : rc;
}

AGPU_EXPORT size_t agpu_matrix_memory_workspace_bytes(const agpu_ctx *ctx, const agpu_matrix_memory_desc *desc) {
    if (!ctx || !desc || !memory_desc_ok(*desc)) return 0;
    Carver c{nullptr};
    MemoryArgs a;
    int *pos;
    memory_carve(*desc, c, a, &pos);
    return c.at;
}

AGPU_EXPORT int32_t agpu_matrix_memory(agpu_ctx *ctx, const agpu_matrix_memory_desc *desc, const float *q, const float *k, const float *v, const float *i,
                                       const float *f, float *state, float *norm, float *out, void *workspace) {
    AGPU_REQUIRE_CTX(ctx);
    for (const void *p : {(const void *)desc, (const void *)q, (const void *)k, (const void *)v, (const void *)i, (const void *)f, (const void *)state,
                          (const void *)norm, (const void *)out, (const void *)workspace})
        AGPU_REQUIRE_PTR(ctx, p);
    if (!memory_desc_ok(*desc)) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "matrix_memory: sizes not supported");
    const agpu_matrix_memory_desc &d = *desc;
    MemoryArgs a;
    a.s = memory_shape(d);
    a.q = q; a.k = k; a.v = v; a.i = i; a.f = f; a.ld = d.ld;
    a.state = state; a.norm = norm; a.batch = d.batch; a.new_len = d.new_len; a.out = out; a.ldo = d.ldo;
    Carver c{(char *)workspace};
    int *pos = nullptr;
    memory_carve(d, c, a, &pos);
    a.pos_dev = pos;
    const int32_t rc = set_position(ctx, pos, d.cached);
    return rc == AGPU_OK ? memory_launch(ctx, a) : rc;
}

AGPU_EXPORT size_t agpu_gated_lru_workspace_bytes(const agpu_ctx *ctx, const agpu_gated_lru_desc *desc) {
    if (!ctx || !desc || !lru_desc_ok(*desc)) return 0;
    Carver c{nullptr};
    LruArgs a;
    int *pos;
    lru_carve(*desc, c, a, &pos);
    return c.at;
}

AGPU_EXPORT int32_t agpu_gated_lru(agpu_ctx *ctx, const agpu_gated_lru_desc *desc, const float *proj, const float *conv, const float *conv_bias,
                                   const uint16_t *gates, const float *gate_bias, const float *lam, float *state, float *ring, float *out,
                                   void *workspace) {
    AGPU_REQUIRE_CTX(ctx);
    for (const void *p : {(const void *)desc, (const void *)proj, (const void *)conv, (const void *)conv_bias, (const void *)gates, (const void *)gate_bias,
                          (const void *)lam, (const void *)state, (const void *)ring, (const void *)out, (const void *)workspace})
        AGPU_REQUIRE_PTR(ctx, p);
    if (!lru_desc_ok(*desc)) return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "gated_lru: sizes not supported");
    const agpu_gated_lru_desc &d = *desc;
    LruArgs a;
    a.s = lru_shape(d);
    a.w.conv = conv; a.w.conv_bias = conv_bias; a.w.gates = gates; a.w.gate_bias = gate_bias; a.w.lam = lam;
    a.proj = proj; a.ld = d.ld; a.col_y = d.col_y; a.col_x = d.col_x;
    a.state = state; a.ring = ring; a.batch = d.batch; a.new_len = d.new_len; a.out = out; a.ldo = d.ldo;
    Carver c{(char *)workspace};
    int *pos = nullptr;
    lru_carve(d, c, a, &pos);
    a.pos_dev = pos;
    const int32_t rc = set_position(ctx, pos, d.cached);
    return rc == AGPU_OK ? lru_launch(ctx, a) : rc;
}
