// Weight slots, owned memory and layer taps of the models with bf16 weights (layered_model.h).
#include "layered_model.h"

#include <cstring>

namespace {

__global__ __launch_bounds__(256) void embed_rows_kernel(const uint32_t *__restrict__ tokens, const uint16_t *__restrict__ table, int ld,
                                                         const float *__restrict__ weight, float *x, float *x0, int vocab, int d, int dp, float eps) {
    __shared__ float red[4];
    const int row = blockIdx.x, t = threadIdx.x;
    const uint16_t *e = table + (size_t)min(tokens[row], (uint32_t)(vocab - 1)) * ld;
    float rs = 1.0f;
    if (weight) {
        float s = 0.0f;
        for (int k = t; k < d; k += 256) {
            const float v = bf16_to_f32(e[k]);
            s += v * v;
        }
        s = wave_sum(s);
        if ((t & 63) == 0) red[t >> 6] = s;
        __syncthreads();
        rs = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)d + eps);
    }
    for (int k = t; k < dp; k += 256) {
        const float v = k < d ? bf16_to_f32(e[k]) * rs * (weight ? 1.0f + weight[k] : 1.0f) : 0.0f;
        x[(size_t)row * dp + k] = v;
        if (x0) x0[(size_t)row * dp + k] = v;
    }
}

}  // namespace

int32_t LayeredModel::own(void **p, size_t bytes, int64_t *count) {
    bytes = (bytes + 15) / 16 * 16;
    AGPU_TRY(dev_alloc(ctx, p, bytes));
    owned.push_back(*p);
    if (count) *count += (int64_t)bytes;
    return fill_u32(ctx, *p, 0u, bytes / 4);
}

int32_t LayeredModel::new_mat(Mat &t, int N, int K) {
    t.N = N;
    t.K = K;
    return own((void **)&t.w, (size_t)N * K * 2, &weight_bytes);
}

// `rows` rows of `cols` values to rows row0, row0 + row_step, ... of t, from column col0 on.
int32_t place_rows(agpu_ctx *ctx, const Mat &t, int row0, int row_step, int col0, const uint16_t *src, int64_t rows, int64_t cols, int64_t src_ld) {
    hipError_t e = hipMemcpy2DAsync(t.w + (size_t)row0 * t.K + col0, (size_t)row_step * t.K * 2, src, (size_t)src_ld * 2, (size_t)cols * 2, (size_t)rows,
                                    hipMemcpyHostToDevice, ctx->stream);
    if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
    return agpu_hip(ctx, e, "hipMemcpy2DAsync(weights)");
}

void LayeredModel::add_mat(const std::string &name, int64_t rows, int64_t cols, std::function<int32_t(const uint16_t *)> place) {
    Slot s;
    s.name = name;
    s.rows = rows;
    s.cols = cols;
    s.place = std::move(place);
    slots.push_back(std::move(s));
}

void LayeredModel::add_rows(const std::string &name, Mat t, int row0, int col0, int64_t rows, int64_t cols, int row_step) {
    add_mat(name, rows, cols, [=](const uint16_t *src) { return place_rows(ctx, t, row0, row_step, col0, src, rows, cols, cols); });
}

void LayeredModel::add_head_rows(const std::string &name, Mat t, int heads, int per, int per_p, int64_t cols, int row0) {
    add_mat(name, (int64_t)heads * per, cols, [=](const uint16_t *src) {
        int32_t rc = AGPU_OK;
        for (int h = 0; h < heads && rc == AGPU_OK; ++h) rc = place_rows(ctx, t, row0 + h * per_p, 1, 0, src + (size_t)h * per * cols, per, cols, cols);
        return rc;
    });
}

void LayeredModel::add_head_cols(const std::string &name, Mat t, int heads, int per, int per_p, int64_t rows) {
    add_mat(name, rows, (int64_t)heads * per, [=](const uint16_t *src) {
        int32_t rc = AGPU_OK;
        for (int h = 0; h < heads && rc == AGPU_OK; ++h) rc = place_rows(ctx, t, 0, 1, h * per_p, src + (size_t)h * per, rows, per, (int64_t)heads * per);
        return rc;
    });
}

int32_t LayeredModel::add_vec(const std::string &name, float **dst, int64_t rows, int64_t cols, size_t alloc, size_t off, size_t part, size_t part_ld) {
    if (!*dst) AGPU_TRY(own((void **)dst, (alloc ? alloc : (size_t)(rows * cols)) * sizeof(float), &weight_bytes));
    Slot s;
    s.name = name;
    s.rows = rows;
    s.cols = cols;
    s.vec = true;
    s.vec_dst = dst;
    s.vec_off = off;
    s.part = part ? part : (size_t)(rows * cols);
    s.part_ld = part ? part_ld : s.part;
    slots.push_back(std::move(s));
    return AGPU_OK;
}

int32_t LayeredModel::gemm(const void *a, int lda, const Mat &w, int M, const DenseOut &o) {
    if (f32) return dense_gemm_f32_launch(ctx, (const float *)a, lda, w.w, w.K, M, w.N, w.K, o);
    return dense_gemm_bf16_launch(ctx, (const uint16_t *)a, lda, w.w, w.K, M, w.N, w.K, o);
}

int32_t LayeredModel::save_tap(size_t run, const float *x, int rows) {
    const size_t n = (size_t)rows * dp;
    return agpu_hip(ctx, hipMemcpyAsync(tap + run * n, x, n * 4, hipMemcpyDeviceToDevice, ctx->stream), "hipMemcpyAsync");
}

int32_t LayeredModel::check_ready() {
    for (const Slot &s : slots)
        if (!s.set) return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "%s: tensor '%s' not set", name, s.name.c_str());
    return AGPU_OK;
}

int32_t embed_rows_launch(agpu_ctx *ctx, const uint32_t *tokens, const uint16_t *table, int ld, const float *weight, float *x, float *x0, int rows,
                          int vocab, int d, int dp, float eps) {
    hipLaunchKernelGGL(embed_rows_kernel, dim3((unsigned)rows), dim3(256), 0, ctx->stream, tokens, table, ld, weight, x, x0, vocab, d, dp, eps);
    return AGPU_LAUNCH_CHECK(ctx, "embed_rows_kernel");
}

void layered_release(LayeredModel *m, std::initializer_list<DevBuf *> buffers) {
    if (m->ctx) (void)hipStreamSynchronize(m->ctx->stream);
    for (void *p : m->owned) (void)hipFree(p);
    for (DevBuf *b : buffers)
        if (b->p) (void)hipFree(b->p);
    lm_release(m);
}

int32_t lm_set_tensor(LayeredModel *m, const char *name, const void *data_host, int32_t dtype, int64_t rows, int64_t cols) {
    agpu_ctx *ctx = m->ctx;
    AGPU_REQUIRE_CTX(ctx);
    if (!name || !data_host) return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "%s_set_tensor: null pointer", m->name);
    if (dtype != AGPU_DTYPE_BF16 && dtype != AGPU_DTYPE_F32) return agpu_fail(ctx, AGPU_ERR_UNSUPPORTED, "%s_set_tensor: unknown dtype %d", m->name, dtype);
    Slot *s = nullptr;
    for (Slot &t : m->slots)
        if (t.name == name) s = &t;
    if (!s) return agpu_fail(ctx, AGPU_ERR_KERNEL_NOT_FOUND, "%s_set_tensor: this configuration has no tensor '%s'", m->name, name);
    if (rows != s->rows || cols != s->cols)
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "%s_set_tensor: '%s' is [%lld, %lld], expected [%lld, %lld]", m->name, name, (long long)rows,
                         (long long)cols, (long long)s->rows, (long long)s->cols);
    const size_t n = (size_t)(rows * cols);
    int32_t rc;
    if (s->vec) {
        std::vector<float> v(n);
        if (dtype == AGPU_DTYPE_F32) {
            std::memcpy(v.data(), data_host, n * sizeof(float));
        } else {
            for (size_t i = 0; i < n; ++i) {
                const uint32_t u = (uint32_t)((const uint16_t *)data_host)[i] << 16;
                std::memcpy(&v[i], &u, 4);
            }
        }
        hipError_t e = hipMemcpy2DAsync(*s->vec_dst + s->vec_off, s->part_ld * 4, v.data(), s->part * 4, s->part * 4, n / s->part, hipMemcpyHostToDevice,
                                        ctx->stream);
        if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
        rc = agpu_hip(ctx, e, "hipMemcpy2DAsync(weights)");
    } else if (dtype == AGPU_DTYPE_BF16) {
        rc = s->place((const uint16_t *)data_host);
    } else {
        std::vector<uint16_t> v(n);
        for (size_t i = 0; i < n; ++i) {
            uint32_t u;
            std::memcpy(&u, (const float *)data_host + i, 4);
            v[i] = (u & 0x7fffffffu) > 0x7f800000u ? (uint16_t)((u >> 16) | 0x40u) : (uint16_t)((u + 0x7fffu + ((u >> 16) & 1u)) >> 16);
        }
        rc = s->place(v.data());
    }
    if (rc == AGPU_OK) s->set = true;
    return rc;
}

int32_t lm_tensor_info(const LayeredModel *m, int32_t i, const char **name_out, int64_t *rows_out, int64_t *cols_out, int32_t *is_set_out) {
    if (!name_out || !rows_out || !cols_out || !is_set_out) return AGPU_ERR_NULL_POINTER;
    if (i < 0 || (size_t)i >= m->slots.size()) return AGPU_ERR_DIM_OUT_OF_RANGE;
    const Slot &s = m->slots[(size_t)i];
    *name_out = s.name.c_str();
    *rows_out = s.rows;
    *cols_out = s.cols;
    *is_set_out = s.set ? 1 : 0;
    return AGPU_OK;
}

int32_t lm_layer_streams(LayeredModel *m, const uint32_t *tokens, int32_t new_len, float *streams_out_host) {
    agpu_ctx *ctx = m->ctx;
    AGPU_REQUIRE_CTX(ctx);
    if (!streams_out_host || new_len <= 0) return agpu_fail(ctx, AGPU_ERR_NULL_POINTER, "%s_layer_streams: null pointer or no tokens", m->name);
    const size_t rows = (size_t)m->layer_runs() * (size_t)new_len;
    AGPU_TRY(dev_alloc(ctx, (void **)&m->tap, rows * m->dp * sizeof(float)));
    int32_t rc = lm_forward_cached(m, tokens, 1, new_len, nullptr, 0);
    if (rc == AGPU_OK) {
        hipError_t e = hipMemcpy2DAsync(streams_out_host, (size_t)m->d * 4, m->tap, (size_t)m->dp * 4, (size_t)m->d * 4, rows, hipMemcpyDeviceToHost,
                                        ctx->stream);
        if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
        rc = agpu_hip(ctx, e, "layer_streams");
    }
    (void)hipStreamSynchronize(ctx->stream);
    (void)hipFree(m->tap);
    m->tap = nullptr;
    return rc;
}
