// What the models with bf16 weights share beneath their layers: named weight slots that know how a tensor of the file reaches
// the device, owned memory, the residual stream's sizes, the taps behind every layer run.  A model derives from
// LayeredModel, fills `slots` when it is created, and supplies its layers.
//
// Storage: matrices are bf16 [N, K] with N and K padded to multiples of 32 by zeros (heads and blocks each on their own,
// where a kernel wants them aligned); activation rows have padded strides whose padding is zero, so no kernel needs to know
// the true sizes except the norms.
#pragma once
#include <functional>
#include <string>
#include <vector>

#include "dense_linear.h"
#include "lm_runtime.h"

inline int pad32(int n) { return (n + 31) / 32 * 32; }

#define AGPU_TRY(expr)                    \
    do {                                  \
        const int32_t rc_ = (expr);       \
        if (rc_ != AGPU_OK) return rc_;   \
    } while (0)

struct Mat {
    uint16_t *w = nullptr;
    int N = 0, K = 0;
};

// A named weight: its shape in the file and how its values reach the device.
struct Slot {
    std::string name;
    int64_t rows = 0, cols = 0;
    bool vec = false, set = false;
    float **vec_dst = nullptr;       // vectors: fp32, from vec_off on, in parts of `part` values `part_ld` apart
    size_t vec_off = 0, part = 0, part_ld = 0;
    std::function<int32_t(const uint16_t *)> place;  // matrices: bf16 rows
};

struct LayeredModel : LmRuntime {
    explicit LayeredModel(const char *model_name) : LmRuntime(model_name) {}
    int32_t check_ready() override;
    int logits_stride() const override { return pad32(V); }
    virtual int layer_runs() const = 0;

    int d = 0, dp = 0;  // width of the residual stream, padded
    bool f32 = false;   // activations, products and cache in fp32
    std::vector<Slot> slots;
    std::vector<void *> owned;  // weights, cache, state, tables
    int64_t weight_bytes = 0, cache_bytes = 0;
    float *tap = nullptr;  // residual stream after every layer run, [runs][rows][dp] (lm_layer_streams)

    // zeroed memory that lives as long as the model; *count (optional) grows by its size
    int32_t own(void **p, size_t bytes, int64_t *count);
    int32_t new_mat(Mat &t, int N, int K);
    void add_mat(const std::string &name, int64_t rows, int64_t cols, std::function<int32_t(const uint16_t *)> place);
    // A matrix that fills rows row0, row0 + row_step, ... of t from column col0 on.
    void add_rows(const std::string &name, Mat t, int row0, int col0, int64_t rows, int64_t cols, int row_step = 1);
    // heads x `per` rows from row0 on, every head moved to a stride of `per_p` rows.
    void add_head_rows(const std::string &name, Mat t, int heads, int per, int per_p, int64_t cols, int row0 = 0);
    // heads x `per` columns, every head moved to a stride of `per_p` columns.
    void add_head_cols(const std::string &name, Mat t, int heads, int per, int per_p, int64_t rows);
    // A vector (or table) of rows x cols values at `off` of *dst, which is allocated with `alloc` floats if it is still null;
    // parts of `part` values are moved to a stride of `part_ld` (0: no parts).
    int32_t add_vec(const std::string &name, float **dst, int64_t rows, int64_t cols, size_t alloc = 0, size_t off = 0, size_t part = 0,
                    size_t part_ld = 0);
    // A Linear on rows that a matrix-core kernel reads: `a` is bf16 or fp32 as the model computes.
    int32_t gemm(const void *a, int lda, const Mat &w, int M, const DenseOut &o);
    int32_t save_tap(size_t run, const float *x, int rows);
};

int32_t place_rows(agpu_ctx *ctx, const Mat &t, int row0, int row_step, int col0, const uint16_t *src, int64_t rows, int64_t cols, int64_t src_ld);
// x (and x0, if not null) = rows of the table [vocab][ld], RMS-normed with 1 + weight where weight is given.
int32_t embed_rows_launch(agpu_ctx *ctx, const uint32_t *tokens, const uint16_t *table, int ld, const float *weight, float *x, float *x0, int rows,
                          int vocab, int d, int dp, float eps);
// Frees the model's memory, the listed buffers and the runtime's.
void layered_release(LayeredModel *m, std::initializer_list<DevBuf *> buffers);

// ---- bodies of the models' entry points ----
int32_t lm_set_tensor(LayeredModel *m, const char *name, const void *data_host, int32_t dtype, int64_t rows, int64_t cols);
int32_t lm_tensor_info(const LayeredModel *m, int32_t i, const char **name_out, int64_t *rows_out, int64_t *cols_out, int32_t *is_set_out);
int32_t lm_layer_streams(LayeredModel *m, const uint32_t *tokens, int32_t new_len, float *streams_out_host);
