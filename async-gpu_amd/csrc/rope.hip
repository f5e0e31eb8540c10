// Rotation tables (rope.h).
#include "rope.h"

#include <algorithm>
#include <cmath>

namespace {

__global__ void rope_table_kernel(float2 *table, int positions, int half, double base, double factor, double lo, double width, double grow) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= (size_t)positions * half) return;
    const int p = (int)(i / half), j = (int)(i % half);
    double f = pow(base, -(double)j / (double)half);
    if (factor > 0.0) {
        const double ramp = fmin(fmax(((double)j - lo) / width, 0.0), 1.0);
        f = f / factor * ramp + f * (1.0 - ramp);
    }
    const double a = (double)p * f;
    table[i] = make_float2((float)(cos(a) * grow), (float)(sin(a) * grow));
}

}  // namespace

int32_t rope_table_launch(agpu_ctx *ctx, float2 *table, int positions, const RopeSpec &s) {
    const int half = s.dims / 2;
    if (half == 0) return AGPU_OK;
    double lo = 0.0, width = 1.0, grow = 1.0;
    if (s.factor > 0.0) {
        // the pair that turns `turns` times over the original context
        auto pair = [&](double turns) { return s.dims * std::log(s.original / (2.0 * M_PI * turns)) / (2.0 * std::log(s.base)); };
        lo = std::max(std::floor(pair(s.fast)), 0.0);
        const double hi = std::min(std::ceil(pair(s.slow)), (double)(s.dims - 1));
        width = std::max(hi - lo, 0.001);
        grow = 0.1 * std::log(s.factor) + 1.0;
    }
    hipLaunchKernelGGL(rope_table_kernel, dim3((unsigned)(((size_t)positions * half + 255) / 256)), dim3(256), 0, ctx->stream, table, positions, half, s.base,
                       s.factor, lo, width, grow);
    return AGPU_LAUNCH_CHECK(ctx, "rope_table_kernel");
}
