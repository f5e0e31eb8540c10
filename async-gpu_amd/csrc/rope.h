// Rotation tables: cos and sin of every position's angle per pair of dimensions, computed in double precision and rounded once.
#pragma once
#include "agpu_internal.h"

struct RopeSpec {
    int dims = 0;  // dimensions that turn; pair i turns by position * base^(-2 i / dims)
    double base = 10000.0;
    // Stretched contexts (YaRN): with factor > 0 pairs that turn less than `slow` times over `original` positions go `factor` times
    // slower, pairs that turn more than `fast` times stay, a linear ramp over the pair index lies between; cos and sin grow by
    // 0.1 ln(factor) + 1.
    double factor = 0.0, original = 0.0, fast = 0.0, slow = 0.0;
    bool operator==(const RopeSpec &o) const {
        return dims == o.dims && base == o.base && factor == o.factor && original == o.original && fast == o.fast && slow == o.slow;
    }
};

// [positions][dims / 2]: cos, sin
int32_t rope_table_launch(agpu_ctx *ctx, float2 *table, int positions, const RopeSpec &spec);
