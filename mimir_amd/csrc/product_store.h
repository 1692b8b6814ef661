// How a product's result leaves the accumulators (ProductOut, stack_ops.h), one column or pair of columns at a time.
#pragma once
#include "device_util.h"
#include "stack_ops.h"

namespace mimir {

// A column that is not one of a pair, with the factor and the activation applied.
__device__ __forceinline__ void store_column(const ProductOut& out, int64_t m, int64_t n, float v) {
    if (out.scale) v *= out.scale[n];
    if (out.relu2) v = v > 0.f ? v * v : 0.f;
    else if (n < out.silu_n) v = v / (1.f + expf(-v));
    const int64_t at = m * out.ld + n;
    if (out.bf16) out.bf16[at] = round_bf16(v);
    else out.f32[at] = out.add ? out.f32[at] + v : v;
}

// Columns n and n + 1, a pair.
__device__ __forceinline__ void store_pair(const ProductOut& out, int64_t m, int64_t n, float z, float u) {
    const float v = z / (1.f + expf(-z)) * u;
    const int64_t at = m * out.pair_ld + ((n - out.pair_from) >> 1);
    if (out.pair_bf16) out.pair_bf16[at] = round_bf16(v);
    else out.pair_f32[at] = v;
}

}  // namespace mimir
