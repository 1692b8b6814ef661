// How a product's result leaves the accumulators (ProductOut, stack_ops.h), one column or pair of columns at a time. What a
// product does not ask for is not in its kernel.
#pragma once
#include "device_util.h"
#include "stack_ops.h"

namespace mimir {

enum class Out { Plain, Pairs, Scaled };  // an activation; and columns in pairs; or factors and what is there already
inline Out out_kind(const ProductOut& o, int64_t N) { return o.pair_from < N ? Out::Pairs : o.scale || o.mid || o.add ? Out::Scaled : Out::Plain; }

// A column that is not one of a pair.
template <Out KIND>
__device__ __forceinline__ void store_column(const ProductOut& out, int64_t m, int64_t n, float v) {
    const int64_t at = m * out.ld + n;
    if constexpr (KIND == Out::Scaled) {
        if (out.scale) v *= out.scale[n];
        if (out.add) v += out.f32[at];
    } else {
        if (out.relu2) v = v > 0.f ? v * v : 0.f;
        else if (n < out.silu_n) v = v / (1.f + expf(-v));
    }
    if (out.f32) out.f32[at] = v;
    else out.bf16[at] = round_bf16(v);
}

// Columns n and n + 1, a pair.
__device__ __forceinline__ void store_pair(const ProductOut& out, int64_t m, int64_t n, float z, float u) {
    const float v = z / (1.f + expf(-z)) * u;
    const int64_t at = m * out.pair_ld + ((n - out.pair_from) >> 1);
    if (out.pair_bf16) out.pair_bf16[at] = round_bf16(v);
    else out.pair_f32[at] = v;
}

}  // namespace mimir
