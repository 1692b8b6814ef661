// y = act(x . W^T) for many rows of bfloat16 x and bfloat16 weights on the bfloat16 matrix cores, float32 sums: the
// prompt product of a model whose weights are bfloat16. The tiles are those of gemm_nt_tile.h, cut as tile_plan.h
// chooses; products with too few tiles of 128 x 256 for the device take tiles of 64 x 128. The activation and the
// rounding to the output's dtype happen as the tile is stored.
#include "gemm_nt_tile.h"
#include "kernels.h"
#include "product_store.h"
#include "stack_ops.h"
#include "tile_plan.h"

namespace mimir {

namespace {

constexpr size_t kLdsBytes = 2 * (size_t)Wide::kStageBytes;

// Costs in Wide tiles' time (qgemm_f16_panel.hip), a Tiny tile's share of the MFMAs with as many more reads from LDS.
constexpr double kNarrowCost = 0.78, kLowCost = 0.56, kTinyCost = 0.19;

template <Out KIND>
struct ActStore {
    ProductOut out;
    bool wide_ok;
    static constexpr bool kTwo = KIND == Out::Scaled;  // the sums over the first out.split of K may have factors of their own
    __device__ __forceinline__ int first_steps(int steps) const { return kTwo && out.mid ? (int)out.split / kStep : steps; }
    __device__ __forceinline__ float mid(int n, int N) const { return kTwo ? out.mid[n < N ? n : N - 1] : 1.f; }
    __device__ __forceinline__ float row(int, int) const { return 0.f; }
    __device__ __forceinline__ void operator()(int m, int n, int N, float, float v[4]) const {
        if (KIND == Out::Pairs && n >= out.pair_from) {  // whole pairs: N is even
            float p[2];
#pragma unroll
            for (int k = 0; k < 2; k++) p[k] = v[2 * k] / (1.f + __expf(-v[2 * k])) * v[2 * k + 1];
            const int64_t at = m * out.pair_ld + ((n - out.pair_from) >> 1);
            const bool both = n + 2 < N;
            if (out.pair_bf16) {
                if (both && out.pair_ld % 2 == 0 && ((uintptr_t)out.pair_bf16 & 3) == 0) {
                    *(uint32_t*)(out.pair_bf16 + at) = pack_bf16(p[0], p[1]);
                } else {
                    out.pair_bf16[at] = round_bf16(p[0]);
                    if (both) out.pair_bf16[at + 1] = round_bf16(p[1]);
                }
            } else {
                out.pair_f32[at] = p[0];
                if (both) out.pair_f32[at + 1] = p[1];
            }
            return;
        }
        if constexpr (KIND == Out::Scaled) {
            if (out.scale) {
#pragma unroll
                for (int k = 0; k < 4; k++) v[k] *= out.scale[n + k < N ? n + k : N - 1];
            }
        } else if (out.relu2) {
#pragma unroll
            for (int k = 0; k < 4; k++) v[k] = v[k] > 0.f ? v[k] * v[k] : 0.f;
        } else if (n < out.silu_n) {
#pragma unroll
            for (int k = 0; k < 4; k++)
                if (n + k < out.silu_n) v[k] = v[k] / (1.f + __expf(-v[k]));
        }
        const int64_t at = m * out.ld + n;
        if (wide_ok && n + 3 < N) {
            if (out.f32) {
                f32x4 o = {v[0], v[1], v[2], v[3]};
                if (KIND == Out::Scaled && out.add) o = o + *(const f32x4*)(out.f32 + at);
                *(f32x4*)(out.f32 + at) = o;
            } else {
                const u32x2 o = {pack_bf16(v[0], v[1]),
                                 pack_bf16(v[2], v[3])};
                *(u32x2*)(out.bf16 + at) = o;
            }
            return;
        }
#pragma unroll
        for (int k = 0; k < 4; k++) {
            if (n + k >= N) continue;
            if (out.f32) out.f32[at + k] = KIND == Out::Scaled && out.add ? out.f32[at + k] + v[k] : v[k];
            else out.bf16[at + k] = round_bf16(v[k]);
        }
    }
};

template <class T, class S>
__device__ __forceinline__ void one_tile(const uint16_t* X, int64_t ldx, const uint16_t* W, int64_t ldw, const S& store, int M, int N, int K, int b,
                                         int tiles_m, int tiles_n, int col0, char* lds) {
    const int t = tile_of(b, tiles_m * tiles_n);
    if (t >= tiles_m * tiles_n) return;  // the whole workgroup
    tile_body<T, Bf16Element>(X, ldx, W, ldw, store, M, N, K, (t % tiles_m) * T::BM, col0 + (t / tiles_m) * T::BN, lds);
}

template <class S>
__global__ __launch_bounds__(512, 2) void gemm_bf16_kernel(const uint16_t* __restrict__ X, int64_t ldx, const uint16_t* __restrict__ W, int64_t ldw, S store,
                                                           int M, int N, int K, PanelPlan plan) {
    extern __shared__ __align__(1024) char lds_gemm[];
    int b = (int)blockIdx.x;
    if (plan.low) {
        one_tile<Low>(X, ldx, W, ldw, store, M, N, K, b, plan.tiles_m, plan.wide_cols, 0, lds_gemm);
        return;
    }
    const int wide_wgs = ((plan.tiles_m * plan.wide_cols + 7) >> 3) << 3;
    if (b < wide_wgs) one_tile<Wide>(X, ldx, W, ldw, store, M, N, K, b, plan.tiles_m, plan.wide_cols, 0, lds_gemm);
    else one_tile<Narrow>(X, ldx, W, ldw, store, M, N, K, b - wide_wgs, plan.tiles_m, plan.narrow_cols, plan.wide_cols * Wide::BN, lds_gemm);
}

// Two workgroups a compute unit: 48 KB of LDS and few registers each.
template <class S>
__global__ __launch_bounds__(512, 4) void gemm_bf16_tiny_kernel(const uint16_t* __restrict__ X, int64_t ldx, const uint16_t* __restrict__ W, int64_t ldw,
                                                                S store, int M, int N, int K, int tiles_m, int tiles_n) {
    extern __shared__ __align__(1024) char lds_gemm[];
    one_tile<Tiny>(X, ldx, W, ldw, store, M, N, K, (int)blockIdx.x, tiles_m, tiles_n, 0, lds_gemm);
}

unsigned die_grid(int tiles) { return (unsigned)((tiles + 7) / 8 * 8); }

template <Out KIND>
hipError_t launch(const uint16_t* W, int64_t ldw, const uint16_t* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st) {
    {
        static std::atomic<bool> raised{false};  // threads may race here: both then set the same attribute
        if (!raised) {
            hipError_t e = hipFuncSetAttribute((const void*)gemm_bf16_kernel<ActStore<KIND>>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLdsBytes);
            if (e != hipSuccess) return e;
            raised = true;
        }
    }
    const int k = (int)((K + 63) / 64 * 64);
    const void* y = out.f32 ? (const void*)out.f32 : (const void*)out.bf16;
    const ActStore<KIND> store{out, out.ld % 4 == 0 && ((uintptr_t)y & 15) == 0};
    PanelPlan plan;
    const double end = plan_panel(M, N, kNarrowCost, kLowCost, &plan);
    const int tm = (int)((M + Tiny::BM - 1) / Tiny::BM), tn = (int)((N + Tiny::BN - 1) / Tiny::BN);
    if (makespan(tm * tn, kTinyCost, 0, 0.0) < end - 1e-9) {
        hipLaunchKernelGGL(gemm_bf16_tiny_kernel<ActStore<KIND>>, dim3(die_grid(tm * tn)), dim3(512), 2 * (size_t)Tiny::kStageBytes, st, x, ldx, W, ldw, store, (int)M,
                           (int)N, k, tm, tn);
        return hipGetLastError();
    }
    const int first = plan.tiles_m * plan.wide_cols, then = plan.tiles_m * plan.narrow_cols;
    hipLaunchKernelGGL(gemm_bf16_kernel<ActStore<KIND>>, dim3(die_grid(first) + die_grid(then)), dim3(512), kLdsBytes, st, x, ldx, W, ldw, store, (int)M, (int)N, k,
                       plan);
    return hipGetLastError();
}

}  // namespace

hipError_t gemm_bf16(const uint16_t* W, int64_t ldw, const uint16_t* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st) {
    if (M == 0 || N == 0) return hipSuccess;
    if (M >= 1 << 24 || N >= 1 << 24 || K >= 1 << 24 || ldx % 8 || ldw % 8 || (out.mid && (out.split <= 0 || out.split >= K || out.split % kStep))) return hipErrorInvalidValue;
    const Out kind = out_kind(out, N);
    if (kind == Out::Plain) return launch<Out::Plain>(W, ldw, x, ldx, M, N, K, out, st);
    return kind == Out::Pairs ? launch<Out::Pairs>(W, ldw, x, ldx, M, N, K, out, st) : launch<Out::Scaled>(W, ldw, x, ldx, M, N, K, out, st);
}

}  // namespace mimir
