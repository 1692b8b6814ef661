// Q4_0 weights by many rows of X on the binary16 matrix cores, for products large enough to pay for a pass over W
// first: the approximate form of the prompt-sized product (weights rounded once to binary16, as qgemm_q4_0.hip's
// template argument HALF does inside its tiles), split into two launches.
//
//   1. panel_prepare_kernel writes W once as a plain binary16 panel P [N, K]: weight (n - 8) d rounded to nearest,
//      the same instruction sequence as the tile kernel's, so the same bits. A weight is converted once here instead
//      of once per 256 rows of X there. The same launch brings X to binary16 (X16, rows scaled by a power of two each,
//      half_rows.h), in workgroups of its own that run beside the panel's.
//   2. hgemm_f16_nt_kernel multiplies X16 [M, K] by P: 256 x 256 tiles of Y, eight wavefronts of 128 x 64 each
//      (gemm_nt_tile.h).
//
// A compute unit holds one workgroup (128 KB of LDS), so a product takes as long as the unit with the most tiles. Where
// 256 x 256 tiles would leave the last round partly empty (2048 x 14336: 448 tiles on 256 units), the right-hand
// columns of Y are cut into tiles of 256 x 192 instead, handed out after the wide ones (32 + 32 column tiles there: one
// wide and one narrow tile a unit); products with too few wide tiles for the device take 128 x 256 tiles. The cut is
// chosen on the host by the time the last tile ends (plan_panel).
//
// Workgroups go round-robin over the eight dies; a die takes a contiguous range of tiles with the tile's row of X
// varying fastest, so the 32 workgroups a die runs together share 4 column panels of P and the 8 row panels of X
// through the die's L2.
//
// Reference semantics: Tensor.MatMulT for a half-precision x and block-quantized w, tensor/quant.go:45-48.
#include "device_util.h"
#include "gemm_nt_tile.h"
#include "half_rows.h"
#include "kernels.h"
#include "tile_plan.h"

namespace mimir {

namespace {

constexpr size_t kLdsBytes = 2 * (size_t)Wide::kStageBytes;

// The pass before the product, one launch: workgroups [0, M) bring a row of X each to binary16 (half_rows.h), the
// others write the panel. Sixteen weights a thread there: the low and the high nibbles of eight bytes of a block, as
// the binary16 values (n - 8) d.
__global__ __launch_bounds__(256) void panel_prepare_kernel(const uint16_t* __restrict__ X, uint16_t* __restrict__ X16, float* __restrict__ scale_back,
                                                            int M, int64_t K, int64_t x_row_stride, const uint8_t* __restrict__ W,
                                                            uint16_t* __restrict__ P, int64_t halves) {
    if ((int)blockIdx.x < M) {
        bf16_row_to_f16_scaled(X, X16, scale_back, K, x_row_stride, blockIdx.x);
        return;
    }
    const int64_t first = (int64_t)((int)blockIdx.x - M) * 256 + threadIdx.x, stride = (int64_t)((int)gridDim.x - M) * 256;
    for (int64_t t = first; t < halves; t += stride) {
        const int q = (int)(t & 1);
        const uint8_t* blk = W + (t >> 1) * 18;
        const uint16_t rd = *(const uint16_t*)blk;  // blocks are 2-byte aligned, no more
        const uint16_t* src = (const uint16_t*)(blk + 2 + 8 * q);
        const uint32_t raw[2] = {(uint32_t)src[0] | (uint32_t)src[1] << 16, (uint32_t)src[2] | (uint32_t)src[3] << 16};
        const _Float16 dh = __builtin_bit_cast(_Float16, rd);
        const f16x2 d2 = {dh, dh}, off = {(_Float16)1032.f, (_Float16)1032.f};
        uint16_t* out = P + (t >> 1) * 32 + 8 * q;  // elements 8 q .. 8 q + 7 (low nibbles) and 16 more on (high nibbles)
#pragma unroll
        for (int half = 0; half < 2; half++) {
            u32x4 v;
#pragma unroll
            for (int i = 0; i < 2; i++) {
                // the nibble into the mantissa of binary16's 1024, minus 1032 is n - 8, times d rounds once
                const uint32_t nib = (raw[i] >> (4 * half)) & 0x0f0f0f0fu;
                const uint32_t p0 = __builtin_amdgcn_perm(0x64646464u, nib, 0x04010400u);
                const uint32_t p1 = __builtin_amdgcn_perm(0x64646464u, nib, 0x04030402u);
                const f16x2 w0 = (__builtin_bit_cast(f16x2, p0) - off) * d2;
                const f16x2 w1 = (__builtin_bit_cast(f16x2, p1) - off) * d2;
                v[2 * i] = __builtin_bit_cast(uint32_t, w0);
                v[2 * i + 1] = __builtin_bit_cast(uint32_t, w1);
            }
            *(u32x4*)(out + 16 * half) = v;
        }
    }
}

// The row's scale undone (a power of two: exact), then one rounding to the output's dtype (f32ToBF16,
// backend/cpu/half.go:42-51).
template <bool OUT_F32>
struct ScaledStore {
    void* Yv;
    const float* row_scale;
    bool wide_ok;
    __device__ __forceinline__ int first_steps(int steps) const { return steps; }
    __device__ __forceinline__ float mid(int, int) const { return 1.f; }
    __device__ __forceinline__ float row(int m, int M) const { return m < M ? row_scale[m] : 0.f; }
    __device__ __forceinline__ void operator()(int m, int n, int N, float back, float v[4]) const {
#pragma unroll
        for (int k = 0; k < 4; k++) v[k] = v[k] * back;
        if (wide_ok && n + 3 < N) {
            if (OUT_F32) {
                const f32x4 o = {v[0], v[1], v[2], v[3]};
                *(f32x4*)((float*)Yv + (int64_t)m * N + n) = o;
            } else {
                const u32x2 o = {(uint32_t)f32_to_bf16_bits(v[0]) | (uint32_t)f32_to_bf16_bits(v[1]) << 16,
                                 (uint32_t)f32_to_bf16_bits(v[2]) | (uint32_t)f32_to_bf16_bits(v[3]) << 16};
                *(u32x2*)((uint16_t*)Yv + (int64_t)m * N + n) = o;
            }
        } else {
#pragma unroll
            for (int k = 0; k < 4; k++) {
                if (n + k >= N) continue;
                if (OUT_F32) ((float*)Yv)[(int64_t)m * N + n + k] = v[k];
                else ((uint16_t*)Yv)[(int64_t)m * N + n + k] = f32_to_bf16_bits(v[k]);
            }
        }
    }
};

template <bool OUT_F32>
__global__ __launch_bounds__(512, 2) void hgemm_f16_nt_kernel(const uint16_t* __restrict__ X16, const uint16_t* __restrict__ P, void* __restrict__ Yv,
                                                              const float* __restrict__ row_scale, int M, int N, int K, PanelPlan plan) {
    extern __shared__ __align__(1024) char lds_gemm[];
    const ScaledStore<OUT_F32> store{Yv, row_scale, (N & 3) == 0 && ((uintptr_t)Yv & 15) == 0};
    int b = (int)blockIdx.x;
    if (plan.low) {
        const int ntiles = plan.tiles_m * plan.wide_cols;
        const int t = tile_of(b, ntiles);
        if (t >= ntiles) return;  // the whole workgroup
        tile_body<Low, F16Element>(X16, K, P, K, store, M, N, K, (t % plan.tiles_m) * Low::BM, (t / plan.tiles_m) * Low::BN, lds_gemm);
        return;
    }
    const int nwide = plan.tiles_m * plan.wide_cols;
    const int wide_wgs = ((nwide + 7) >> 3) << 3;
    if (b < wide_wgs) {
        const int t = tile_of(b, nwide);
        if (t >= nwide) return;
        tile_body<Wide, F16Element>(X16, K, P, K, store, M, N, K, (t % plan.tiles_m) * Wide::BM, (t / plan.tiles_m) * Wide::BN, lds_gemm);
        return;
    }
    b -= wide_wgs;
    const int nnarrow = plan.tiles_m * plan.narrow_cols;
    const int t = tile_of(b, nnarrow);
    if (t >= nnarrow) return;
    tile_body<Narrow, F16Element>(X16, K, P, K, store, M, N, K, (t % plan.tiles_m) * Narrow::BM, plan.wide_cols * Wide::BN + (t / plan.tiles_m) * Narrow::BN,
                               lds_gemm);
}

// Costs in Wide tiles' time: a Narrow tile has three quarters of the MFMAs and reads a little more from LDS for each,
// a Low tile half of them and a third more.
constexpr double kNarrowCost = 0.78, kLowCost = 0.56;

}  // namespace

size_t qgemm_f16_panel_bytes(int64_t N, int64_t K) { return ((size_t)N * K * 2 + 255) & ~(size_t)255; }

// Whether the two launches beat the one whose tiles convert W for themselves: the panel costs a pass over W
// (N K (0.5625 + 2) bytes), which at least 1024 rows of X repay when the tiles keep 70 % of the device busy
// until the last one ends (at 512 x 14336 x 4096 the two routes measured the same, 544 and 551 TFLOP/s).
bool qgemm_f16_panel_pays(int64_t M, int64_t N, int64_t K) {
    if (!(M >= 1024 && K % kStep == 0 && K >= kStep && M < (1 << 24) && N < (1 << 24) && K < (1 << 24) && N > 0)) return false;
    PanelPlan plan;
    const double end = plan_panel(M, N, kNarrowCost, kLowCost, &plan);
    const double work = (double)M * (double)N / (256.0 * 256.0);
    return work >= 0.70 * kUnits * end;
}

hipError_t qgemm_f16_panel(const void* W, const void* X, int64_t x_row_stride, void* X16, float* row_scale, void* Y, int64_t M, int64_t N, int64_t K,
                           bool out_f32, void* panel, hipStream_t st) {
    {
        static std::atomic<bool> raised{false};  // threads may race here: both then set the same attribute
        if (!raised) {
            hipError_t e = hipFuncSetAttribute((const void*)hgemm_f16_nt_kernel<true>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLdsBytes);
            if (e == hipSuccess) e = hipFuncSetAttribute((const void*)hgemm_f16_nt_kernel<false>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLdsBytes);
            if (e != hipSuccess) return e;
            raised = true;
        }
    }
    const int64_t halves = N * K / 16;
    const int64_t want = (halves + 255) / 256;
    hipLaunchKernelGGL(panel_prepare_kernel, dim3((unsigned)(M + (want > 8192 ? 8192 : want))), dim3(256), 0, st, (const uint16_t*)X, (uint16_t*)X16, row_scale,
                       (int)M, K, x_row_stride, (const uint8_t*)W, (uint16_t*)panel, halves);
    PanelPlan plan;
    plan_panel(M, N, kNarrowCost, kLowCost, &plan);
    const int first = plan.tiles_m * plan.wide_cols, then = plan.tiles_m * plan.narrow_cols;
    note_kernel("hgemm_f16_nt_kernel: %d x %d tiles of %s, %d x %d tiles of 256 x 192", plan.tiles_m, plan.wide_cols, plan.low ? "128 x 256" : "256 x 256",
                plan.tiles_m, plan.narrow_cols);
    const dim3 grid((unsigned)(((first + 7) / 8) * 8 + ((then + 7) / 8) * 8));
    if (out_f32)
        hipLaunchKernelGGL(hgemm_f16_nt_kernel<true>, grid, dim3(512), kLdsBytes, st, (const uint16_t*)X16, (const uint16_t*)panel, Y, row_scale, (int)M,
                           (int)N, (int)K, plan);
    else
        hipLaunchKernelGGL(hgemm_f16_nt_kernel<false>, grid, dim3(512), kLdsBytes, st, (const uint16_t*)X16, (const uint16_t*)panel, Y, row_scale, (int)M,
                           (int)N, (int)K, plan);
    return hipGetLastError();
}

}  // namespace mimir
