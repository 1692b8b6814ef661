// y = x . W^T for a float32, binary16 or bfloat16 W [N, K] and few rows of
// x: the product a Linear takes when its weight is not block-quantized
// (tensor/quant.go:40-42 -> product, tensor/movement.go:232-243: half operands
// are widened to float32 and multiplied there). Tiny Llama fixtures keep some
// projections in these types; the decode path of a quantized model does not
// come here. One wavefront per row of W.
//
// gemv_bf16 is the product of a decoding step whose weights are bfloat16 (the mixer stack's): a wavefront takes a few
// rows of W for up to eight rows of x, sixteen bytes of W a lane at a time, and applies the activation behind it.
#include "device_util.h"
#include "kernels.h"
#include "product_store.h"
#include "stack_ops.h"

#include <type_traits>

namespace mimir {

template <typename T>
__device__ __forceinline__ float widen(T v);
template <>
__device__ __forceinline__ float widen<float>(float v) { return v; }
struct half_bits { uint16_t v; };
struct bf16_bits { uint16_t v; };
template <>
__device__ __forceinline__ float widen<half_bits>(half_bits v) { return f16_bits_to_f32(v.v); }
template <>
__device__ __forceinline__ float widen<bf16_bits>(bf16_bits v) { return bf16_bits_to_f32(v.v); }

template <typename T>
__global__ __launch_bounds__(256) void gemv_float_kernel(const T* __restrict__ W, const float* __restrict__ x, float* __restrict__ y,
                                                         int N, int K, int64_t x_row_stride) {
    const int lane = threadIdx.x & 63, row = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
    if (row >= N) return;
    const T* w = W + (int64_t)row * K;
    const float* xr = x + (int64_t)blockIdx.y * x_row_stride;
    float acc = 0.f;
    for (int k = lane; k < K; k += 64) acc = fmaf(xr[k], widen<T>(w[k]), acc);
    acc = wave_sum(acc);
    if (lane == 0) y[(int64_t)blockIdx.y * N + row] = acc;
}

hipError_t gemv_float(int dt, const void* W, const float* x, float* y, int64_t M, int64_t N, int64_t K, int64_t x_row_stride,
                      hipStream_t st) {
    if (M == 0 || N == 0) return hipSuccess;
    dim3 grid((unsigned)((N + 3) / 4), (unsigned)M);
    if (dt == kF32)
        hipLaunchKernelGGL(gemv_float_kernel<float>, grid, dim3(256), 0, st, (const float*)W, x, y, (int)N, (int)K, x_row_stride);
    else if (dt == kF16)
        hipLaunchKernelGGL(gemv_float_kernel<half_bits>, grid, dim3(256), 0, st, (const half_bits*)W, x, y, (int)N, (int)K, x_row_stride);
    else
        hipLaunchKernelGGL(gemv_float_kernel<bf16_bits>, grid, dim3(256), 0, st, (const bf16_bits*)W, x, y, (int)N, (int)K, x_row_stride);
    return hipGetLastError();
}

// M rows of x against R rows of W a wavefront, eight elements of K a lane and step (the rows are padded with zeros to
// a multiple of 64). The x of a step serves all R rows from registers.
template <int M, int R, Out KIND>
__global__ __launch_bounds__(256) void gemv_bf16_kernel(const uint16_t* __restrict__ W, int64_t ldw, const float* __restrict__ x, int64_t ldx, int N, int K,
                                                        ProductOut out) {
    const int lane = threadIdx.x & 63, n0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * R;
    if (n0 >= N) return;
    const int64_t m0 = (int64_t)blockIdx.y * M;
    const uint16_t* w[R];
#pragma unroll
    for (int r = 0; r < R; r++) w[r] = W + (int64_t)(n0 + r < N ? n0 + r : N - 1) * ldw;
    float acc[M][R];
#pragma unroll
    for (int m = 0; m < M; m++)
#pragma unroll
        for (int r = 0; r < R; r++) acc[m][r] = 0.f;
    auto sum = [&](int from, int to) {
#pragma unroll 4
        for (int k = from + lane * 8; k < to; k += 512) {
            u32x4 wv[R];
#pragma unroll
            for (int r = 0; r < R; r++) wv[r] = *(const u32x4*)(w[r] + k);
#pragma unroll
            for (int m = 0; m < M; m++) {
                const f32x4* xp = (const f32x4*)(x + (m0 + m) * ldx + k);
                const f32x4 a = xp[0], b = xp[1];
#pragma unroll
                for (int r = 0; r < R; r++) {
                    float t = acc[m][r];
#pragma unroll
                    for (int i = 0; i < 4; i++) {
                        const float x0 = i < 2 ? a[2 * i] : b[2 * i - 4], x1 = i < 2 ? a[2 * i + 1] : b[2 * i - 3];
                        t = fmaf(x0, __uint_as_float(wv[r][i] << 16), t);
                        t = fmaf(x1, __uint_as_float(wv[r][i] & 0xffff0000u), t);
                    }
                    acc[m][r] = t;
                }
            }
        }
    };
    const int split = KIND == Out::Scaled && out.mid ? (int)out.split : 0;
    if constexpr (KIND == Out::Scaled) {  // the sums below split and from there on have factors of their own
        sum(0, split);
#pragma unroll
        for (int r = 0; r < R; r++) {
            const float f = out.mid ? out.mid[n0 + r < N ? n0 + r : N - 1] : 1.f;
#pragma unroll
            for (int m = 0; m < M; m++) acc[m][r] *= f;
        }
    }
    sum(split, K);
#pragma unroll
    for (int m = 0; m < M; m++) {
        float v[R];
#pragma unroll
        for (int r = 0; r < R; r++) v[r] = wave_sum(acc[m][r]);
        if (lane != 0) continue;
#pragma unroll
        for (int r = 0; r < R; r++) {
            const int n = n0 + r;
            if (n >= N) break;
            if (KIND != Out::Pairs || n < out.pair_from) store_column<KIND>(out, m0 + m, n, v[r]);
            else if (r + 1 < R && (r & 1) == 0) store_pair(out, m0 + m, n, v[r], v[r + 1 < R ? r + 1 : r]);
        }
    }
}

namespace {

template <int M>
void launch_gemv_bf16(const uint16_t* W, int64_t ldw, const float* x, int64_t ldx, int64_t groups, int64_t N, int64_t K, const ProductOut& out, hipStream_t st) {
    const int k = (int)((K + 63) / 64 * 64);
    auto launch = [&](auto kernel, int rows) {
        hipLaunchKernelGGL(kernel, dim3((unsigned)((N + 4 * rows - 1) / (4 * rows)), (unsigned)groups), dim3(256), 0, st, W, ldw, x, ldx, (int)N, k, out);
    };
    // more rows a wavefront read x less often; fewer give a small matrix enough wavefronts
    const Out kind = out_kind(out, N);
    const int rows = N >= 8192 && M <= 4 ? 4 : N >= 2048 || kind == Out::Pairs ? 2 : 1;
    auto by_kind = [&](auto rows_tag) {
        constexpr int R = decltype(rows_tag)::value;
        if (kind == Out::Scaled) launch(gemv_bf16_kernel<M, R, Out::Scaled>, R);
        else if (kind == Out::Plain) launch(gemv_bf16_kernel<M, R, Out::Plain>, R);
        else if constexpr (R > 1) launch(gemv_bf16_kernel<M, R, Out::Pairs>, R);
    };
    if (rows == 4) by_kind(std::integral_constant<int, (M <= 4 ? 4 : 2)>{});
    else if (rows == 2) by_kind(std::integral_constant<int, 2>{});
    else by_kind(std::integral_constant<int, 1>{});
}

}  // namespace

hipError_t gemv_bf16(const uint16_t* W, int64_t ldw, const float* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st) {
    int64_t m = 0;
    auto rest = [&](int64_t rows, int64_t each) {  // whole groups of `each` rows from row m on
        ProductOut o = out;
        if (o.f32) o.f32 += m * o.ld;
        else if (o.bf16) o.bf16 += m * o.ld;
        if (o.pair_f32) o.pair_f32 += m * o.pair_ld;
        else if (o.pair_bf16) o.pair_bf16 += m * o.pair_ld;
        const float* xr = x + m * ldx;
        const int64_t groups = rows / each;
        if (each == 8) launch_gemv_bf16<8>(W, ldw, xr, ldx, groups, N, K, o, st);
        else if (each == 4) launch_gemv_bf16<4>(W, ldw, xr, ldx, groups, N, K, o, st);
        else if (each == 2) launch_gemv_bf16<2>(W, ldw, xr, ldx, groups, N, K, o, st);
        else launch_gemv_bf16<1>(W, ldw, xr, ldx, groups, N, K, o, st);
        m += groups * each;
    };
    for (int64_t each = 8; each >= 1; each >>= 1)
        if (M - m >= each) rest(M - m, each);
    return hipGetLastError();
}

}  // namespace mimir
