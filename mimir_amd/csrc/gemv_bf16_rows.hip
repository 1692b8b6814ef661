// y = act(x . W^T) for two to eight rows of float32 x and bfloat16 weights, W read once, on the bfloat16 matrix cores: the
// product of a decoding step of several sequences. v_mfma_f32_16x16x32_bf16 multiplies sixteen rows of W by sixteen
// columns; the columns are the rows of x twice, once their bfloat16 value and once what rounding left of them (a float32's
// first sixteen bits of significand), whose results are added at the end: near float32's accuracy for the price of one
// product. The wavefronts of a workgroup (eight, or sixteen for long rows) share its rows of W and cut K into pieces; W goes from memory straight into
// the operand registers (a lane's sixteen bytes of one row), x is converted on the way.
#include "device_util.h"
#include "product_store.h"
#include "stack_ops.h"

#include <type_traits>

namespace mimir {

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

// T: groups of sixteen rows of W a workgroup.
template <int T, int kWaves, Out KIND>
__global__ __launch_bounds__(64 * kWaves) void gemv_bf16_rows_kernel(const uint16_t* __restrict__ W, int64_t ldw, const float* __restrict__ x, int64_t ldx,
                                                                     int M, int N, int K, ProductOut out) {
    __shared__ float red[kWaves][T * 16][17];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int n0 = blockIdx.x * 16 * T;
    const int m = r16 & 7;
    const bool low = r16 >= 8;
    // steps of 32 along K, in pieces of whole pairs (64) a wavefront
    const int pairs = K / 64, per = (pairs + kWaves - 1) / kWaves;
    const int k0 = wave * per * 64, k1 = k0 + per * 64 < K ? k0 + per * 64 : K;
    const float* xp = x + (int64_t)(m < M ? m : M - 1) * ldx + g * 8;
    const uint16_t* wp[T];
#pragma unroll
    for (int t = 0; t < T; t++) wp[t] = W + (int64_t)(n0 + t * 16 + r16 < N ? n0 + t * 16 + r16 : N - 1) * ldw + g * 8;
    f32x4 acc[T];
#pragma unroll
    for (int t = 0; t < T; t++) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    auto sum_of = [&](int from, int to) {
#pragma unroll 2
        for (int k = from; k < to; k += 64) {
            u32x4 w[2][T];
#pragma unroll
            for (int t = 0; t < T; t++)
#pragma unroll
                for (int s = 0; s < 2; s++) w[s][t] = *(const u32x4*)(wp[t] + k + 32 * s);
#pragma unroll
            for (int s = 0; s < 2; s++) {
                const f32x4 a = *(const f32x4*)(xp + k + 32 * s), b = *(const f32x4*)(xp + k + 32 * s + 4);
                float v[8] = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
                u32x4 q;
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    if (low) {
                        v[2 * i] = low_part(v[2 * i]);
                        v[2 * i + 1] = low_part(v[2 * i + 1]);
                    }
                    q[i] = pack_bf16(v[2 * i], v[2 * i + 1]);
                }
#pragma unroll
                for (int t = 0; t < T; t++)
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, w[s][t]), __builtin_bit_cast(bf16x8, q), acc[t], 0, 0, 0);
            }
        }
    };
    int from = k0;
    if (KIND == Out::Scaled && out.mid) {  // what of this wavefront's piece lies below split has a factor of its own
        const int to = out.split < k1 ? (int)out.split : k1;
        sum_of(k0, to);
#pragma unroll
        for (int t = 0; t < T; t++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int n = n0 + t * 16 + 4 * g + i;
                acc[t][i] *= out.mid[n < N ? n : N - 1];
            }
        if (to > from) from = to;
    }
    sum_of(from, k1);
    // a lane holds column r16 of rows 4 g .. 4 g + 3
#pragma unroll
    for (int t = 0; t < T; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) red[wave][t * 16 + 4 * g + i][r16] = acc[t][i];
    __syncthreads();
    for (int o = tid; o < T * 128; o += 64 * kWaves) {
        const int row = o >> 3, col = o & 7, n = n0 + row;
        if (col >= M || n >= N) continue;
        auto sum = [&](int r) {
            float v = 0.f;
#pragma unroll
            for (int i = 0; i < kWaves; i++) v += red[i][r][col] + red[i][r][col + 8];
            return v;
        };
        if (KIND != Out::Pairs || n < out.pair_from) store_column<KIND>(out, col, n, sum(row));
        else if ((row & 1) == 0) store_pair(out, col, n, sum(row), sum(row + 1));
    }
}

}  // namespace

hipError_t gemv_bf16_rows(const uint16_t* W, int64_t ldw, const float* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st) {
    if (M == 0 || N == 0) return hipSuccess;
    if (M > kGemvRows || ldw % 8 || ldx % 4) return hipErrorInvalidValue;
    const int k = (int)((K + 63) / 64 * 64);
    auto launch = [&](auto kernel, int rows, int waves) {
        hipLaunchKernelGGL(kernel, dim3((unsigned)((N + rows - 1) / rows)), dim3(64 * waves), 0, st, W, ldw, x, ldx, (int)M, (int)N, k, out);
    };
    auto by_kind = [&](auto t, auto waves) {
        constexpr int T = decltype(t)::value, kWaves = decltype(waves)::value;
        const Out kind = out_kind(out, N);
        if (kind == Out::Plain) launch(gemv_bf16_rows_kernel<T, kWaves, Out::Plain>, 16 * T, kWaves);
        else if (kind == Out::Pairs) launch(gemv_bf16_rows_kernel<T, kWaves, Out::Pairs>, 16 * T, kWaves);
        else launch(gemv_bf16_rows_kernel<T, kWaves, Out::Scaled>, 16 * T, kWaves);
    };
    using std::integral_constant;
    if (N >= 8192) by_kind(integral_constant<int, 2>{}, integral_constant<int, 8>{});
    else if (k >= 8192) by_kind(integral_constant<int, 1>{}, integral_constant<int, 16>{});
    else by_kind(integral_constant<int, 1>{}, integral_constant<int, 8>{});
    return hipGetLastError();
}

}  // namespace mimir
