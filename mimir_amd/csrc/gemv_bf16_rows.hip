// y = act(x . W^T) for two to eight rows of float32 x and bfloat16 weights, W read once, on the bfloat16 matrix cores: the
// product of a decoding step of several sequences. v_mfma_f32_16x16x32_bf16 multiplies sixteen rows of W by sixteen
// columns; the columns are the rows of x twice, once their bfloat16 value and once what rounding left of them (a float32's
// first sixteen bits of significand), whose results are added at the end: near float32's accuracy for the price of one
// product. The wavefronts of a workgroup (eight, or sixteen for long rows) share its rows of W and cut K into pieces; W goes from memory straight into
// the operand registers (a lane's sixteen bytes of one row), x is converted on the way.
#include "device_util.h"
#include "stack_ops.h"

namespace mimir {

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

// T: groups of sixteen rows of W a workgroup.
template <int T, int kWaves>
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
#pragma unroll 2
    for (int k = k0; k < k1; k += 64) {
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
    // a lane holds column r16 of rows 4 g .. 4 g + 3
#pragma unroll
    for (int t = 0; t < T; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) red[wave][t * 16 + 4 * g + i][r16] = acc[t][i];
    __syncthreads();
    for (int o = tid; o < T * 128; o += 64 * kWaves) {
        const int row = o >> 3, col = o & 7, n = n0 + row;
        if (col >= M || n >= N) continue;
        float v = 0.f;
#pragma unroll
        for (int i = 0; i < kWaves; i++) v += red[i][row][col] + red[i][row][col + 8];
        if (out.relu2) v = v > 0.f ? v * v : 0.f;
        else if (n < out.silu_n) v = v / (1.f + expf(-v));
        const int64_t at = (int64_t)col * out.ld + n;
        if (out.f32) out.f32[at] = v;
        else out.bf16[at] = round_bf16(v);
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
    if (N >= 8192) launch(gemv_bf16_rows_kernel<2, 8>, 32, 8);
    else if (k >= 8192) launch(gemv_bf16_rows_kernel<1, 16>, 16, 16);
    else launch(gemv_bf16_rows_kernel<1, 8>, 16, 8);
    return hipGetLastError();
}

}  // namespace mimir
