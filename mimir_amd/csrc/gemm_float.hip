// y = act(x . W^T) for many rows of float32 x and bfloat16 weights on the float32 matrix cores
// (v_mfma_f32_32x32x2_f32): nothing is rounded below float32 on the way. The prompt product of a model that runs in
// float32, and in any model that of the few columns that must not be rounded (a recurrence's gates).
// A workgroup of four wavefronts owns 64 x 64 of y, a wavefront 32 x 32; steps of 32 along K go through LDS. Where W has
// few rows, a workgroup owns 16 rows of x and up to 64 of W instead, and its eight wavefronts cut K
// (gemm_f32_narrow_kernel): the tiles above would leave most of the device without work.
#include "device_util.h"
#include "product_store.h"
#include "stack_ops.h"

namespace mimir {

namespace {

typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr int kTile = 64, kStep = 32, kPad = kStep + 1;

template <Out KIND>
__global__ __launch_bounds__(256) void gemm_f32_kernel(const uint16_t* __restrict__ W, int64_t ldw, const float* __restrict__ x, int64_t ldx, int64_t M,
                                                       int64_t N, int64_t K, ProductOut out) {
    __shared__ float xs[2][kTile * kPad], ws[2][kTile * kPad];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r32 = lane & 31, hi = lane >> 5;
    const int64_t m0 = (int64_t)blockIdx.y * kTile, n0 = (int64_t)blockIdx.x * kTile;
    const int wm = (wave >> 1) * 32, wn = (wave & 1) * 32;
    // a thread brings eight neighbouring elements of one row of each operand
    const int lr = tid >> 2, lk = (tid & 3) * 8;
    const float* xp = x + (m0 + lr < M ? m0 + lr : M - 1) * ldx + lk;
    const uint16_t* wp = W + (n0 + lr < N ? n0 + lr : N - 1) * ldw + lk;
    f32x16 acc;
#pragma unroll
    for (int i = 0; i < 16; i++) acc[i] = 0.f;
    float xv[8];
    uint16_t wv[8];
    auto fetch = [&](int64_t k0) {
#pragma unroll
        for (int i = 0; i < 8; i++) xv[i] = k0 + lk + i < K ? xp[k0 + i] : 0.f;
#pragma unroll
        for (int i = 0; i < 8; i++) wv[i] = k0 + lk + i < K ? wp[k0 + i] : (uint16_t)0;
    };
    fetch(0);
    int p = 0;
    for (int64_t k0 = 0; k0 < K; k0 += kStep, p ^= 1) {
#pragma unroll
        for (int i = 0; i < 8; i++) {
            xs[p][lr * kPad + lk + i] = xv[i];
            ws[p][lr * kPad + lk + i] = bf16_bits_to_f32(wv[i]);
        }
        __syncthreads();  // the other stage is written next only after everyone has passed the next barrier
        if (k0 + kStep < K) fetch(k0 + kStep);
        // a step's sum on its own and then added: the matrix cores add one product after the other, and the error of a
        // long chain grows with its length
        f32x16 part;
#pragma unroll
        for (int i = 0; i < 16; i++) part[i] = 0.f;
#pragma unroll
        for (int k = 0; k < kStep; k += 2)
            part = __builtin_amdgcn_mfma_f32_32x32x2f32(xs[p][(wm + r32) * kPad + k + hi], ws[p][(wn + r32) * kPad + k + hi], part, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < 16; i++) acc[i] += part[i];
        if (KIND == Out::Scaled && out.mid && k0 + kStep == out.split) {
            const float f = out.mid[n0 + wn + r32 < N ? n0 + wn + r32 : N - 1];
#pragma unroll
            for (int i = 0; i < 16; i++) acc[i] *= f;
        }
    }
#pragma unroll
    for (int i = 0; i < 16; i++) {
        const int64_t m = m0 + wm + (i & 3) + 8 * (i >> 2) + 4 * hi, n = n0 + wn + r32;
        const float beside = KIND == Out::Pairs ? __shfl_xor(acc[i], 1) : 0.f;  // the column beside this one
        if (m >= M || n >= N) continue;
        if (KIND != Out::Pairs || n < out.pair_from) store_column<KIND>(out, m, n, acc[i]);
        else if ((n & 1) == 0) store_pair(out, m, n, acc[i], beside);
    }
}

constexpr int kNarrow = 64;  // rows of W a workgroup

// v_mfma_f32_16x16x4: lane (row, k). A lane brings four neighbouring elements of K of its row, so the four products of a step
// of sixteen take K in the order 4 k + j, in both operands alike.
template <Out KIND>
__global__ __launch_bounds__(512) void gemm_f32_narrow_kernel(const uint16_t* __restrict__ W, int64_t ldw, const float* __restrict__ x, int64_t ldx, int64_t M,
                                                              int64_t N, int64_t K, ProductOut out) {
    __shared__ float red[8][16][kNarrow + 1];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int64_t m0 = (int64_t)blockIdx.y * 16, n0 = (int64_t)blockIdx.x * kNarrow;
    const int64_t steps = (K + 15) / 16, per = (steps + 7) / 8, k0 = wave * per * 16, k1 = k0 + per * 16 < steps * 16 ? k0 + per * 16 : steps * 16;
    const float* xp = x + (m0 + r16 < M ? m0 + r16 : M - 1) * ldx + g * 4;
    const uint16_t* wp[kNarrow / 16];
#pragma unroll
    for (int t = 0; t < kNarrow / 16; t++) wp[t] = W + (n0 + t * 16 + r16 < N ? n0 + t * 16 + r16 : N - 1) * ldw + g * 4;
    f32x4 acc[kNarrow / 16];
#pragma unroll
    for (int t = 0; t < kNarrow / 16; t++) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    auto sum_of = [&](int64_t from, int64_t to) {
#pragma unroll 4
        for (int64_t k = from; k < to; k += 16) {  // both operands' rows are padded to a multiple of 64
            const f32x4 a = *(const f32x4*)(xp + k);
            u32x2 w[kNarrow / 16];
#pragma unroll
            for (int t = 0; t < kNarrow / 16; t++) w[t] = *(const u32x2*)(wp[t] + k);
#pragma unroll
            for (int t = 0; t < kNarrow / 16; t++)
#pragma unroll
                for (int j = 0; j < 4; j++)
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], __uint_as_float(j & 1 ? w[t][j >> 1] & 0xffff0000u : w[t][j >> 1] << 16), acc[t], 0, 0, 0);
        }
    };
    int64_t from = k0;
    if (KIND == Out::Scaled && out.mid) {  // what of this wavefront's piece lies below split has a factor of its own
        const int64_t to = out.split < k1 ? out.split : k1;
        sum_of(k0, to);
#pragma unroll
        for (int t = 0; t < kNarrow / 16; t++) acc[t] = acc[t] * out.mid[n0 + t * 16 + r16 < N ? n0 + t * 16 + r16 : N - 1];
        if (to > from) from = to;
    }
    sum_of(from, k1);
#pragma unroll
    for (int t = 0; t < kNarrow / 16; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) red[wave][4 * g + i][t * 16 + r16] = acc[t][i];
    __syncthreads();
    for (int o = tid; o < 16 * kNarrow; o += 512) {
        const int row = o / kNarrow, col = o % kNarrow;
        const int64_t m = m0 + row, n = n0 + col;
        if (m >= M || n >= N) continue;
        auto sum = [&](int c) {
            float v = 0.f;
#pragma unroll
            for (int i = 0; i < 8; i++) v += red[i][row][c];
            return v;
        };
        if (KIND != Out::Pairs || n < out.pair_from) store_column<KIND>(out, m, n, sum(col));
        else if ((col & 1) == 0) store_pair(out, m, n, sum(col), sum(col + 1));
    }
}

template <Out KIND>
void launch(const uint16_t* W, int64_t ldw, const float* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st) {
    if (N <= 2 * kNarrow && ldx % 4 == 0 && ldw % 4 == 0)
        hipLaunchKernelGGL(gemm_f32_narrow_kernel<KIND>, dim3((unsigned)((N + kNarrow - 1) / kNarrow), (unsigned)((M + 15) / 16)), dim3(512), 0, st, W, ldw, x, ldx,
                           M, N, K, out);
    else
        hipLaunchKernelGGL(gemm_f32_kernel<KIND>, dim3((unsigned)((N + kTile - 1) / kTile), (unsigned)((M + kTile - 1) / kTile)), dim3(256), 0, st, W, ldw, x, ldx,
                           M, N, K, out);
}

}  // namespace

hipError_t gemm_f32(const uint16_t* W, int64_t ldw, const float* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st) {
    if (M == 0 || N == 0) return hipSuccess;
    const Out kind = out_kind(out, N);
    if (kind == Out::Plain) launch<Out::Plain>(W, ldw, x, ldx, M, N, K, out, st);
    else if (kind == Out::Pairs) launch<Out::Pairs>(W, ldw, x, ldx, M, N, K, out, st);
    else launch<Out::Scaled>(W, ldw, x, ldx, M, N, K, out, st);
    return hipGetLastError();
}

}  // namespace mimir
