// What lies between the products of a stack's layers, on whole rows: norms in groups with the residual sum, the depth
// average over earlier layers' results, the short causal convolution of a mixer's input, and the gated norm of a
// mixer's output. A row's steps are one launch (norm_chain), since each would be a pass over the row alone. All float32.
#include "device_util.h"
#include "stack_ops.h"

namespace mimir {

namespace {

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.f / (1.f + expf(-z)); }

// 1 / sqrt(mean(part^2) + eps) of every group of a row in LDS. Wavefronts share the groups' sums: a group is cut into
// parts where there are more wavefronts than groups. `part` holds groups * parts sums. Ends with a barrier.
__device__ __forceinline__ void group_scales(const float* row, int width, int groups, float eps, float* part, float* scale) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    const int gs = width / groups, parts = nw > groups ? nw / groups : 1, per = (gs + parts - 1) / parts;
    for (int item = wave; item < groups * parts; item += nw) {
        const int g = item / parts, p = item % parts;
        const int hi = (p + 1) * per < gs ? (p + 1) * per : gs;
        float ss = 0.f;
        for (int i = p * per + lane; i < hi; i += 64) {
            const float v = row[g * gs + i];
            ss = fmaf(v, v, ss);
        }
        ss = wave_sum(ss);
        if (lane == 0) part[item] = ss;
    }
    __syncthreads();
    for (int g = threadIdx.x; g < groups; g += blockDim.x) {
        float t = 0.f;
        for (int p = 0; p < parts; p++) t += part[g * parts + p];
        scale[g] = 1.f / __builtin_sqrtf(t / (float)gs + eps);
    }
    __syncthreads();
}

__device__ __forceinline__ void put(float* f, uint16_t* b, int64_t at, float v) {
    if (f) f[at] = v;
    if (b) b[at] = f32_to_bf16_bits(v);
}

// floats of LDS: the row, the groups' parts and scales
size_t chain_lds(int width, int groups, int threads) {
    const int nw = threads / 64;
    return (size_t)(width + (groups > nw ? groups : nw) + groups) * 4;
}
int row_threads(int width) { return width >= 2048 ? 1024 : 256; }

__global__ __launch_bounds__(1024) void norm_chain_kernel(NormChain a) {
    extern __shared__ float lds_chain[];
    const int W = a.width, nw = blockDim.x >> 6, gs = W / a.groups;
    float* row = lds_chain;
    float* part = row + W;
    float* scale = part + (a.groups > nw ? a.groups : nw);
    const int64_t r = blockIdx.x;
    if (a.tokens) {
        const uint16_t* e = a.table + (int64_t)a.tokens[r] * a.table_ld;
        for (int i = threadIdx.x; i < W; i += blockDim.x) row[i] = bf16_bits_to_f32(e[i]);
    } else {
        for (int i = threadIdx.x; i < W; i += blockDim.x) row[i] = a.y[r * a.ldy + i];
    }
    __syncthreads();
    group_scales(row, W, a.groups, a.eps, part, scale);
    const float own = a.dwa ? a.dwa[a.n_streams] : 1.f;
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
        float z = row[i] * scale[i / gs] * a.w_post[i];
        if (!a.tokens) z += a.x[r * W + i];
        if (a.stream_out) a.stream_out[r * W + i] = z;
        if (a.dwa) {
            float acc = 0.f;
            for (int j0 = 0; j0 < a.n_streams; j0 += 8) {  // eight earlier results requested at a time
                float v[8];
#pragma unroll
                for (int u = 0; u < 8; u++) v[u] = j0 + u < a.n_streams ? a.streams[(j0 + u) * a.stream_stride + r * W + i] : 0.f;
#pragma unroll
                for (int u = 0; u < 8; u++)
                    if (j0 + u < a.n_streams) acc = fmaf(a.dwa[j0 + u], v[u], acc);
            }
            z = fmaf(own, z, acc);
        }
        if (a.x_out) a.x_out[r * W + i] = z;
        row[i] = z;
    }
    if (!a.w_next) return;
    __syncthreads();
    group_scales(row, W, a.groups, a.eps, part, scale);
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
        float h = row[i] * scale[i / gs] * a.w_next[i];
        if (a.conv_w) {
            const float* w = a.conv_w + (int64_t)i * a.taps;
            float* hist = a.conv_state + r * (a.taps - 1) * W + i;
            float acc = 0.f;
            for (int j = 0; j + 1 < a.taps; j++) {
                const float old = hist[(int64_t)j * W];
                acc = fmaf(w[j], old, acc);
                if (j > 0) hist[(int64_t)(j - 1) * W] = old;
            }
            acc = fmaf(w[a.taps - 1], h, acc);
            if (a.taps > 1) hist[(int64_t)(a.taps - 2) * W] = h;
            h += acc;
        }
        put(a.h_f32, a.h_bf16, r * a.ldh + i, h);
    }
}

__global__ __launch_bounds__(1024) void norm_rows_kernel(const float* __restrict__ x, const int64_t* __restrict__ rows, const float* __restrict__ w, int W,
                                                         int groups, float eps, float* out_f32, uint16_t* out_bf16, int64_t ldo) {
    extern __shared__ float lds_chain[];
    const int nw = blockDim.x >> 6, gs = W / groups;
    float* row = lds_chain;
    float* part = row + W;
    float* scale = part + (groups > nw ? groups : nw);
    const float* from = x + rows[blockIdx.x] * W;
    for (int i = threadIdx.x; i < W; i += blockDim.x) row[i] = from[i];
    __syncthreads();
    group_scales(row, W, groups, eps, part, scale);
    for (int i = threadIdx.x; i < W; i += blockDim.x) put(out_f32, out_bf16, blockIdx.x * ldo + i, row[i] * scale[i / gs] * w[i]);
}

__global__ __launch_bounds__(1024) void gated_norm_kernel(const float* __restrict__ o, const void* __restrict__ g, int g_bf16, int64_t ldg,
                                                          const float* __restrict__ w, int W, int groups, float eps, float* out_f32, uint16_t* out_bf16,
                                                          int64_t ldo) {
    extern __shared__ float lds_chain[];
    const int nw = blockDim.x >> 6, gs = W / groups;
    float* row = lds_chain;
    float* part = row + W;
    float* scale = part + (groups > nw ? groups : nw);
    const int64_t r = blockIdx.x;
    for (int i = threadIdx.x; i < W; i += blockDim.x) row[i] = o[r * W + i];
    __syncthreads();
    group_scales(row, W, groups, eps, part, scale);
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
        const float z = g_bf16 ? bf16_bits_to_f32(((const uint16_t*)g)[r * ldg + i]) : ((const float*)g)[r * ldg + i];
        put(out_f32, out_bf16, r * ldo + i, row[i] * scale[i / gs] * w[i] * sigmoid_f32(z));
    }
}

__global__ __launch_bounds__(256) void causal_conv_kernel(const float* __restrict__ h, const float* __restrict__ w, const float* __restrict__ state,
                                                          int taps, int64_t s, int W, float* out_f32, uint16_t* out_bf16, int64_t ldo) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= W) return;
    const int64_t r = blockIdx.y, b = r / s, t = r % s;
    const float own = h[r * W + c];
    float acc = 0.f;
    for (int j = 0; j < taps; j++) {
        const int64_t at = t - (taps - 1) + j;
        const float v = at >= 0 ? h[(b * s + at) * W + c] : state[(b * (taps - 1) + at + taps - 1) * W + c];
        acc = fmaf(w[(int64_t)c * taps + j], v, acc);
    }
    put(out_f32, out_bf16, r * ldo + c, own + acc);
}

// state row j of taps - 1 becomes the row s positions later; ascending, since a later row is read before it is written.
__global__ __launch_bounds__(256) void conv_state_kernel(const float* __restrict__ h, float* __restrict__ state, int taps, int64_t s, int W) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= W) return;
    const int64_t b = blockIdx.y;
    float* mine = state + b * (taps - 1) * W + c;
    for (int j = 0; j + 1 < taps; j++) {
        const int64_t at = s - (taps - 1) + j;
        mine[(int64_t)j * W] = at >= 0 ? h[(b * s + at) * W + c] : mine[(at + taps - 1) * W];
    }
}

}  // namespace

hipError_t norm_chain(const NormChain& a, int64_t rows, hipStream_t st) {
    if (rows == 0) return hipSuccess;
    const int threads = row_threads(a.width);
    hipLaunchKernelGGL(norm_chain_kernel, dim3((unsigned)rows), dim3(threads), chain_lds(a.width, a.groups, threads), st, a);
    return hipGetLastError();
}

hipError_t norm_rows(const float* x, const int64_t* rows, int64_t n, const float* w, int width, int groups, float eps, float* out_f32,
                     uint16_t* out_bf16, int64_t ldo, hipStream_t st) {
    if (n == 0) return hipSuccess;
    const int threads = row_threads(width);
    hipLaunchKernelGGL(norm_rows_kernel, dim3((unsigned)n), dim3(threads), chain_lds(width, groups, threads), st, x, rows, w, width, groups, eps, out_f32,
                       out_bf16, ldo);
    return hipGetLastError();
}

hipError_t gated_norm(const float* o, const void* g, bool g_bf16, int64_t ldg, const float* w, int64_t rows, int width, int groups, float eps,
                      float* out_f32, uint16_t* out_bf16, int64_t ldo, hipStream_t st) {
    if (rows == 0) return hipSuccess;
    const int threads = row_threads(width);
    hipLaunchKernelGGL(gated_norm_kernel, dim3((unsigned)rows), dim3(threads), chain_lds(width, groups, threads), st, o, g, (int)g_bf16, ldg, w, width,
                       groups, eps, out_f32, out_bf16, ldo);
    return hipGetLastError();
}

hipError_t causal_conv(const float* h, const float* w, float* state, int taps, int batch, int64_t s, int width, float* out_f32, uint16_t* out_bf16,
                       int64_t ldo, hipStream_t st) {
    if (batch * s == 0) return hipSuccess;
    const unsigned cols = (unsigned)((width + 255) / 256);
    hipLaunchKernelGGL(causal_conv_kernel, dim3(cols, (unsigned)(batch * s)), dim3(256), 0, st, h, w, state, taps, s, width, out_f32, out_bf16, ldo);
    if (taps > 1) hipLaunchKernelGGL(conv_state_kernel, dim3(cols, (unsigned)batch), dim3(256), 0, st, h, state, taps, s, width);
    return hipGetLastError();
}

}  // namespace mimir
