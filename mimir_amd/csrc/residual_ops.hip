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
    if (b) b[at] = round_bf16(v);
}

// The pair table's row for one row of the call, whose token is kept for the next: the thread with `keeps` does that.
__device__ __forceinline__ const uint16_t* pair_row(const PairTable& p, const int32_t* tokens, int64_t r, bool keeps) {
    const int64_t b = r / p.s, t = r % p.s, pos = p.past + (p.past_dev ? *p.past_dev : 0) + t;
    int32_t* held = p.held + b * p.held_ld;
    const int64_t token = tokens[r];
    int64_t row = p.buckets;
    if (pos > 0) row = ((int64_t)(t > 0 ? tokens[r - 1] : held[pos - 1]) * p.mul_prev + token * p.mul_cur) % p.buckets;
    if (keeps) held[pos] = (int32_t)token;
    return p.table + row * p.ld;
}

// floats of LDS: the row, the groups' parts and scales
size_t chain_lds(int width, int groups, int threads) {
    const int nw = threads / 64;
    return (size_t)(width + (groups > nw ? groups : nw) + groups) * 4;
}
int row_threads(int width) { return width >= 2048 ? 1024 : 256; }

template <bool EMBED>
__global__ __launch_bounds__(1024) void norm_chain_kernel(NormChain a) {
    extern __shared__ float lds_chain[];
    const int W = a.width, nw = blockDim.x >> 6, gs = W / a.groups;
    float* row = lds_chain;
    float* part = row + W;
    float* scale = part + (a.groups > nw ? a.groups : nw);
    const int64_t r = blockIdx.x;
    if constexpr (EMBED) {
        const uint16_t* e = a.table + (int64_t)a.tokens[r] * a.table_ld;
        for (int i = threadIdx.x; i < W; i += blockDim.x) row[i] = bf16_bits_to_f32(e[i]);
        if (a.pairs.table) {
            const uint16_t* pr = pair_row(a.pairs, a.tokens, r, threadIdx.x == 0);
            for (int i = threadIdx.x; i < W; i += blockDim.x) row[i] += bf16_bits_to_f32(pr[i]);
        }
    } else {
        for (int i = threadIdx.x; i < W; i += blockDim.x) row[i] = a.y ? a.y[r * a.ldy + i] : 0.f;
    }
    __syncthreads();
    if (a.w_post) group_scales(row, W, a.groups, a.eps, part, scale);
    const float own = a.dwa ? a.dwa[a.n_streams] : 1.f;
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
        float z = a.w_post ? row[i] * scale[i / gs] * a.w_post[i] : row[i];
        if (!EMBED) z += a.x[r * W + i];
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

// The same for rows whose groups are whole wavefronts of 256 elements: a thread owns E runs of four neighbouring elements in
// registers, everything that does not depend on a sum is requested at once, and a norm costs one barrier.
template <int E, bool EMBED>
__global__ __launch_bounds__(1024) void norm_chain_wide_kernel(NormChain a) {
    __shared__ float part[2][64];
    const int W = a.width, gs = W / a.groups, lane = threadIdx.x & 63;
    const int64_t r = blockIdx.x;
    int at[E];
    bool in[E];
#pragma unroll
    for (int e = 0; e < E; e++) {
        at[e] = (threadIdx.x + e * blockDim.x) * 4;
        in[e] = at[e] < W;  // whole wavefronts
    }
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    auto read = [&](const float* p, int e) { return in[e] ? *(const f32x4*)(p + at[e]) : zero; };
    // sums of squares: one of each wavefront's run, then the runs of a thread's own group
    auto norm = [&](const f32x4 v[E], float* sums, f32x4 out[E]) {
#pragma unroll
        for (int e = 0; e < E; e++) {
            const float ss = wave_sum(fmaf(v[e][0], v[e][0], fmaf(v[e][1], v[e][1], fmaf(v[e][2], v[e][2], v[e][3] * v[e][3]))));
            if (lane == 0 && in[e]) sums[at[e] >> 8] = ss;
        }
        __syncthreads();
        const int runs = gs >> 8;
#pragma unroll
        for (int e = 0; e < E; e++) {
            if (!in[e]) continue;
            const float* mine = sums + at[e] / gs * runs;
            float t = 0.f;
            for (int i = 0; i < runs; i++) t += mine[i];
            const float scale = 1.f / __builtin_sqrtf(t / (float)gs + a.eps);
            out[e] = v[e] * scale;
        }
    };
    f32x4 y[E], x[E], wp[E], wn[E], z[E], avg[E];
    const uint16_t* row = EMBED ? a.table + (int64_t)a.tokens[r] * a.table_ld : nullptr;
    const uint16_t* pair = EMBED && a.pairs.table ? pair_row(a.pairs, a.tokens, r, threadIdx.x == 0) : nullptr;
#pragma unroll
    for (int e = 0; e < E; e++) {
        if constexpr (EMBED) {
            u32x2 v = {0, 0};
            if (in[e]) v = *(const u32x2*)(row + at[e]);
            y[e] = f32x4{__uint_as_float(v[0] << 16), __uint_as_float(v[0] & 0xffff0000u), __uint_as_float(v[1] << 16), __uint_as_float(v[1] & 0xffff0000u)};
            if (pair && in[e]) {
                v = *(const u32x2*)(pair + at[e]);
                y[e] = y[e] + f32x4{__uint_as_float(v[0] << 16), __uint_as_float(v[0] & 0xffff0000u), __uint_as_float(v[1] << 16), __uint_as_float(v[1] & 0xffff0000u)};
            }
            x[e] = zero;
        } else {
            y[e] = a.y ? read(a.y + r * a.ldy, e) : zero;
            x[e] = read(a.x + r * W, e);
        }
        wp[e] = a.w_post ? read(a.w_post, e) : zero;
        wn[e] = a.w_next ? read(a.w_next, e) : zero;
        avg[e] = zero;
    }
    if (a.dwa)
        for (int j = 0; j < a.n_streams; j++) {
            const float w = a.dwa[j];
#pragma unroll
            for (int e = 0; e < E; e++) {
                const f32x4 v = read(a.streams + j * a.stream_stride + r * W, e);
#pragma unroll
                for (int i = 0; i < 4; i++) avg[e][i] = fmaf(w, v[i], avg[e][i]);
            }
        }
    if (a.w_post) norm(y, part[0], z);
    const float own = a.dwa ? a.dwa[a.n_streams] : 1.f;
#pragma unroll
    for (int e = 0; e < E; e++) {
        if (!in[e]) continue;
        z[e] = a.w_post ? x[e] + z[e] * wp[e] : x[e] + y[e];
        if (a.stream_out) *(f32x4*)(a.stream_out + r * W + at[e]) = z[e];
        if (a.dwa) {
#pragma unroll
            for (int i = 0; i < 4; i++) z[e][i] = fmaf(own, z[e][i], avg[e][i]);
        }
        if (a.x_out) *(f32x4*)(a.x_out + r * W + at[e]) = z[e];
    }
    if (!a.w_next) return;
#pragma unroll
    for (int e = 0; e < E; e++)
        if (!in[e]) z[e] = zero;
    f32x4 h[E];
    norm(z, part[1], h);
#pragma unroll
    for (int e = 0; e < E; e++) {
        if (!in[e]) continue;
        h[e] = h[e] * wn[e];
        if (a.conv_w) {
            const float* w = a.conv_w + (int64_t)at[e] * a.taps;
            float* hist = a.conv_state + r * (a.taps - 1) * W + at[e];
            f32x4 acc = zero;
            for (int j = 0; j + 1 < a.taps; j++) {
                const f32x4 old = *(const f32x4*)(hist + (int64_t)j * W);
#pragma unroll
                for (int i = 0; i < 4; i++) acc[i] = fmaf(w[i * a.taps + j], old[i], acc[i]);
                if (j > 0) *(f32x4*)(hist + (int64_t)(j - 1) * W) = old;
            }
#pragma unroll
            for (int i = 0; i < 4; i++) acc[i] = fmaf(w[(i + 1) * a.taps - 1], h[e][i], acc[i]);
            if (a.taps > 1) *(f32x4*)(hist + (int64_t)(a.taps - 2) * W) = h[e];
            h[e] = h[e] + acc;
        }
        if (a.h_f32) *(f32x4*)(a.h_f32 + r * a.ldh + at[e]) = h[e];
        if (a.h_bf16) *(u32x2*)(a.h_bf16 + r * a.ldh + at[e]) = u32x2{pack_bf16(h[e][0], h[e][1]), pack_bf16(h[e][2], h[e][3])};
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

// The same on whole wavefronts of 64 * 4 elements or groups that divide them: a thread's four elements in registers. A group is
// `lanes` lanes (a power of two up to 64) or whole wavefronts.
__global__ __launch_bounds__(1024) void gated_norm_wide_kernel(const float* __restrict__ o, const void* __restrict__ g, int g_bf16, int64_t ldg,
                                                               const float* __restrict__ w, int W, int groups, float eps, float* out_f32,
                                                               uint16_t* out_bf16, int64_t ldo) {
    __shared__ float part[16];
    const int i = threadIdx.x * 4, gs = W / groups, lane = threadIdx.x & 63;
    const int64_t r = blockIdx.x;
    const f32x4 v = *(const f32x4*)(o + r * W + i), wv = *(const f32x4*)(w + i);
    f32x4 z;
    if (g_bf16) {
        const u32x2 b = *(const u32x2*)((const uint16_t*)g + r * ldg + i);
        z = f32x4{__uint_as_float(b[0] << 16), __uint_as_float(b[0] & 0xffff0000u), __uint_as_float(b[1] << 16), __uint_as_float(b[1] & 0xffff0000u)};
    } else {
        z = *(const f32x4*)((const float*)g + r * ldg + i);
    }
    float ss = fmaf(v[0], v[0], fmaf(v[1], v[1], fmaf(v[2], v[2], v[3] * v[3])));
    if (gs >= 256) {
        ss = wave_sum(ss);
        if (lane == 0) part[threadIdx.x >> 6] = ss;
        __syncthreads();
        ss = 0.f;
        for (int k = 0; k < gs >> 8; k++) ss += part[(i / gs) * (gs >> 8) + k];
    } else {
        for (int d = gs >> 3; d > 0; d >>= 1) ss += __shfl_xor(ss, d);
    }
    const float scale = 1.f / __builtin_sqrtf(ss / (float)gs + eps);
    f32x4 y;
#pragma unroll
    for (int k = 0; k < 4; k++) y[k] = v[k] * scale * wv[k] * sigmoid_f32(z[k]);
    if (out_f32) *(f32x4*)(out_f32 + r * ldo + i) = y;
    if (out_bf16) *(u32x2*)(out_bf16 + r * ldo + i) = u32x2{pack_bf16(y[0], y[1]), pack_bf16(y[2], y[3])};
}

constexpr int kConvRun = 8;  // positions a thread walks

// A thread owns V neighbouring channels and walks kConvRun positions, its last taps - 1 inputs in registers (TAPS > 0) or
// read again (TAPS 0: any number of taps).
template <int TAPS, int V>
__global__ __launch_bounds__(256) void causal_conv_kernel(const float* __restrict__ h, const float* __restrict__ w, const float* __restrict__ state,
                                                          int taps_any, int64_t s, int W, float* out_f32, uint16_t* out_bf16, int64_t ldo) {
    const int taps = TAPS ? TAPS : taps_any;
    const int c = (blockIdx.x * 256 + threadIdx.x) * V;
    if (c >= W) return;
    const int64_t b = blockIdx.z, t0 = (int64_t)blockIdx.y * kConvRun, t1 = t0 + kConvRun < s ? t0 + kConvRun : s;
    typedef float vec __attribute__((ext_vector_type(V)));
    auto input = [&](int64_t t) { return *(const vec*)(t >= 0 ? h + (b * s + t) * W + c : state + (b * (taps - 1) + t + taps - 1) * W + c); };
    auto emit = [&](int64_t t, vec v) {
        if (out_f32) *(vec*)(out_f32 + (b * s + t) * ldo + c) = v;
        if (out_bf16) {
            uint16_t* o = out_bf16 + (b * s + t) * ldo + c;
            if constexpr (V == 4) *(u32x2*)o = u32x2{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3])};
            else o[0] = round_bf16(v[0]);
        }
    };
    if constexpr (TAPS > 0) {
        vec past[TAPS], k[TAPS], next[kConvRun];
#pragma unroll
        for (int j = 0; j < TAPS; j++)
#pragma unroll
            for (int i = 0; i < V; i++) k[j][i] = w[(int64_t)(c + i) * TAPS + j];
#pragma unroll
        for (int j = 0; j + 1 < TAPS; j++) past[j] = input(t0 - (TAPS - 1) + j);
#pragma unroll
        for (int u = 0; u < kConvRun; u++)
            if (t0 + u < t1) next[u] = input(t0 + u);
#pragma unroll
        for (int u = 0; u < kConvRun; u++) {
            if (t0 + u >= t1) break;
            past[TAPS - 1] = next[u];
            vec acc = k[0] * past[0];
#pragma unroll
            for (int j = 1; j < TAPS; j++)
#pragma unroll
                for (int i = 0; i < V; i++) acc[i] = fmaf(k[j][i], past[j][i], acc[i]);
            emit(t0 + u, next[u] + acc);
#pragma unroll
            for (int j = 0; j + 1 < TAPS; j++) past[j] = past[j + 1];
        }
    } else {
        for (int64_t t = t0; t < t1; t++) {
            vec acc;
            for (int i = 0; i < V; i++) acc[i] = 0.f;
            for (int j = 0; j < taps; j++) {
                const vec v = input(t - (taps - 1) + j);
                for (int i = 0; i < V; i++) acc[i] = fmaf(w[(int64_t)(c + i) * taps + j], v[i], acc[i]);
            }
            emit(t, input(t) + acc);
        }
    }
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
    auto whole = [](const void* p, int64_t ld) { return !p || (((uintptr_t)p & 15) == 0 && ld % 4 == 0); };
    if (a.width / a.groups % 256 == 0 && a.width <= 16384 && whole(a.table, a.table_ld) && whole(a.pairs.table, a.pairs.ld) && whole(a.y, a.ldy) && whole(a.x, 4) && whole(a.h_f32, a.ldh) &&
        whole(a.h_bf16, a.ldh) && whole(a.streams, a.stream_stride) && whole(a.stream_out, 4) && whole(a.x_out, 4) && whole(a.conv_state, 4)) {
        const int threads = a.width < 4096 ? a.width / 4 : 1024;  // a multiple of 64
        auto launch = [&](auto kernel) { hipLaunchKernelGGL(kernel, dim3((unsigned)rows), dim3(threads), 0, st, a); };
        if (a.width <= 4096) a.tokens ? launch(norm_chain_wide_kernel<1, true>) : launch(norm_chain_wide_kernel<1, false>);
        else if (a.width <= 8192) a.tokens ? launch(norm_chain_wide_kernel<2, true>) : launch(norm_chain_wide_kernel<2, false>);
        else a.tokens ? launch(norm_chain_wide_kernel<4, true>) : launch(norm_chain_wide_kernel<4, false>);
        return hipGetLastError();
    }
    const int threads = row_threads(a.width);
    const size_t lds = chain_lds(a.width, a.groups, threads);
    if (a.tokens) hipLaunchKernelGGL(norm_chain_kernel<true>, dim3((unsigned)rows), dim3(threads), lds, st, a);
    else hipLaunchKernelGGL(norm_chain_kernel<false>, dim3((unsigned)rows), dim3(threads), lds, st, a);
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
    const int gs = width / groups;
    if (width % 256 == 0 && width <= 4096 && ldg % 4 == 0 && ldo % 4 == 0 && ((uintptr_t)g & 15) == 0 && (gs % 256 == 0 || (gs < 256 && gs >= 4 && (gs & (gs - 1)) == 0))) {
        hipLaunchKernelGGL(gated_norm_wide_kernel, dim3((unsigned)rows), dim3(width / 4), 0, st, o, g, (int)g_bf16, ldg, w, width, groups, eps, out_f32, out_bf16,
                           ldo);
        return hipGetLastError();
    }
    const int threads = row_threads(width);
    hipLaunchKernelGGL(gated_norm_kernel, dim3((unsigned)rows), dim3(threads), chain_lds(width, groups, threads), st, o, g, (int)g_bf16, ldg, w, width,
                       groups, eps, out_f32, out_bf16, ldo);
    return hipGetLastError();
}

hipError_t causal_conv(const float* h, const float* w, float* state, int taps, int batch, int64_t s, int width, float* out_f32, uint16_t* out_bf16,
                       int64_t ldo, hipStream_t st) {
    if (batch * s == 0) return hipSuccess;
    const unsigned runs = (unsigned)((s + kConvRun - 1) / kConvRun), cols = (unsigned)((width + 255) / 256), cols4 = (unsigned)((width + 1023) / 1024);
    if (width % 4 == 0 && ldo % 4 == 0 && taps == 4)
        hipLaunchKernelGGL((causal_conv_kernel<4, 4>), dim3(cols4, runs, (unsigned)batch), dim3(256), 0, st, h, w, state, taps, s, width, out_f32, out_bf16, ldo);
    else if (width % 4 == 0 && ldo % 4 == 0)
        hipLaunchKernelGGL((causal_conv_kernel<0, 4>), dim3(cols4, runs, (unsigned)batch), dim3(256), 0, st, h, w, state, taps, s, width, out_f32, out_bf16, ldo);
    else
        hipLaunchKernelGGL((causal_conv_kernel<0, 1>), dim3(cols, runs, (unsigned)batch), dim3(256), 0, st, h, w, state, taps, s, width, out_f32, out_bf16, ldo);
    if (taps > 1) hipLaunchKernelGGL(conv_state_kernel, dim3(cols, (unsigned)batch), dim3(256), 0, st, h, state, taps, s, width);
    return hipGetLastError();
}

}  // namespace mimir
