// Latent attention: a head's keys and values are W_uk c and W_uv c of a latent c of `rank`, beside a rotated key part that
// all heads share, and only c and that part are kept (struct Latent, stack_ops.h).
//
// latent_absorbed serves few query rows (a decoding step, a short portion) and everything in float32 without forming
// keys or values: q_h . (W_uk,h c_j) = (W_uk,h^T q_h) . c_j, so a head's query goes to the latents' space once
// (latent_absorb_kernel) and all heads read the same cache rows; the weighted sum of the latents comes back through W_uv,h
// (latent_combine_kernel). The keys of a row are cut into shares that workgroups take side by side.
#include "device_util.h"
#include "stack_ops.h"

namespace mimir {

namespace {

__device__ __forceinline__ float block_sum_256(float v, float* part) {
    v = wave_sum(v);
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
    __syncthreads();
    return (part[0] + part[1]) + (part[2] + part[3]);
}

__device__ __forceinline__ int64_t past_of(const Latent& a) { return a.past + (a.past_dev ? *a.past_dev : 0); }

// One workgroup a row: the latent's norm and the rotations.
__global__ __launch_bounds__(256) void latent_prepare_kernel(Latent a, float* __restrict__ proj, int64_t ldp, uint16_t* __restrict__ q16, int64_t ldq) {
    __shared__ float part[4];
    const int64_t r = blockIdx.x, b = r / a.s, pos = past_of(a) + r % a.s;
    const int D = a.dim + a.rot_dim, half = a.rot_dim / 2;
    float* p = proj + r * ldp;
    const float* low = p + (int64_t)a.heads * D;
    const float *cs = a.cos_t + pos * half, *sn = a.sin_t + pos * half;
    float ss = 0.f;
    for (int i = threadIdx.x; i < a.rank; i += 256) ss = fmaf(low[i], low[i], ss);
    ss = block_sum_256(ss, part);
    const float scale = 1.f / __builtin_sqrtf(ss / (float)a.rank + a.eps);
    const int64_t at = (b * a.context + pos) * a.ldc;
    float* c32 = a.cache_bf16 ? nullptr : (float*)a.cache + at;
    uint16_t* c16 = a.cache_bf16 ? (uint16_t*)a.cache + at : nullptr;
    auto keep = [&](int i, float v) {
        if (c32) c32[i] = v;
        else c16[i] = f32_to_bf16_bits(v);
    };
    for (int i = threadIdx.x; i < a.rank; i += 256) keep(i, low[i] * scale * a.norm_w[i]);
    for (int i = threadIdx.x; i < half; i += 256) {
        const float u = low[a.rank + 2 * i], v = low[a.rank + 2 * i + 1];
        keep(a.rank + 2 * i, u * cs[i] - v * sn[i]);
        keep(a.rank + 2 * i + 1, v * cs[i] + u * sn[i]);
    }
    for (int i = threadIdx.x; i < a.heads * half; i += 256) {
        const int h = i / half, j = i % half;
        const int64_t o = (int64_t)h * D + a.dim + 2 * j;
        const float u = p[o], v = p[o + 1];
        const float x = u * cs[j] - v * sn[j], y = v * cs[j] + u * sn[j];
        if (q16) {
            q16[r * ldq + o] = f32_to_bf16_bits(x);
            q16[r * ldq + o + 1] = f32_to_bf16_bits(y);
        } else {
            p[o] = x;
            p[o + 1] = y;
        }
    }
    if (q16)
        for (int i = threadIdx.x; i < a.heads * a.dim; i += 256) {
            const int64_t o = (int64_t)(i / a.dim) * D + i % a.dim;
            q16[r * ldq + o] = f32_to_bf16_bits(p[o]);
        }
}

// q'[row, h, :] = W_uk,h^T q_h: 256 columns a workgroup, eight a thread, the head's rows of W_uk shared by eight groups.
__global__ __launch_bounds__(256) void latent_absorb_kernel(Latent a, const float* __restrict__ proj, int64_t ldp, float* __restrict__ qa) {
    __shared__ float red[8][256 + 8];
    const int64_t r = blockIdx.x;
    const int h = blockIdx.y, c0 = blockIdx.z * 256 + (threadIdx.x & 31) * 8, g = threadIdx.x >> 5;
    const float* q = proj + r * ldp + (int64_t)h * (a.dim + a.rot_dim);
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (c0 < a.rank)
        for (int d = g; d < a.dim; d += 8) {
            const u32x4 w = *(const u32x4*)(a.w_uk + ((int64_t)h * a.dim + d) * a.ldw + c0);  // rows are padded with zeros
            const float x = q[d];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                acc[2 * i] = fmaf(x, __uint_as_float(w[i] << 16), acc[2 * i]);
                acc[2 * i + 1] = fmaf(x, __uint_as_float(w[i] & 0xffff0000u), acc[2 * i + 1]);
            }
        }
#pragma unroll
    for (int i = 0; i < 8; i++) red[g][(threadIdx.x & 31) * 8 + i] = acc[i];
    __syncthreads();
    const int c = blockIdx.z * 256 + threadIdx.x;
    if (c >= a.rank) return;
    float v = 0.f;
#pragma unroll
    for (int i = 0; i < 8; i++) v += red[i][threadIdx.x];
    qa[(r * a.heads + h) * a.rank + c] = v;
}

constexpr int kHeads = 16;  // heads a workgroup
constexpr int kKeys = 64;   // keys a tile

// Eight cache elements from `at` on, as float32.
template <typename T>
__device__ __forceinline__ void load8(const T* p, float v[8]);
template <>
__device__ __forceinline__ void load8<float>(const float* p, float v[8]) {
    const f32x4 x = ((const f32x4*)p)[0], y = ((const f32x4*)p)[1];
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = x[i], v[4 + i] = y[i];
}
template <>
__device__ __forceinline__ void load8<uint16_t>(const uint16_t* p, float v[8]) {
    const u32x4 x = *(const u32x4*)p;
#pragma unroll
    for (int i = 0; i < 4; i++) v[2 * i] = __uint_as_float(x[i] << 16), v[2 * i + 1] = __uint_as_float(x[i] & 0xffff0000u);
}
__device__ __forceinline__ float widen1(float v) { return v; }
__device__ __forceinline__ float widen1(uint16_t v) { return bf16_bits_to_f32(v); }

// The share `split` of the keys of one row, for kHeads heads: scores with a lane's key against four heads a
// wavefront, a running softmax, and the weighted sum of the latents with a thread's columns tid + 256 u.
// parts: [rows, splits, heads, rank] sums, then [rows, splits, heads, 2] (maximum, sum of weights).
template <typename T, int U>
__global__ __launch_bounds__(256) void latent_attend_kernel(Latent a, const float* __restrict__ proj, int64_t ldp, const float* __restrict__ qa, int splits,
                                                            float* __restrict__ part_o, float* __restrict__ part_ml) {
    extern __shared__ __align__(16) float lds_latent[];
    const int L8 = (a.rank + a.rot_dim + 7) / 8 * 8;
    float* qs = lds_latent;                    // [L8][kHeads]
    float* ps = qs + (size_t)L8 * kHeads;      // [kKeys][kHeads]: scores, then weights
    float* ml = ps + kKeys * kHeads;           // [kHeads] rescaling of this tile
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int split = blockIdx.x, h0 = blockIdx.y * kHeads;
    const int64_t r = blockIdx.z, b = r / a.s;
    const int64_t seen = past_of(a) + r % a.s + 1;
    int64_t share = (seen + splits - 1) / splits;
    share = (share + kKeys - 1) / kKeys * kKeys;
    const int64_t lo = split * share, hi = lo + share < seen ? lo + share : seen;
    const int64_t pr = (r * splits + split) * a.heads;
    if (lo >= hi) {  // the whole workgroup: nothing to add
        if (tid < kHeads && h0 + tid < a.heads) {
            part_ml[(pr + h0 + tid) * 2] = -__builtin_inff();
            part_ml[(pr + h0 + tid) * 2 + 1] = 0.f;
        }
        return;
    }
    for (int i = tid; i < L8 * kHeads; i += 256) {
        const int d = i / kHeads, h = h0 + i % kHeads;
        float v = 0.f;
        if (h < a.heads) {
            if (d < a.rank) v = qa[(r * a.heads + h) * a.rank + d];
            else if (d < a.rank + a.rot_dim) v = proj[r * ldp + (int64_t)h * (a.dim + a.rot_dim) + a.dim + d - a.rank];
        }
        qs[i] = v * a.scale;
    }
    const T* cache = (const T*)a.cache + b * a.context * a.ldc;
    float acc[kHeads][U];
#pragma unroll
    for (int h = 0; h < kHeads; h++)
#pragma unroll
        for (int u = 0; u < U; u++) acc[h][u] = 0.f;
    const int sh = tid >> 4, sk = tid & 15;  // the softmax's head and first key of this thread (16 threads a head)
    float m = -__builtin_inff(), l = 0.f;
    __syncthreads();
    for (int64_t j0 = lo; j0 < hi; j0 += kKeys) {
        {
            const int64_t j = j0 + lane < hi ? j0 + lane : hi - 1;
            const T* c = cache + j * a.ldc;
            f32x4 sc = {0.f, 0.f, 0.f, 0.f};
            for (int d = 0; d < L8; d += 8) {  // a row is padded to a multiple of 8
                float v[8];
                load8(c + d, v);
#pragma unroll
                for (int i = 0; i < 8; i++) {
                    const f32x4 q = *(const f32x4*)(qs + (d + i) * kHeads + wave * 4);
#pragma unroll
                    for (int h = 0; h < 4; h++) sc[h] = fmaf(q[h], v[i], sc[h]);
                }
            }
            *(f32x4*)(ps + lane * kHeads + wave * 4) = sc;
        }
        __syncthreads();
        {
            float s[kKeys / 16], top = -__builtin_inff();
#pragma unroll
            for (int i = 0; i < kKeys / 16; i++) {
                s[i] = j0 + sk + 16 * i < hi ? ps[(sk + 16 * i) * kHeads + sh] : -__builtin_inff();
                top = fmaxf(top, s[i]);
            }
#pragma unroll
            for (int o = 8; o > 0; o >>= 1) top = fmaxf(top, __shfl_xor(top, o));
            const float next = fmaxf(m, top), back = expf(m - next);  // the first tile's m: exp(-inf) = 0
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < kKeys / 16; i++) {
                const float p = expf(s[i] - next);
                sum += p;
                ps[(sk + 16 * i) * kHeads + sh] = p;
            }
#pragma unroll
            for (int o = 8; o > 0; o >>= 1) sum += __shfl_xor(sum, o);
            m = next;
            l = l * back + sum;
            if (sk == 0) ml[sh] = back;
        }
        __syncthreads();
        float back[kHeads];
#pragma unroll
        for (int h = 0; h < kHeads; h += 4) {
            const f32x4 v = *(const f32x4*)(ml + h);
#pragma unroll
            for (int i = 0; i < 4; i++) back[h + i] = v[i];
        }
        const int n = hi - j0 < kKeys ? (int)(hi - j0) : kKeys;
        if (tid < a.rank) {
#pragma unroll
            for (int h = 0; h < kHeads; h++)
#pragma unroll
                for (int u = 0; u < U; u++) acc[h][u] *= back[h];
#pragma unroll 4
            for (int j = 0; j < n; j++) {
                const T* c = cache + (j0 + j) * a.ldc;
                float v[U];
#pragma unroll
                for (int u = 0; u < U; u++) v[u] = tid + 256 * u < a.rank ? widen1(c[tid + 256 * u]) : 0.f;
#pragma unroll
                for (int h = 0; h < kHeads; h += 4) {
                    const f32x4 p = *(const f32x4*)(ps + j * kHeads + h);
#pragma unroll
                    for (int i = 0; i < 4; i++)
#pragma unroll
                        for (int u = 0; u < U; u++) acc[h + i][u] = fmaf(p[i], v[u], acc[h + i][u]);
                }
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int h = 0; h < kHeads; h++)
#pragma unroll
        for (int u = 0; u < U; u++)
            if (h0 + h < a.heads && tid + 256 * u < a.rank) part_o[(pr + h0 + h) * a.rank + tid + 256 * u] = acc[h][u];
    if (sk == 0 && h0 + sh < a.heads) {
        part_ml[(pr + h0 + sh) * 2] = m;
        part_ml[(pr + h0 + sh) * 2 + 1] = l;
    }
}

constexpr int kValues = 32;  // values a workgroup of latent_combine_kernel

// The shares of a head brought together, then its values: out[row, h, e] = W_uv[h, e, :] . (sum of latents).
__global__ __launch_bounds__(256) void latent_combine_kernel(Latent a, int splits, const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                                             float* __restrict__ out_f32, uint16_t* __restrict__ out_bf16, int64_t ldo) {
    extern __shared__ __align__(16) float lds_latent[];
    float* oc = lds_latent;  // [rank to a multiple of 64]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.y;
    const int64_t r = blockIdx.x;
    const int R64 = (a.rank + 63) / 64 * 64;
    const float* mlp = part_ml + (r * splits * a.heads + h) * 2;
    const int64_t step = (int64_t)a.heads * 2;
    float top = -__builtin_inff();
    for (int s = lane; s < splits; s += 64) top = fmaxf(top, mlp[s * step]);
    top = wave_max(top);
    float sum = 0.f;
    for (int s = lane; s < splits; s += 64) sum = fmaf(mlp[s * step + 1], expf(mlp[s * step] - top), sum);
    const float inv = 1.f / wave_sum(sum);
    for (int c = tid; c < R64; c += 256) {
        float v = 0.f;
        if (c < a.rank)
            for (int s = 0; s < splits; s++) {
                const float m = mlp[s * step];
                if (m == -__builtin_inff()) continue;  // a share without keys wrote no sums
                v = fmaf(part_o[((r * splits + s) * a.heads + h) * a.rank + c], expf(m - top), v);
            }
        oc[c] = v * inv;
    }
    __syncthreads();
    const int e1 = (int)(blockIdx.z + 1) * kValues < a.vdim ? (int)(blockIdx.z + 1) * kValues : a.vdim;
    for (int e = blockIdx.z * kValues + wave; e < e1; e += 4) {
        const uint16_t* w = a.w_uv + ((int64_t)h * a.vdim + e) * a.ldw;
        float v = 0.f;
        for (int c = lane * 8; c < R64; c += 512) {
            const u32x4 x = *(const u32x4*)(w + c);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                v = fmaf(oc[c + 2 * i], __uint_as_float(x[i] << 16), v);
                v = fmaf(oc[c + 2 * i + 1], __uint_as_float(x[i] & 0xffff0000u), v);
            }
        }
        v = wave_sum(v);
        if (lane == 0) {
            const int64_t at = r * ldo + (int64_t)h * a.vdim + e;
            if (out_f32) out_f32[at] = v;
            else out_bf16[at] = f32_to_bf16_bits(v);
        }
    }
}

template <typename T, int U>
hipError_t launch_attend(const Latent& a, const float* proj, int64_t ldp, const float* qa, int splits, float* po, float* ml, hipStream_t st) {
    const size_t lds = ((size_t)(a.rank + a.rot_dim + 7) / 8 * 8 * kHeads + kKeys * kHeads + kHeads) * 4;
    if (lds > 64 * 1024) {
        hipError_t e = hipFuncSetAttribute((const void*)latent_attend_kernel<T, U>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    const dim3 grid((unsigned)splits, (unsigned)((a.heads + kHeads - 1) / kHeads), (unsigned)(a.batch * a.s));
    hipLaunchKernelGGL((latent_attend_kernel<T, U>), grid, dim3(256), lds, st, a, proj, ldp, qa, splits, po, ml);
    return hipGetLastError();
}

// ---- many query rows ------------------------------------------------------------------------
// A wavefront owns 32 query rows of one head and walks the keys in tiles of 64 with a running maximum and sum per row.
// Both products are computed transposed (scores^T = K Q^T, result^T = V^T P^T), so that a row's scores and results lie in
// one lane and its partner 32 lanes on, and the weights go from the exponential straight into the second product's
// operand: the order in which the scores' registers hold the keys is the order in which V^T's fragment is read. Four
// wavefronts with consecutive rows share a tile of keys and values in LDS; the next tile is requested while one is used.

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

__device__ __forceinline__ f32x16 mfma_bf16(u32x4 a, u32x4 b, f32x16 c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
__device__ __forceinline__ uint32_t pack2(float lo, float hi) { return (uint32_t)f32_to_bf16_bits(lo) | (uint32_t)f32_to_bf16_bits(hi) << 16; }
__device__ __forceinline__ float low_part(float v) { return v - bf16_bits_to_f32(f32_to_bf16_bits(v)); }

struct PromptArgs {
    const uint16_t *q, *keys, *vt, *cache;  // cache: the sequence's rows
    uint16_t* out;
    int64_t ldq, ldk, ldv, ldc, ldo;
    int heads, dim, rot_dim, vdim, rank;
    int past, s;
    float scale;  // times log2(e)
};

constexpr int kPromptRows = 128;

// DT: sixteenths of dim + rot_dim, rounded up; VT: 32nds of vdim, rounded up. WHOLE: rows and their parts are multiples of
// 16 bytes (else keys and queries are brought element by element).
template <int DT, int VT, bool WHOLE>
__global__ __launch_bounds__(256, DT > 12 ? 1 : 2) void latent_prompt_kernel(PromptArgs p) {
    constexpr int kKey = DT * 16 + 8, kVal = kKeys + 8;  // elements between rows in LDS
    constexpr int kKeyLoads = (kKeys * DT * 2 + 255) / 256;
    __shared__ __align__(16) uint16_t ks[kKeys * kKey];
    __shared__ __align__(16) uint16_t vs[VT * 32 * kVal];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r32 = lane & 31, hi = lane >> 5;
    const int h = blockIdx.x, first = (int)(gridDim.y - 1 - blockIdx.y) * kPromptRows;  // the last rows first: they see the most keys
    const int D = p.dim + p.rot_dim, n_keys = p.past + p.s;
    const int row = first + wave * 32 + r32, pos = p.past + row;  // sees keys 0 .. pos
    const int last_wg = first + kPromptRows < p.s ? first + kPromptRows : p.s;
    const int seen_wg = p.past + last_wg;
    const int seen_wave = first + wave * 32 < p.s ? (p.past + (first + wave * 32 + 32 < p.s ? first + wave * 32 + 32 : p.s)) : 0;

    u32x4 q[DT];
    {
        const uint16_t* qr = p.q + (int64_t)(row < p.s ? row : p.s - 1) * p.ldq + (int64_t)h * D;
#pragma unroll
        for (int k = 0; k < DT; k++) {
            const int d = k * 16 + hi * 8;
            if (WHOLE) {
                q[k] = d < D ? *(const u32x4*)(qr + d) : u32x4{0, 0, 0, 0};
                continue;
            }
            uint16_t e[8];
#pragma unroll
            for (int i = 0; i < 8; i++) e[i] = d + i < D ? qr[d + i] : (uint16_t)0;
            __builtin_memcpy(&q[k], e, 16);
        }
    }
    u32x4 kreg[kKeyLoads], vreg[VT];
    auto fetch = [&](int j0) {
#pragma unroll
        for (int n = 0; n < kKeyLoads; n++) {
            const int item = tid + 256 * n, r = item / (DT * 2), d = item % (DT * 2) * 8;
            if (kKeys * DT * 2 % 256 != 0 && item >= kKeys * DT * 2) break;
            const int64_t j = j0 + r < n_keys ? j0 + r : n_keys - 1;  // past the last key: never seen
            const uint16_t* k = p.keys + j * p.ldk + (int64_t)h * p.dim;
            const uint16_t* c = p.cache + j * p.ldc + p.rank - p.dim;
            if (WHOLE) {  // pieces past the last feature meet zeros of q: any finite value does
                kreg[n] = *(const u32x4*)(d < p.dim ? k + d : d < D ? c + d : k);
            } else {
                uint16_t e[8];
#pragma unroll
                for (int i = 0; i < 8; i++) e[i] = d + i < p.dim ? k[d + i] : d + i < D ? c[d + i] : (uint16_t)0;
                __builtin_memcpy(&kreg[n], e, 16);
            }
        }
#pragma unroll
        for (int n = 0; n < VT; n++) {
            const int item = tid + 256 * n, r = item >> 3;
            vreg[n] = *(const u32x4*)(p.vt + ((int64_t)h * p.vdim + (r < p.vdim ? r : p.vdim - 1)) * p.ldv + j0 + (item & 7) * 8);
        }
    };
    auto stage = [&]() {
#pragma unroll
        for (int n = 0; n < kKeyLoads; n++) {
            const int item = tid + 256 * n;
            if (kKeys * DT * 2 % 256 != 0 && item >= kKeys * DT * 2) break;
            *(u32x4*)(ks + item / (DT * 2) * kKey + item % (DT * 2) * 8) = kreg[n];
        }
#pragma unroll
        for (int n = 0; n < VT; n++) {
            const int item = tid + 256 * n;
            *(u32x4*)(vs + (item >> 3) * kVal + (item & 7) * 8) = vreg[n];
        }
    };
    f32x16 o[VT];
#pragma unroll
    for (int t = 0; t < VT; t++)
#pragma unroll
        for (int i = 0; i < 16; i++) o[t][i] = 0.f;
    float m = -__builtin_inff(), l = 0.f;  // the row's maximum (in units of log2); the sum over the keys this half of the lanes holds
    fetch(0);
    for (int j0 = 0; j0 < seen_wg; j0 += kKeys) {
        __syncthreads();  // the tile before has been read
        stage();
        __syncthreads();
        if (j0 + kKeys < seen_wg) fetch(j0 + kKeys);
        if (j0 >= seen_wave) continue;
        f32x16 sc[2];
#pragma unroll
        for (int b = 0; b < 2; b++) {
#pragma unroll
            for (int i = 0; i < 16; i++) sc[b][i] = 0.f;
#pragma unroll
            for (int k = 0; k < DT; k++) sc[b] = mfma_bf16(*(const u32x4*)(ks + (b * 32 + r32) * kKey + k * 16 + hi * 8), q[k], sc[b]);
        }
        const bool whole = j0 + kKeys - 1 <= p.past + first + wave * 32;  // every row of the wavefront sees the whole tile
        float top = -__builtin_inff();
#pragma unroll
        for (int b = 0; b < 2; b++)
#pragma unroll
            for (int i = 0; i < 16; i++) {
                float v = sc[b][i] * p.scale;
                if (!whole && j0 + b * 32 + (i & 3) + 8 * (i >> 2) + 4 * hi > pos) v = -__builtin_inff();
                sc[b][i] = v;
                top = fmaxf(top, v);
            }
        top = fmaxf(top, __shfl_xor(top, 32));
        const float next = fmaxf(m, top);  // a row past the end sees keys too: finite from the first tile on
        if (__any(next > m)) {
            const float back = __builtin_amdgcn_exp2f(m - next);
            l *= back;
#pragma unroll
            for (int t = 0; t < VT; t++)
#pragma unroll
                for (int i = 0; i < 16; i++) o[t][i] *= back;
            m = next;
        }
#pragma unroll
        for (int b = 0; b < 2; b++)
#pragma unroll
            for (int half = 0; half < 2; half++) {
                u32x4 high, low;
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const float x = __builtin_amdgcn_exp2f(sc[b][half * 8 + 2 * i] - m), y = __builtin_amdgcn_exp2f(sc[b][half * 8 + 2 * i + 1] - m);
                    l += x + y;
                    high[i] = pack2(x, y);
                    low[i] = pack2(low_part(x), low_part(y));
                }
#pragma unroll
                for (int t = 0; t < VT; t++) {
                    const uint16_t* v = vs + (t * 32 + r32) * kVal + b * 32 + half * 16 + hi * 4;
                    const u32x2 v0 = *(const u32x2*)v, v1 = *(const u32x2*)(v + 8);
                    const u32x4 a = {v0[0], v0[1], v1[0], v1[1]};
                    o[t] = mfma_bf16(a, high, o[t]);
                    o[t] = mfma_bf16(a, low, o[t]);
                }
            }
    }
    const float inv = 1.f / (l + __shfl_xor(l, 32));
    if (row >= p.s) return;
    uint16_t* out = p.out + (int64_t)row * p.ldo + (int64_t)h * p.vdim;
#pragma unroll
    for (int t = 0; t < VT; t++)
#pragma unroll
        for (int g = 0; g < 4; g++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int e = t * 32 + 8 * g + 4 * hi + i;
                if (e < p.vdim) out[e] = f32_to_bf16_bits(o[t][4 * g + i] * inv);
            }
}

template <int DT, int VT>
void launch_prompt(const PromptArgs& p, hipStream_t st) {
    const dim3 grid((unsigned)p.heads, (unsigned)((p.s + kPromptRows - 1) / kPromptRows));
    const bool whole = p.dim % 8 == 0 && p.rot_dim % 8 == 0 && p.rank % 8 == 0 && p.ldq % 8 == 0 && p.ldk % 8 == 0 && p.ldc % 8 == 0 &&
                       (((uintptr_t)p.q | (uintptr_t)p.keys | (uintptr_t)p.cache) & 15) == 0;
    if (whole) hipLaunchKernelGGL((latent_prompt_kernel<DT, VT, true>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((latent_prompt_kernel<DT, VT, false>), grid, dim3(256), 0, st, p);
}

}  // namespace

hipError_t latent_prepare(const Latent& a, float* proj, int64_t ldp, uint16_t* q_bf16, int64_t ldq, hipStream_t st) {
    if (a.batch * a.s == 0) return hipSuccess;
    hipLaunchKernelGGL(latent_prepare_kernel, dim3((unsigned)(a.batch * a.s)), dim3(256), 0, st, a, proj, ldp, q_bf16, ldq);
    return hipGetLastError();
}

// By the capacity, not by how many positions are held: a recorded step keeps its grid.
int latent_splits(const Latent& a) {
    const int64_t wgs = (int64_t)a.batch * a.s * ((a.heads + kHeads - 1) / kHeads), most = (a.context + kKeys - 1) / kKeys;
    const int64_t want = (512 + wgs - 1) / wgs;
    return (int)(want < most ? want : most);
}

// rows * splits <= rows * (512 / rows + 1)
size_t latent_absorbed_ws_floats(const Latent& a, int64_t rows) {
    return (size_t)rows * a.heads * a.rank + (size_t)(512 + rows) * a.heads * (a.rank + 2);
}

hipError_t latent_absorbed(const Latent& a, const float* proj, int64_t ldp, float* ws, float* out_f32, uint16_t* out_bf16, int64_t ldo, hipStream_t st) {
    const int64_t rows = (int64_t)a.batch * a.s;
    if (rows == 0) return hipSuccess;
    if (a.rank > 1024 || rows > 65535) return hipErrorInvalidValue;
    const int splits = latent_splits(a);
    float* qa = ws;
    float* po = qa + (size_t)rows * a.heads * a.rank;
    float* ml = po + (size_t)rows * splits * a.heads * a.rank;
    hipLaunchKernelGGL(latent_absorb_kernel, dim3((unsigned)rows, (unsigned)a.heads, (unsigned)((a.rank + 255) / 256)), dim3(256), 0, st, a, proj, ldp, qa);
    hipError_t e;
    if (a.cache_bf16)
        e = a.rank <= 256   ? launch_attend<uint16_t, 1>(a, proj, ldp, qa, splits, po, ml, st)
            : a.rank <= 512 ? launch_attend<uint16_t, 2>(a, proj, ldp, qa, splits, po, ml, st)
                            : launch_attend<uint16_t, 4>(a, proj, ldp, qa, splits, po, ml, st);
    else
        e = a.rank <= 256   ? launch_attend<float, 1>(a, proj, ldp, qa, splits, po, ml, st)
            : a.rank <= 512 ? launch_attend<float, 2>(a, proj, ldp, qa, splits, po, ml, st)
                            : launch_attend<float, 4>(a, proj, ldp, qa, splits, po, ml, st);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)rows, (unsigned)a.heads, (unsigned)((a.vdim + kValues - 1) / kValues)), dim3(256),
                       (size_t)((a.rank + 63) / 64 * 64) * 4, st, a, splits, po, ml, out_f32, out_bf16, ldo);
    return hipGetLastError();
}

bool latent_prompt_ok(const Latent& a) {
    return a.cache_bf16 && a.dim + a.rot_dim <= 256 && a.vdim <= 256 && a.past + a.s < 1 << 30 && !a.past_dev;
}

hipError_t latent_prompt(const Latent& a, int sequence, const uint16_t* q, int64_t ldq, const uint16_t* keys, int64_t ldk, const uint16_t* values_t,
                         int64_t ldv, uint16_t* out, int64_t ldo, hipStream_t st) {
    if (a.s == 0) return hipSuccess;
    if (!latent_prompt_ok(a) || ldv % 64 || ((uintptr_t)values_t & 15)) return hipErrorInvalidValue;
    PromptArgs p;
    p.q = q; p.keys = keys; p.vt = values_t; p.cache = (const uint16_t*)a.cache + sequence * a.context * a.ldc; p.out = out;
    p.ldq = ldq; p.ldk = ldk; p.ldv = ldv; p.ldc = a.ldc; p.ldo = ldo;
    p.heads = a.heads; p.dim = a.dim; p.rot_dim = a.rot_dim; p.vdim = a.vdim; p.rank = a.rank;
    p.past = (int)a.past; p.s = (int)a.s;
    p.scale = a.scale * 1.4426950408889634f;
    const int d = a.dim + a.rot_dim, v = a.vdim;
    if (d <= 64 && v <= 64) launch_prompt<4, 2>(p, st);
    else if (d <= 128 && v <= 128) launch_prompt<8, 4>(p, st);
    else if (d <= 192 && v <= 128) launch_prompt<12, 4>(p, st);
    else launch_prompt<16, 8>(p, st);
    return hipGetLastError();
}

}  // namespace mimir
