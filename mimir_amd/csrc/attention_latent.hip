// Latent attention: a head's keys and values are W_uk c and W_uv c of a latent c of `rank`, beside a rotated key part that
// all heads share, and only c and that part are kept (struct Latent, stack_ops.h).
//
// latent_absorbed serves few query rows (a decoding step, a short portion) and everything in float32 without forming
// keys or values: q_h . (W_uk,h c_j) = (W_uk,h^T q_h) . c_j, so a head's query goes to the latents' space once
// (latent_queries_kernel, which also turns the rotated parts and writes the new cache rows) and all heads read the same
// cache rows; the weighted sum of the latents comes back through W_uv,h (latent_combine_kernel). The keys of a row are cut
// into shares that workgroups take side by side, on the vector units (latent_attend_kernel, any sizes, float32 or
// bfloat16 cache) or, for a bfloat16 cache, on the matrix cores (latent_attend_mfma_kernel).
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

// A row's cache entry: the latent over its root mean square times the norm's weight, and the turned key part. 256 threads.
__device__ __forceinline__ void write_cache_row(const Latent& a, const float* low, int64_t b, int64_t pos, const float* cs, const float* sn) {
    __shared__ float part[4];
    float ss = 0.f;
    for (int i = threadIdx.x; i < a.rank; i += 256) ss = fmaf(low[i], low[i], ss);
    ss = block_sum_256(ss, part);
    const float scale = 1.f / __builtin_sqrtf(ss / (float)a.rank + a.eps);
    const int64_t at = (b * a.context + pos) * a.ldc;
    float* c32 = a.cache_bf16 ? nullptr : (float*)a.cache + at;
    uint16_t* c16 = a.cache_bf16 ? (uint16_t*)a.cache + at : nullptr;
    auto keep = [&](int i, float v) {
        if (c32) c32[i] = v;
        else c16[i] = round_bf16(v);
    };
    for (int i = threadIdx.x; i < a.rank; i += 256) keep(i, low[i] * scale * a.norm_w[i]);
    for (int i = threadIdx.x; i < a.rot_dim / 2; i += 256) {
        const float u = low[a.rank + 2 * i], v = low[a.rank + 2 * i + 1];
        keep(a.rank + 2 * i, u * cs[i] - v * sn[i]);
        keep(a.rank + 2 * i + 1, v * cs[i] + u * sn[i]);
    }
}

// For formed keys, one workgroup a row: the cache row, and the queries turned and rounded.
__global__ __launch_bounds__(256) void latent_prepare_kernel(Latent a, const float* __restrict__ proj, int64_t ldp, uint16_t* __restrict__ q16, int64_t ldq) {
    const int64_t r = blockIdx.x, b = r / a.s, pos = past_of(a) + r % a.s;
    const int D = a.dim + a.rot_dim, half = a.rot_dim / 2;
    const float* p = proj + r * ldp;
    const float *cs = a.cos_t + pos * half, *sn = a.sin_t + pos * half;
    write_cache_row(a, p + (int64_t)a.heads * D, b, pos, cs, sn);
    for (int i = threadIdx.x; i < a.heads * half; i += 256) {
        const int h = i / half, j = i % half;
        const int64_t o = (int64_t)h * D + a.dim + 2 * j;
        const float u = p[o], v = p[o + 1];
        q16[r * ldq + o] = round_bf16(u * cs[j] - v * sn[j]);
        q16[r * ldq + o + 1] = round_bf16(v * cs[j] + u * sn[j]);
    }
    for (int i = threadIdx.x; i < a.heads * a.dim; i += 256) {
        const int64_t o = (int64_t)(i / a.dim) * D + i % a.dim;
        q16[r * ldq + o] = round_bf16(p[o]);
    }
}

constexpr int kAbsorbCols = 128;  // latent features a workgroup

__device__ __forceinline__ int query_ld(const Latent& a) { return (a.rank + a.rot_dim + 31) / 32 * 32; }

// Without formed keys: qa[row, h, :] = (W_uk,h^T q_h | the turned part) * scale, zeros up to query_ld. Workgroups (row, h, z):
// 128 latent features each, eight a thread, the head's rows of W_uk shared by sixteen groups; those of head 0's first
// piece also write the row's cache entry.
__global__ __launch_bounds__(256) void latent_queries_kernel(Latent a, const float* __restrict__ proj, int64_t ldp, float* __restrict__ qa) {
    __shared__ float red[16][kAbsorbCols + 4];
    const int64_t r = blockIdx.x, pos = past_of(a) + r % a.s;
    const int h = blockIdx.y, half = a.rot_dim / 2, D = a.dim + a.rot_dim, lq = query_ld(a);
    const int c0 = blockIdx.z * kAbsorbCols + (threadIdx.x & 15) * 8, g = threadIdx.x >> 4;
    const float *cs = a.cos_t + pos * half, *sn = a.sin_t + pos * half;
    const float* q = proj + r * ldp + (int64_t)h * D;
    float* to = qa + (r * a.heads + h) * lq;
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (c0 < a.rank) {
        const uint16_t* w0 = a.w_uk + (int64_t)h * a.dim * a.ldw + c0;  // rows are padded with zeros
#pragma unroll 4
        for (int d = g; d < a.dim; d += 16) {
            const u32x4 w = *(const u32x4*)(w0 + (int64_t)d * a.ldw);
            const float x = q[d];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                acc[2 * i] = fmaf(x, __uint_as_float(w[i] << 16), acc[2 * i]);
                acc[2 * i + 1] = fmaf(x, __uint_as_float(w[i] & 0xffff0000u), acc[2 * i + 1]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < 8; i++) red[g][(threadIdx.x & 15) * 8 + i] = acc[i];
    __syncthreads();
    const int c = blockIdx.z * kAbsorbCols + threadIdx.x;
    if (threadIdx.x < kAbsorbCols && c < a.rank) {
        float v = 0.f;
#pragma unroll
        for (int i = 0; i < 16; i++) v += red[i][threadIdx.x];
        to[c] = v * a.scale;
    }
    if (blockIdx.z == 0) {
        for (int i = threadIdx.x; i < half; i += 256) {
            const float u = q[a.dim + 2 * i], v = q[a.dim + 2 * i + 1];
            to[a.rank + 2 * i] = (u * cs[i] - v * sn[i]) * a.scale;
            to[a.rank + 2 * i + 1] = (v * cs[i] + u * sn[i]) * a.scale;
        }
        for (int i = a.rank + a.rot_dim + threadIdx.x; i < lq; i += 256) to[i] = 0.f;
        if (h == 0) write_cache_row(a, proj + r * ldp + (int64_t)a.heads * D, r / a.s, pos, cs, sn);  // the whole workgroup
    }
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

// How many of a row's keys a share has: whole tiles.
__device__ __forceinline__ int64_t share_of(int64_t seen, int splits) {
    const int64_t share = (seen + splits - 1) / splits;
    return (share + kKeys - 1) / kKeys * kKeys;
}

// The share `split` of the keys of one row, for kHeads heads: scores with a lane's key against four heads a
// wavefront, a running softmax, and the weighted sum of the latents with a thread's columns tid + 256 u.
// parts: [rows, splits, heads, rank] sums, then [rows, splits, heads, 2] (maximum, sum of weights).
template <typename T, int U>
__global__ __launch_bounds__(256) void latent_attend_kernel(Latent a, const float* __restrict__ qa, int splits, float* __restrict__ part_o,
                                                            float* __restrict__ part_ml) {
    extern __shared__ __align__(16) float lds_latent[];
    const int L8 = (a.rank + a.rot_dim + 7) / 8 * 8;
    float* qs = lds_latent;                    // [L8][kHeads]
    float* ps = qs + (size_t)L8 * kHeads;      // [kKeys][kHeads]: scores, then weights
    float* ml = ps + kKeys * kHeads;           // [kHeads] rescaling of this tile
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int split = blockIdx.x, h0 = blockIdx.y * kHeads;
    const int64_t r = blockIdx.z, b = r / a.s;
    const int64_t seen = past_of(a) + r % a.s + 1;
    const int64_t share = share_of(seen, splits);
    const int64_t lo = split * share, hi = lo + share < seen ? lo + share : seen;
    const int64_t pr = (r * splits + split) * a.heads;
    if (lo >= hi) return;  // the whole workgroup: latent_combine_kernel does not look at this share
    for (int i = tid; i < L8 * kHeads; i += 256) {
        const int d = i / kHeads, h = h0 + i % kHeads;
        qs[i] = h < a.heads ? qa[(r * a.heads + h) * query_ld(a) + d] : 0.f;
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

// The same on the matrix cores, a bfloat16 cache: tiles of 64 keys in LDS, 32 heads a workgroup. Scores: the eight
// wavefronts cut the features (KS steps of 32 each), queries as the sum of two bfloat16 in registers, and the partial
// sums meet in LDS, where sixteen threads a head do the softmax. Sum of latents: the wavefronts cut the latent's features
// (RT tiles of sixteen each), weights as the sum of two bfloat16.
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

__device__ __forceinline__ f32x4 mfma16_bf16(u32x4 a, u32x4 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

constexpr int kMHeads = 32, kMWaves = 8;
constexpr int kScoreLd = kMHeads + 1, kWeightLd = kKeys + 8;

// Features of a tile's row in LDS: a constant, so that the addresses of a column are one register and immediate offsets.
int attend_mfma_row(const Latent& a) {
    const int n = a.rank + a.rot_dim;
    return n <= 128 ? 128 : n <= 256 ? 256 : n <= 576 ? 576 : 640;
}
constexpr size_t attend_mfma_lds(int lq) {
    return (size_t)kKeys * (lq + 8) * 2 + (size_t)kMWaves * kKeys * kScoreLd * 4 + (size_t)2 * kMHeads * kWeightLd * 2 + kMHeads * 4;
}
static_assert(attend_mfma_lds(640) <= 160 * 1024, "a compute unit's LDS");

template <int LQ>
__global__ __launch_bounds__(64 * kMWaves) void latent_attend_mfma_kernel(Latent a, const float* __restrict__ qa, int splits, float* __restrict__ part_o,
                                                                              float* __restrict__ part_ml) {
    extern __shared__ __align__(16) float lds_latent[];
    constexpr int ldt = LQ + 8, steps = LQ / 32, KS = (steps + kMWaves - 1) / kMWaves, RT = LQ <= 128 ? 1 : LQ <= 256 ? 2 : 4;
    const int lq = query_ld(a), L = a.rank + a.rot_dim;
    float* ps = lds_latent;                                    // [kMWaves][kKeys][kScoreLd]
    float* back = ps + kMWaves * kKeys * kScoreLd;             // [kMHeads]
    uint16_t* tile = (uint16_t*)(back + kMHeads);              // [kKeys][ldt]
    uint16_t* wH = tile + (size_t)kKeys * ldt;                 // [kMHeads][kWeightLd], high parts
    uint16_t* wL = wH + kMHeads * kWeightLd;                   // low parts
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int split = blockIdx.x, h0 = blockIdx.y * kMHeads;
    const int64_t r = blockIdx.z, b = r / a.s;
    const int64_t seen = past_of(a) + r % a.s + 1, share = share_of(seen, splits);
    const int64_t lo = split * share, hi = lo + share < seen ? lo + share : seen;
    const int64_t pr = (r * splits + split) * a.heads;
    if (lo >= hi) return;  // the whole workgroup: latent_combine_kernel does not look at this share
    const uint16_t* cache = (const uint16_t*)a.cache + b * a.context * a.ldc;
    // a tile's pieces of 16 bytes, this thread's: all requested at once, the first tile's before the queries
    constexpr int pieces = LQ / 8, kPieces = kKeys * pieces / (64 * kMWaves);
    auto each_piece = [&](auto body) {
#pragma unroll
        for (int u = 0; u < kPieces; u++) {
            const int i = tid + 64 * kMWaves * u;
            body(u, i / pieces, i % pieces * 8);
        }
    };
    u32x4 piece[kPieces];
    auto fetch = [&](int64_t j0) {
        each_piece([&](int u, int j, int d) {
            const int64_t row = j0 + j < hi ? j0 + j : hi - 1;
            piece[u] = u32x4{0, 0, 0, 0};
            if (d < L) piece[u] = *(const u32x4*)(cache + row * a.ldc + d);  // a row is padded with zeros to a multiple of 8
        });
    };
    fetch(lo);
    // this wavefront's steps of the features: wave, wave + kMWaves, ...
    u32x4 qh[KS][2], ql[KS][2];
#pragma unroll
    for (int i = 0; i < KS; i++)
#pragma unroll
        for (int t = 0; t < 2; t++) {
            const int h = h0 + t * 16 + r16, step = wave + kMWaves * i;
            f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = x;
            if (h < a.heads && step * 32 < lq) {
                const f32x4* q = (const f32x4*)(qa + (r * a.heads + h) * lq + step * 32 + g * 8);
                x = q[0];
                y = q[1];
            }
            qh[i][t] = u32x4{pack_bf16(x[0], x[1]), pack_bf16(x[2], x[3]), pack_bf16(y[0], y[1]), pack_bf16(y[2], y[3])};
            ql[i][t] = u32x4{pack_bf16(low_part(x[0]), low_part(x[1])), pack_bf16(low_part(x[2]), low_part(x[3])), pack_bf16(low_part(y[0]), low_part(y[1])),
                             pack_bf16(low_part(y[2]), low_part(y[3]))};
        }
    f32x4 acc[RT][2];
#pragma unroll
    for (int t = 0; t < RT; t++)
#pragma unroll
        for (int i = 0; i < 2; i++) acc[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int sh = tid >> 4, sk = tid & 15;  // the softmax's head and first key of this thread
    float m = -__builtin_inff(), l = 0.f;
    for (int64_t j0 = lo; j0 < hi; j0 += kKeys) {
        each_piece([&](int u, int j, int d) {
            *(u32x4*)(tile + j * ldt + d) = piece[u];
        });
        __syncthreads();
        if (j0 + kKeys < hi) fetch(j0 + kKeys);
        f32x4 sc[4][2];
#pragma unroll
        for (int k = 0; k < 4; k++)
#pragma unroll
            for (int t = 0; t < 2; t++) sc[k][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < KS; i++) {
            const int step = wave + kMWaves * i;
            if (step >= steps) break;
#pragma unroll
            for (int k = 0; k < 4; k++) {
                const u32x4 c = *(const u32x4*)(tile + (k * 16 + r16) * ldt + step * 32 + g * 8);
#pragma unroll
                for (int t = 0; t < 2; t++) {
                    sc[k][t] = mfma16_bf16(c, qh[i][t], sc[k][t]);
                    sc[k][t] = mfma16_bf16(c, ql[i][t], sc[k][t]);
                }
            }
        }
#pragma unroll
        for (int k = 0; k < 4; k++)
#pragma unroll
            for (int t = 0; t < 2; t++)
#pragma unroll
                for (int i = 0; i < 4; i++) ps[(wave * kKeys + k * 16 + 4 * g + i) * kScoreLd + t * 16 + r16] = sc[k][t][i];
        __syncthreads();
        {
            float s[4], top = -__builtin_inff();
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int j = sk * 4 + i;
                float v = 0.f;
#pragma unroll
                for (int w = 0; w < kMWaves; w++) v += ps[(w * kKeys + j) * kScoreLd + sh];
                s[i] = j0 + j < hi ? v : -__builtin_inff();
                top = fmaxf(top, s[i]);
            }
            top = group8_max(top);
            top = fmaxf(top, __shfl_xor(top, 8));
            const float next = fmaxf(m, top), scale = expf(m - next);  // the first tile's m: exp(-inf) = 0
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < 4; i++) {
                s[i] = expf(s[i] - next);
                sum += s[i];
            }
            *(u32x2*)(wH + sh * kWeightLd + sk * 4) = u32x2{pack_bf16(s[0], s[1]), pack_bf16(s[2], s[3])};
            *(u32x2*)(wL + sh * kWeightLd + sk * 4) = u32x2{pack_bf16(low_part(s[0]), low_part(s[1])), pack_bf16(low_part(s[2]), low_part(s[3]))};
            sum = group8_sum(sum);
            l = l * scale + (sum + __shfl_xor(sum, 8));
            m = next;
            if (sk == 0) back[sh] = scale;
        }
        __syncthreads();
        if (j0 > lo)
#pragma unroll
            for (int t = 0; t < 2; t++) {
                const f32x4 f = *(const f32x4*)(back + t * 16 + 4 * g);
#pragma unroll
                for (int k = 0; k < RT; k++) acc[k][t] = acc[k][t] * f;
            }
#pragma unroll
        for (int half = 0; half < 2; half++) {
            u32x4 pw[2][2];
#pragma unroll
            for (int t = 0; t < 2; t++) {
                pw[t][0] = *(const u32x4*)(wH + (t * 16 + r16) * kWeightLd + half * 32 + g * 8);
                pw[t][1] = *(const u32x4*)(wL + (t * 16 + r16) * kWeightLd + half * 32 + g * 8);
            }
#pragma unroll
            for (int k = 0; k < RT; k++) {
                const int c0 = (wave + kMWaves * k) * 16;
                if (c0 >= a.rank) break;
                // eight keys of one feature: a column of the tile (features past the rank are the rotated part or zeros: not stored)
                const uint16_t* col = tile + (half * 32 + g * 8) * ldt + c0 + r16;
                u32x4 v;
#pragma unroll
                for (int i = 0; i < 4; i++) v[i] = (uint32_t)col[2 * i * ldt] | (uint32_t)col[(2 * i + 1) * ldt] << 16;
#pragma unroll
                for (int t = 0; t < 2; t++) {
                    acc[k][t] = mfma16_bf16(pw[t][0], v, acc[k][t]);
                    acc[k][t] = mfma16_bf16(pw[t][1], v, acc[k][t]);
                }
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int k = 0; k < RT; k++) {
        const int c = (wave + kMWaves * k) * 16 + r16;
#pragma unroll
        for (int t = 0; t < 2; t++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int h = h0 + t * 16 + 4 * g + i;
                if (c < a.rank && h < a.heads) part_o[(pr + h) * a.rank + c] = acc[k][t][i];
            }
    }
    if (sk == 0 && h0 + sh < a.heads) {
        part_ml[(pr + h0 + sh) * 2] = m;
        part_ml[(pr + h0 + sh) * 2 + 1] = l;
    }
}

constexpr int kValues = 64;      // values a workgroup of latent_combine_kernel
constexpr int kMaxSplits = 512;

// The shares of a head brought together, then its values: out[row, h, e] = W_uv[h, e, :] . (sum of latents).
__global__ __launch_bounds__(256) void latent_combine_kernel(Latent a, int splits, const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                                             float* __restrict__ out_f32, uint16_t* __restrict__ out_bf16, int64_t ldo) {
    extern __shared__ __align__(16) float lds_latent[];
    __shared__ float weight[kMaxSplits];
    float* oc = lds_latent;  // [rank to a multiple of 64]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.y;
    const int64_t r = blockIdx.x;
    const int R64 = (a.rank + 63) / 64 * 64;
    const int64_t seen = past_of(a) + r % a.s + 1, share = share_of(seen, splits);
    const int live = (int)((seen + share - 1) / share);  // shares that have keys
    const float* mlp = part_ml + (r * splits * a.heads + h) * 2;
    const int64_t step = (int64_t)a.heads * 2;
    if (wave == 0) {
        float top = -__builtin_inff();
        for (int s = lane; s < live; s += 64) top = fmaxf(top, mlp[s * step]);
        top = wave_max(top);
        float sum = 0.f;
        for (int s = lane; s < live; s += 64) {
            const float w = expf(mlp[s * step] - top);
            weight[s] = w;
            sum = fmaf(mlp[s * step + 1], w, sum);
        }
        const float inv = 1.f / wave_sum(sum);
        for (int s = lane; s < live; s += 64) weight[s] *= inv;
    }
    __syncthreads();
    const float* po = part_o + (r * splits * a.heads + h) * a.rank;
    const int64_t ostep = (int64_t)a.heads * a.rank;
    for (int c = tid; c < R64; c += 256) {
        float v = 0.f;
        if (c < a.rank) {
#pragma unroll 8
            for (int s = 0; s < live; s++) v = fmaf(po[s * ostep + c], weight[s], v);
        }
        oc[c] = v;
    }
    __syncthreads();
    const int e0 = blockIdx.z * kValues, e1 = e0 + kValues < a.vdim ? e0 + kValues : a.vdim;
    const uint16_t* w0 = a.w_uv + (int64_t)h * a.vdim * a.ldw;
    for (int e = e0 + wave * 4; e < e1; e += 16) {  // four values a wavefront at a time
        float v[4] = {0.f, 0.f, 0.f, 0.f};
        for (int c = lane * 8; c < R64; c += 512) {
            u32x4 x[4];
#pragma unroll
            for (int u = 0; u < 4; u++) x[u] = *(const u32x4*)(w0 + (int64_t)(e + u < e1 ? e + u : e1 - 1) * a.ldw + c);
#pragma unroll
            for (int u = 0; u < 4; u++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    v[u] = fmaf(oc[c + 2 * i], __uint_as_float(x[u][i] << 16), v[u]);
                    v[u] = fmaf(oc[c + 2 * i + 1], __uint_as_float(x[u][i] & 0xffff0000u), v[u]);
                }
        }
#pragma unroll
        for (int u = 0; u < 4; u++) {
            const float sum = wave_sum(v[u]);
            if (lane == 0 && e + u < e1) {
                const int64_t at = r * ldo + (int64_t)h * a.vdim + e + u;
                if (out_f32) out_f32[at] = sum;
                else out_bf16[at] = round_bf16(sum);
            }
        }
    }
}

template <typename T, int U>
hipError_t launch_attend(const Latent& a, const float* qa, int splits, float* po, float* ml, hipStream_t st) {
    const size_t lds = ((size_t)(a.rank + a.rot_dim + 7) / 8 * 8 * kHeads + kKeys * kHeads + kHeads) * 4;
    if (lds > 64 * 1024) {
        hipError_t e = hipFuncSetAttribute((const void*)latent_attend_kernel<T, U>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    const dim3 grid((unsigned)splits, (unsigned)((a.heads + kHeads - 1) / kHeads), (unsigned)(a.batch * a.s));
    hipLaunchKernelGGL((latent_attend_kernel<T, U>), grid, dim3(256), lds, st, a, qa, splits, po, ml);
    return hipGetLastError();
}

template <int LQ>
hipError_t launch_attend_mfma(const Latent& a, const float* qa, int splits, float* po, float* ml, hipStream_t st) {
    constexpr size_t lds = attend_mfma_lds(LQ);
    hipError_t e = hipFuncSetAttribute((const void*)latent_attend_mfma_kernel<LQ>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
    const dim3 grid((unsigned)splits, (unsigned)((a.heads + kMHeads - 1) / kMHeads), (unsigned)(a.batch * a.s));
    hipLaunchKernelGGL(latent_attend_mfma_kernel<LQ>, grid, dim3(64 * kMWaves), lds, st, a, qa, splits, po, ml);
    return hipGetLastError();
}

bool attend_mfma_ok(const Latent& a) { return a.cache_bf16 && a.rank <= 512 && a.rank + a.rot_dim <= 640 && a.ldc % 8 == 0; }

// ---- many query rows ------------------------------------------------------------------------
// A wavefront owns 32 query rows of one head and walks the keys in tiles of 64 with a running maximum and sum per row.
// Both products are computed transposed (scores^T = K Q^T, result^T = V^T P^T), so that a row's scores and results lie in
// one lane and its partner 32 lanes on, and the weights go from the exponential straight into the second product's
// operand: the order in which the scores' registers hold the keys is the order in which V^T's fragment is read. Four
// wavefronts with consecutive rows share a tile of keys and values in LDS; the next tile is requested while one is used.

__device__ __forceinline__ f32x16 mfma_bf16(u32x4 a, u32x4 b, f32x16 c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

struct PromptArgs {
    const uint16_t *q, *keys, *vt, *cache;
    uint16_t* out;
    int64_t ldq, ldk, ldv, ldc, ldo, context;
    int heads, dim, rot_dim, vdim, rank;
    int past, s, batch;
    int fold;
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
    // the last rows first: they see the most keys. Where all workgroups fit the device at once, two a compute unit, the
    // second half goes the other way, so that long ones and short ones share a unit.
    const int h = blockIdx.x, nb = gridDim.y, by = blockIdx.y;
    const int first = (p.fold && by >= (nb + 1) / 2 ? by - (nb + 1) / 2 : nb - 1 - by) * kPromptRows;
    const int64_t seq = blockIdx.z;
    p.q += seq * p.s * p.ldq;
    p.keys += seq * p.context * p.ldk;
    p.vt += seq * p.context;
    p.cache += seq * p.context * p.ldc;
    p.out += seq * p.s * p.ldo;
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
                    high[i] = pack_bf16(x, y);
                    low[i] = pack_bf16(low_part(x), low_part(y));
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
                if (e < p.vdim) out[e] = round_bf16(o[t][4 * g + i] * inv);
            }
}

template <int DT, int VT>
void launch_prompt(PromptArgs p, hipStream_t st) {
    const dim3 grid((unsigned)p.heads, (unsigned)((p.s + kPromptRows - 1) / kPromptRows), (unsigned)p.batch);
    p.fold = (int64_t)grid.x * grid.y * grid.z <= 512;
    const bool whole = p.dim % 8 == 0 && p.rot_dim % 8 == 0 && p.rank % 8 == 0 && p.ldq % 8 == 0 && p.ldk % 8 == 0 && p.ldc % 8 == 0 &&
                       (((uintptr_t)p.q | (uintptr_t)p.keys | (uintptr_t)p.cache) & 15) == 0;
    if (whole) hipLaunchKernelGGL((latent_prompt_kernel<DT, VT, true>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((latent_prompt_kernel<DT, VT, false>), grid, dim3(256), 0, st, p);
}

}  // namespace

hipError_t latent_prepare(const Latent& a, const float* proj, int64_t ldp, uint16_t* q_bf16, int64_t ldq, hipStream_t st) {
    if (a.batch * a.s == 0) return hipSuccess;
    hipLaunchKernelGGL(latent_prepare_kernel, dim3((unsigned)(a.batch * a.s)), dim3(256), 0, st, a, proj, ldp, q_bf16, ldq);
    return hipGetLastError();
}

// By the capacity, not by how many positions are held: a recorded step keeps its grid.
int latent_splits(const Latent& a) {
    const int heads = attend_mfma_ok(a) ? kMHeads : kHeads;
    const int64_t wgs = (int64_t)a.batch * a.s * ((a.heads + heads - 1) / heads), most = (a.context + kKeys - 1) / kKeys;
    const int64_t want = (kMaxSplits + wgs - 1) / wgs;
    return (int)(want < most ? want : most);
}

// rows * splits <= rows * (kMaxSplits / rows + 1)
size_t latent_absorbed_ws_floats(const Latent& a, int64_t rows) {
    return (size_t)rows * a.heads * ((a.rank + a.rot_dim + 31) / 32 * 32) + (size_t)(kMaxSplits + rows) * a.heads * (a.rank + 2);
}

hipError_t latent_absorbed(const Latent& a, const float* proj, int64_t ldp, float* ws, float* out_f32, uint16_t* out_bf16, int64_t ldo, hipStream_t st) {
    const int64_t rows = (int64_t)a.batch * a.s;
    if (rows == 0) return hipSuccess;
    if (a.rank > 1024 || rows > 65535) return hipErrorInvalidValue;
    const int splits = latent_splits(a);
    float* qa = ws;
    float* po = qa + (size_t)rows * a.heads * ((a.rank + a.rot_dim + 31) / 32 * 32);
    float* ml = po + (size_t)rows * splits * a.heads * a.rank;
    hipLaunchKernelGGL(latent_queries_kernel, dim3((unsigned)rows, (unsigned)a.heads, (unsigned)((a.rank + kAbsorbCols - 1) / kAbsorbCols)), dim3(256), 0, st, a,
                       proj, ldp, qa);
    hipError_t e;
    const int row = attend_mfma_row(a);
    if (attend_mfma_ok(a))
        e = row == 128   ? launch_attend_mfma<128>(a, qa, splits, po, ml, st)
            : row == 256 ? launch_attend_mfma<256>(a, qa, splits, po, ml, st)
            : row == 576 ? launch_attend_mfma<576>(a, qa, splits, po, ml, st)
                         : launch_attend_mfma<640>(a, qa, splits, po, ml, st);
    else if (a.cache_bf16)
        e = a.rank <= 256   ? launch_attend<uint16_t, 1>(a, qa, splits, po, ml, st)
            : a.rank <= 512 ? launch_attend<uint16_t, 2>(a, qa, splits, po, ml, st)
                            : launch_attend<uint16_t, 4>(a, qa, splits, po, ml, st);
    else
        e = a.rank <= 256   ? launch_attend<float, 1>(a, qa, splits, po, ml, st)
            : a.rank <= 512 ? launch_attend<float, 2>(a, qa, splits, po, ml, st)
                            : launch_attend<float, 4>(a, qa, splits, po, ml, st);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)rows, (unsigned)a.heads, (unsigned)((a.vdim + kValues - 1) / kValues)), dim3(256),
                       (size_t)((a.rank + 63) / 64 * 64) * 4, st, a, splits, po, ml, out_f32, out_bf16, ldo);
    return hipGetLastError();
}

bool latent_prompt_ok(const Latent& a) {
    return a.cache_bf16 && a.dim + a.rot_dim <= 256 && a.vdim <= 256 && a.past + a.s < 1 << 30 && !a.past_dev;
}

hipError_t latent_prompt(const Latent& a, const uint16_t* q, int64_t ldq, const uint16_t* keys, int64_t ldk, const uint16_t* values_t, int64_t ldv,
                         uint16_t* out, int64_t ldo, hipStream_t st) {
    if (a.batch * a.s == 0) return hipSuccess;
    if (!latent_prompt_ok(a) || ldv % 8 || a.context % 64 || ((uintptr_t)values_t & 15)) return hipErrorInvalidValue;
    PromptArgs p;
    p.q = q; p.keys = keys; p.vt = values_t; p.cache = (const uint16_t*)a.cache; p.out = out;
    p.ldq = ldq; p.ldk = ldk; p.ldv = ldv; p.ldc = a.ldc; p.ldo = ldo; p.context = a.context;
    p.heads = a.heads; p.dim = a.dim; p.rot_dim = a.rot_dim; p.vdim = a.vdim; p.rank = a.rank;
    p.past = (int)a.past; p.s = (int)a.s; p.batch = a.batch; p.fold = 0;
    p.scale = a.scale * 1.4426950408889634f;
    const int d = a.dim + a.rot_dim, v = a.vdim;
    if (d <= 64 && v <= 64) launch_prompt<4, 2>(p, st);
    else if (d <= 128 && v <= 128) launch_prompt<8, 4>(p, st);
    else if (d <= 192 && v <= 128) launch_prompt<12, 4>(p, st);
    else launch_prompt<16, 8>(p, st);
    return hipGetLastError();
}

}  // namespace mimir
