// Attention whose keys and values are kept for every key head (struct HeadAttention, stack_ops.h): query heads share key
// heads in groups, and each of these is a parameter: queries and keys over their root mean square, a rotation of the first
// features, a soft cap of the scores, values mixed with those of an earlier layer, a gate a head.
//
// Keys lie as rows of features, values as rows of positions (transposed), in runs of sixteen positions whose middle two
// quarters are exchanged: the order in which a lane of the matrix core's 32 x 32 result holds the scores, so that
// heads_prompt_kernel reads its second product's operand in whole pieces. value_slot is that order.
//
// Few query rows (a decoding step, a short portion, everything in float32) cut the keys into shares that workgroups take
// side by side, on the matrix cores (heads_attend_kernel; in a decoding step it also turns the new queries and keys and
// writes the cache) or on the vector units for any sizes and float32 (heads_attend_any_kernel); heads_combine_kernel
// brings the shares together. Prompts go through heads_prompt_kernel behind heads_prepare_kernel.
#include "gemm_nt_tile.h"
#include "kernels.h"
#include "stack_ops.h"

namespace mimir {

namespace {

constexpr int kKeys = 64;   // keys a tile
constexpr int kHeads = 8;   // heads of a group that a workgroup of few rows takes
constexpr int kMaxSplits = 512;

__device__ __forceinline__ int value_slot(int p) { return (p & ~12) | ((p & 4) << 1) | ((p & 8) >> 1); }
__device__ __forceinline__ int64_t past_of(const HeadAttention& a) { return a.past + (a.past_dev ? *a.past_dev : 0); }
__device__ __forceinline__ float soft_cap(float s, float cap) { return cap > 0.f ? cap * tanhf(s / cap) : s; }
__device__ __forceinline__ float sigmoid_f32(float z) { return 1.f / (1.f + expf(-z)); }

// A wavefront's head of a query or key row: each(i, value) for the features that this lane has, turned and over the root
// mean square where that is asked for.
template <class F>
__device__ __forceinline__ void head_features(const HeadAttention& a, const float* x, int64_t pos, F each) {
    const int lane = threadIdx.x & 63, half = a.rot_dim >> 1;
    float scale = 1.f;
    if (a.unit) {
        float ss = 0.f;
        for (int i = lane; i < a.dim; i += 64) ss = fmaf(x[i], x[i], ss);
        scale = 1.f / __builtin_sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
    }
    for (int i = lane; i < a.dim; i += 64) {
        float v = x[i] * scale;
        if (i < 2 * half) {
            const int j = i < half ? i : i - half;
            const float cs = a.cos_t[pos * half + j], sn = a.sin_t[pos * half + j], other = x[i < half ? i + half : i - half] * scale;
            v = i < half ? v * cs - other * sn : v * cs + other * sn;
        }
        each(i, v);
    }
}

__device__ __forceinline__ float mixed_with(float own, float first, float mix) { return fmaf(mix, first, (1.f - mix) * own); }

// The value that a position keeps, of feature c of all value features; what later layers mix in is kept beside.
__device__ __forceinline__ float mixed_value(const HeadAttention& a, int64_t row, int c) {
    const int64_t vn = (int64_t)a.kv_heads * a.vdim;
    float v = a.proj[row * a.ldp + (int64_t)(a.heads + a.kv_heads) * a.dim + c];
    if (a.first_out) a.first_out[row * vn + c] = v;
    if (a.first) v = mixed_with(v, a.first[row * vn + c], *a.mix);
    return v;
}
__device__ __forceinline__ void keep(void* cache, bool bf16, int64_t at, float v) {
    if (bf16) ((uint16_t*)cache)[at] = round_bf16(v);
    else ((float*)cache)[at] = v;
}
__device__ __forceinline__ int64_t key_row(const HeadAttention& a, int64_t b, int hk, int64_t pos) { return ((b * a.kv_heads + hk) * a.context + pos) * a.ldk; }
__device__ __forceinline__ int64_t value_row(const HeadAttention& a, int64_t b, int hk, int e) { return ((b * a.kv_heads + hk) * a.vdim + e) * a.context; }
__device__ __forceinline__ float gate_of(const HeadAttention& a, int64_t row, int h) {
    return a.gated ? sigmoid_f32(a.proj[row * a.ldp + (int64_t)(a.heads + a.kv_heads) * a.dim + (int64_t)a.kv_heads * a.vdim + h]) : 1.f;
}

// The same of a head on LANES lanes, four neighbouring features a lane (head_fours_ok): put(i, features i .. i + 3).
template <int LANES, class F>
__device__ __forceinline__ void head_fours(const HeadAttention& a, const float* x, int64_t pos, F put) {
    const int i = (threadIdx.x & (LANES - 1)) * 4, half = a.rot_dim >> 1;
    const bool in = i < a.dim, turns = i < a.rot_dim;
    f32x4 v = {0.f, 0.f, 0.f, 0.f}, other = v, cs = v, sn = v;
    if (in) v = *(const f32x4*)(x + i);
    if (turns) {
        const int j = i < half ? i : i - half;
        other = *(const f32x4*)(x + (i < half ? i + half : i - half));
        cs = *(const f32x4*)(a.cos_t + pos * half + j);
        sn = *(const f32x4*)(a.sin_t + pos * half + j);
    }
    float scale = 1.f;
    if (a.unit) {
        float ss = fmaf(v[0], v[0], fmaf(v[1], v[1], fmaf(v[2], v[2], v[3] * v[3])));
#pragma unroll
        for (int d = LANES / 2; d > 0; d >>= 1) ss += __shfl_xor(ss, d);
        scale = 1.f / __builtin_sqrtf(ss / (float)a.dim + a.eps);
    }
    v = v * scale;
    if (turns) {
        other = other * (i < half ? -scale : scale);
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] = v[e] * cs[e] + other[e] * sn[e];
    }
    if (i < a.ldk) put(i, v);  // zeros behind the last feature
}
bool head_fours_ok(const HeadAttention& a) {
    return a.dim % 4 == 0 && a.dim <= 256 && a.rot_dim % 8 == 0 && a.ldp % 4 == 0 && ((uintptr_t)a.proj & 15) == 0;
}

__device__ __forceinline__ u32x2 pack_four(f32x4 v) { return u32x2{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3])}; }

// The cache entries of all new positions, and the queries times q_scale: as bfloat16 rows of heads * ldk for
// heads_prompt_kernel (zeros behind a head's features), or as float32, [rows, heads, dim]. The first workgroups take queries and keys,
// 256 / LANES heads of a row each (LANES 0: a head a wavefront, any size); the others 64 positions of 64 value features,
// which change places through LDS.
template <int LANES>
__global__ __launch_bounds__(256) void heads_prepare_kernel(HeadAttention a, uint16_t* __restrict__ q16, float* __restrict__ q32, float q_scale) {
    __shared__ float tile[64][65];
    constexpr int kAtOnce = LANES ? 256 / LANES : 4;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int units = a.heads + a.kv_heads, chunks = (units + kAtOnce - 1) / kAtOnce;
    const int64_t rows = a.batch * a.s;
    if ((int64_t)blockIdx.x < rows * chunks) {
        const int64_t r = blockIdx.x / chunks, b = r / a.s, pos = past_of(a) + r % a.s;
        const int u = (int)(blockIdx.x % chunks) * kAtOnce + (int)threadIdx.x / (LANES ? LANES : 64);
        if (u >= units) return;  // whole groups of lanes
        const float* x = a.proj + r * a.ldp + (int64_t)u * a.dim;
        const int64_t key = u < a.heads ? 0 : key_row(a, b, u - a.heads, pos), query = r * a.heads + u;
        if constexpr (LANES > 0) {
            head_fours<LANES>(a, x, pos, [&](int i, f32x4 v) {
                if (u >= a.heads) {
                    if (a.cache_bf16) *(u32x2*)((uint16_t*)a.keys + key + i) = pack_four(v);
                    else *(f32x4*)((float*)a.keys + key + i) = v;
                } else if (q16) {
                    *(u32x2*)(q16 + query * a.ldk + i) = pack_four(v * q_scale);
                } else if (i < a.dim) {
                    *(f32x4*)(q32 + query * a.dim + i) = v * q_scale;
                }
            });
        } else {
            head_features(a, x, pos, [&](int i, float v) {
                if (u >= a.heads) keep(a.keys, a.cache_bf16, key + i, v);
                else if (q16) q16[query * a.ldk + i] = round_bf16(v * q_scale);
                else q32[query * a.dim + i] = v * q_scale;
            });
            if (u < a.heads && q16)
                for (int i = a.dim + lane; i < a.ldk; i += 64) q16[query * a.ldk + i] = 0;
        }
        return;
    }
    const int vn = a.kv_heads * a.vdim, cols = (vn + 63) / 64;
    const int64_t w = blockIdx.x - rows * chunks, runs = (a.s + 63) / 64;
    const int c = (int)(w % cols) * 64 + lane;
    const int64_t b = w / cols / runs, t0 = w / cols % runs * 64, r0 = b * a.s + t0;
    const float* from = a.proj + (int64_t)(a.heads + a.kv_heads) * a.dim;
    float own[16], first[16];
    auto in = [&](int u) { return t0 + wave + 4 * u < a.s && c < vn; };
#pragma unroll
    for (int u = 0; u < 16; u++) own[u] = in(u) ? from[(r0 + wave + 4 * u) * a.ldp + c] : 0.f;
    if (a.first) {
#pragma unroll
        for (int u = 0; u < 16; u++) first[u] = in(u) ? a.first[(r0 + wave + 4 * u) * vn + c] : 0.f;
        const float mix = *a.mix;
#pragma unroll
        for (int u = 0; u < 16; u++) own[u] = mixed_with(own[u], first[u], mix);
    }
#pragma unroll
    for (int u = 0; u < 16; u++) {
        tile[wave + 4 * u][lane] = own[u];
        if (a.first_out && in(u)) a.first_out[(r0 + wave + 4 * u) * vn + c] = own[u];
    }
    __syncthreads();
    if (t0 + lane >= a.s) return;
    const int64_t slot = value_slot((int)(past_of(a) + t0) + lane);
    const int c0 = c - lane;
    for (int i = wave; i < 64 && c0 + i < vn; i += 4)
        keep(a.values, a.cache_bf16, value_row(a, b, (c0 + i) / a.vdim, (c0 + i) % a.vdim) + slot, tile[lane][i]);
}

// ---- few query rows -------------------------------------------------------------------------

// How many of a row's keys a share has: whole tiles.
__device__ __forceinline__ int64_t share_of(int64_t seen, int splits) {
    const int64_t share = (seen + splits - 1) / splits;
    return (share + kKeys - 1) / kKeys * kKeys;
}

struct Parts {
    float *o, *ml;  // [rows, splits, heads, vdim] sums; [rows, splits, heads, 2]: maximum, sum of weights
    int splits;
    float* out_f32;  // exactly one of the two: [rows, heads * vdim]
    uint16_t* out_bf16;
    int64_t ldo;
};
__device__ __forceinline__ void put(const Parts& p, int64_t at, float v) {
    if (p.out_f32) p.out_f32[at] = v;
    else p.out_bf16[at] = round_bf16(v);
}

__device__ __forceinline__ f32x4 mfma16_bf16(u32x4 a, u32x4 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

// A share of one row's keys for up to kHeads heads of one group, bfloat16 cache: workgroups (share, group and part of its heads,
// row) of four wavefronts. The sixteen columns of an MFMA are the heads twice, once the bfloat16 value of their queries
// (and weights) and once what rounding left. Scores: a wavefront has sixteen keys of a tile of 64; they meet in LDS, where
// every wavefront reads all of them and does the softmax of its lanes' heads; sums: a wavefront has every fourth tile of
// sixteen value features (VT of them). KS: steps of 32 features of a key. Keys and values go from the cache straight into
// operand registers. STEP: one position a sequence, from the projections; the workgroup whose share has the new position
// writes its cache entries and puts them into its operands itself.
template <int KS, int VT, bool STEP>
__global__ __launch_bounds__(256) void heads_attend_kernel(HeadAttention a, const float* __restrict__ q32, Parts parts) {
    __shared__ __align__(16) float qs[STEP ? kHeads : 1][KS * 32];
    __shared__ __align__(16) float ps[2][kHeads][kKeys + 4];
    __shared__ __align__(16) uint16_t knew[STEP ? KS * 32 : 8], vnew[STEP ? VT * 64 : 8];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int per = a.heads / a.kv_heads, chunks = (per + kHeads - 1) / kHeads;
    const int hk = blockIdx.y / chunks, h0 = hk * per + blockIdx.y % chunks * kHeads, nh = min(kHeads, (hk + 1) * per - h0);
    const int split = blockIdx.x;
    const int64_t r = blockIdx.z, b = r / a.s, pos = past_of(a) + r % a.s, seen = pos + 1;
    const int64_t share = share_of(seen, parts.splits), lo = split * share, hi = lo + share < seen ? lo + share : seen;
    if (lo >= hi) return;  // the whole workgroup: heads_combine_kernel does not look at this share
    const uint16_t* keys = (const uint16_t*)a.keys + key_row(a, b, hk, 0) + g * 8;
    const uint16_t* values = (const uint16_t*)a.values + value_row(a, b, hk, 0) + g * 8;
    u32x4 kf[KS], vf[2][VT];
    auto fetch_keys = [&](int64_t j0) {
        const int64_t j = j0 + wave * 16 + r16;
        const uint16_t* k = keys + (j < hi ? j : hi - 1) * a.ldk;
#pragma unroll
        for (int i = 0; i < KS; i++) {  // features past the last meet zeros of q
            kf[i] = u32x4{0, 0, 0, 0};
            if (i * 32 + g * 8 < a.ldk) kf[i] = *(const u32x4*)(k + i * 32);
        }
    };
    auto fetch_values = [&](int64_t j0) {
#pragma unroll
        for (int v = 0; v < VT; v++) {
            const int e = (wave + 4 * v) * 16 + r16;
            const uint16_t* x = values + (int64_t)(e < a.vdim ? e : a.vdim - 1) * a.context + j0;
#pragma unroll
            for (int half = 0; half < 2; half++) vf[half][v] = *(const u32x4*)(x + half * 32);
        }
    };
    fetch_keys(lo);
    fetch_values(lo);
    const bool mine = STEP && hi == seen;  // this share has the new position
    u32x4 q[KS];
    {
        const bool low = r16 >= 8;
        const int h = r16 & 7;
        if constexpr (STEP) {
            const float* p = a.proj + r * a.ldp;
            for (int u = wave; u < kHeads + (mine ? 1 : 0); u += 4) {
                if (u == kHeads) {
                    uint16_t* to = (uint16_t*)a.keys + key_row(a, b, hk, pos);
                    head_features(a, p + (int64_t)(a.heads + hk) * a.dim, pos, [&](int i, float v) { knew[i] = to[i] = round_bf16(v); });
                    for (int i = a.dim + lane; i < KS * 32; i += 64) knew[i] = 0;
                } else {
                    if (u < nh) head_features(a, p + (int64_t)(h0 + u) * a.dim, pos, [&](int i, float v) { qs[u][i] = v * a.scale; });
                    for (int i = (u < nh ? a.dim : 0) + lane; i < KS * 32; i += 64) qs[u][i] = 0.f;
                }
            }
            if (mine)
                for (int e = tid; e < a.vdim; e += 256) {
                    const uint16_t v = round_bf16(mixed_value(a, r, hk * a.vdim + e));
                    vnew[e] = v;
                    ((uint16_t*)a.values)[value_row(a, b, hk, e) + value_slot((int)pos)] = v;
                }
            __syncthreads();
        }
#pragma unroll
        for (int i = 0; i < KS; i++) {
            float x[8];
            const int d = i * 32 + g * 8;
#pragma unroll
            for (int e = 0; e < 8; e++) {
                if constexpr (STEP) x[e] = qs[h][d + e];
                else x[e] = h < nh && d + e < a.dim ? q32[(r * a.heads + h0 + h) * a.dim + d + e] : 0.f;
            }
#pragma unroll
            for (int e = 0; e < 4; e++) q[i][e] = low ? pack_bf16(low_part(x[2 * e]), low_part(x[2 * e + 1])) : pack_bf16(x[2 * e], x[2 * e + 1]);
        }
    }
    f32x4 acc[VT];
#pragma unroll
    for (int v = 0; v < VT; v++) acc[v] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -__builtin_inff(), l = 0.f;  // of head r16 % 8
    int parity = 0;
    for (int64_t j0 = lo; j0 < hi; j0 += kKeys, parity ^= 1) {
        if (STEP && mine && j0 + kKeys >= hi) {  // the new position: its key's row and its values' slot
            const int at = (int)(pos - j0);
            if (at == wave * 16 + r16) {
#pragma unroll
                for (int i = 0; i < KS; i++) kf[i] = *(const u32x4*)(knew + i * 32 + g * 8);
            }
            const int slot = value_slot(at);
            if (((slot >> 3) & 3) == g) {
#pragma unroll
                for (int v = 0; v < VT; v++) {
                    const int e = (wave + 4 * v) * 16 + r16;
                    const uint32_t x = vnew[e < a.vdim ? e : a.vdim - 1];
#pragma unroll
                    for (int half = 0; half < 2; half++)
#pragma unroll
                        for (int i = 0; i < 8; i++)
                            if (half * 32 + g * 8 + i == slot) vf[half][v][i >> 1] = i & 1 ? (vf[half][v][i >> 1] & 0xffffu) | x << 16 : (vf[half][v][i >> 1] & 0xffff0000u) | x;
                }
            }
        }
        f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < KS; i++) sc = mfma16_bf16(kf[i], q[i], sc);
#pragma unroll
        for (int i = 0; i < 4; i++) {
            sc[i] += __shfl_xor(sc[i], 8);
            sc[i] = j0 + wave * 16 + 4 * g + i < hi ? soft_cap(sc[i], a.softcap) : -__builtin_inff();
        }
        if (r16 < 8) *(f32x4*)(&ps[parity][r16][wave * 16 + 4 * g]) = sc;
        if (j0 + kKeys < hi) fetch_keys(j0 + kKeys);
        __syncthreads();  // the other half of ps is written next, by wavefronts that have passed this
        float s[16], top = -__builtin_inff();
#pragma unroll
        for (int n = 0; n < 4; n++) {  // slots g * 8 .. of either half of the tile
            const f32x4 x = *(const f32x4*)(&ps[parity][r16 & 7][(n >> 1) * 32 + (g >> 1) * 16 + (g & 1) * 4 + (n & 1) * 8]);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                s[4 * n + i] = x[i];
                top = fmaxf(top, x[i]);
            }
        }
        top = fmaxf(top, __shfl_xor(top, 16));
        top = fmaxf(top, __shfl_xor(top, 32));
        const float next = fmaxf(m, top), back = expf(m - next);  // the first tile's m: exp(-inf) = 0
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < 16; i++) {
            s[i] = expf(s[i] - next);
            sum += s[i];
        }
        sum += __shfl_xor(sum, 16);
        l = l * back + (sum + __shfl_xor(sum, 32));
        m = next;
#pragma unroll
        for (int v = 0; v < VT; v++) acc[v] = acc[v] * back;
#pragma unroll
        for (int half = 0; half < 2; half++) {
            u32x4 w;
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const float x = s[half * 8 + 2 * i], y = s[half * 8 + 2 * i + 1];
                w[i] = r16 >= 8 ? pack_bf16(low_part(x), low_part(y)) : pack_bf16(x, y);
            }
#pragma unroll
            for (int v = 0; v < VT; v++) acc[v] = mfma16_bf16(vf[half][v], w, acc[v]);
        }
        if (j0 + kKeys < hi) fetch_values(j0 + kKeys);
    }
    const int h = h0 + (r16 & 7);
    const bool whole = parts.splits == 1;
    const float inv = whole ? gate_of(a, r, h < a.heads ? h : a.heads - 1) / l : 1.f;
    const int64_t pr = (r * parts.splits + split) * a.heads;
#pragma unroll
    for (int v = 0; v < VT; v++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float x = acc[v][i] + __shfl_xor(acc[v][i], 8);
            const int e = (wave + 4 * v) * 16 + 4 * g + i;
            if (r16 >= nh || e >= a.vdim) continue;
            if (whole) put(parts, r * parts.ldo + (int64_t)h * a.vdim + e, x * inv);
            else parts.o[(pr + h) * a.vdim + e] = x;
        }
    if (!whole && wave == 0 && g == 0 && r16 < nh) {
        parts.ml[(pr + h) * 2] = m;
        parts.ml[(pr + h) * 2 + 1] = l;
    }
}

// Eight cache elements from `at` on, as float32.
__device__ __forceinline__ void load8(const float* p, float v[8]) {
    const f32x4 x = ((const f32x4*)p)[0], y = ((const f32x4*)p)[1];
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = x[i], v[4 + i] = y[i];
}
__device__ __forceinline__ void load8(const uint16_t* p, float v[8]) {
    const u32x4 x = *(const u32x4*)p;
#pragma unroll
    for (int i = 0; i < 4; i++) v[2 * i] = __uint_as_float(x[i] << 16), v[2 * i + 1] = __uint_as_float(x[i] & 0xffff0000u);
}

// The same on the vector units, behind heads_prepare_kernel: scores with a lane's key against two heads a wavefront, sums with
// a thread's features tid + 256 u.
template <typename T, int U>
__global__ __launch_bounds__(256) void heads_attend_any_kernel(HeadAttention a, const float* __restrict__ q32, Parts parts) {
    extern __shared__ __align__(16) float lds_heads[];
    const int D8 = (int)a.ldk;
    float* qs = lds_heads;               // [D8][kHeads]
    float* ps = qs + D8 * kHeads;        // [kKeys][kHeads]: scores, then weights
    float* ml = ps + kKeys * kHeads;     // [kHeads] rescaling of this tile; at the end the sums of weights
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int per = a.heads / a.kv_heads, chunks = (per + kHeads - 1) / kHeads;
    const int hk = blockIdx.y / chunks, h0 = hk * per + blockIdx.y % chunks * kHeads, nh = min(kHeads, (hk + 1) * per - h0);
    const int split = blockIdx.x;
    const int64_t r = blockIdx.z, b = r / a.s, seen = past_of(a) + r % a.s + 1;
    const int64_t share = share_of(seen, parts.splits), lo = split * share, hi = lo + share < seen ? lo + share : seen;
    if (lo >= hi) return;  // the whole workgroup: heads_combine_kernel does not look at this share
    for (int i = tid; i < D8 * kHeads; i += 256) {
        const int d = i / kHeads, h = i % kHeads;
        qs[i] = h < nh && d < a.dim ? q32[(r * a.heads + h0 + h) * a.dim + d] : 0.f;
    }
    const T* keys = (const T*)a.keys + key_row(a, b, hk, 0);
    const T* values = (const T*)a.values + value_row(a, b, hk, 0);
    float acc[kHeads][U];
#pragma unroll
    for (int h = 0; h < kHeads; h++)
#pragma unroll
        for (int u = 0; u < U; u++) acc[h][u] = 0.f;
    const int sh = tid >> 5, sk = tid & 31;  // the softmax's head and first key of this thread (32 threads a head)
    float m = -__builtin_inff(), l = 0.f;
    __syncthreads();
    for (int64_t j0 = lo; j0 < hi; j0 += kKeys) {
        {
            const T* k = keys + (j0 + lane < hi ? j0 + lane : hi - 1) * a.ldk;
            float s0 = 0.f, s1 = 0.f;
            for (int d = 0; d < D8; d += 8) {
                float v[8];
                load8(k + d, v);
#pragma unroll
                for (int i = 0; i < 8; i++) {
                    s0 = fmaf(qs[(d + i) * kHeads + wave * 2], v[i], s0);
                    s1 = fmaf(qs[(d + i) * kHeads + wave * 2 + 1], v[i], s1);
                }
            }
            ps[lane * kHeads + wave * 2] = soft_cap(s0, a.softcap);
            ps[lane * kHeads + wave * 2 + 1] = soft_cap(s1, a.softcap);
        }
        __syncthreads();
        {
            float s[2], top = -__builtin_inff();
#pragma unroll
            for (int i = 0; i < 2; i++) {
                s[i] = j0 + sk + 32 * i < hi ? ps[(sk + 32 * i) * kHeads + sh] : -__builtin_inff();
                top = fmaxf(top, s[i]);
            }
#pragma unroll
            for (int o = 16; o > 0; o >>= 1) top = fmaxf(top, __shfl_xor(top, o));
            const float next = fmaxf(m, top), back = expf(m - next);  // the first tile's m: exp(-inf) = 0
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < 2; i++) {
                const float p = expf(s[i] - next);
                sum += p;
                ps[(sk + 32 * i) * kHeads + sh] = p;
            }
#pragma unroll
            for (int o = 16; o > 0; o >>= 1) sum += __shfl_xor(sum, o);
            m = next;
            l = l * back + sum;
            if (sk == 0) ml[sh] = back;
        }
        __syncthreads();
        if (tid < a.vdim) {
#pragma unroll
            for (int h = 0; h < kHeads; h++)
#pragma unroll
                for (int u = 0; u < U; u++) acc[h][u] *= ml[h];
            for (int c = 0; c < kKeys; c += 8) {  // eight slots: two runs of four keys
                const int key = (c & ~15) + (c & 8 ? 4 : 0);
                float v[U][8];
#pragma unroll
                for (int u = 0; u < U; u++) {
                    const int e = tid + 256 * u;
                    load8(values + (int64_t)(e < a.vdim ? e : tid) * a.context + j0 + c, v[u]);
                }
#pragma unroll
                for (int i = 0; i < 8; i++) {
                    const int j = key + (i & 3) + (i & 4) * 2;
                    if (j0 + j >= hi) continue;
#pragma unroll
                    for (int h = 0; h < kHeads; h++)
#pragma unroll
                        for (int u = 0; u < U; u++) acc[h][u] = fmaf(ps[j * kHeads + h], v[u][i], acc[h][u]);
                }
            }
        }
        __syncthreads();
    }
    const int64_t pr = (r * parts.splits + split) * a.heads;
    const bool whole = parts.splits == 1;
    if (sk == 0 && sh < nh) {
        ml[sh] = l;
        if (!whole) {
            parts.ml[(pr + h0 + sh) * 2] = m;
            parts.ml[(pr + h0 + sh) * 2 + 1] = l;
        }
    }
    __syncthreads();
#pragma unroll
    for (int h = 0; h < kHeads; h++) {
        if (h >= nh) break;
        const float f = whole ? gate_of(a, r, h0 + h) / ml[h] : 1.f;
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int e = tid + 256 * u;
            if (e >= a.vdim) continue;
            if (whole) put(parts, r * parts.ldo + (int64_t)(h0 + h) * a.vdim + e, acc[h][u] * f);
            else parts.o[(pr + h0 + h) * a.vdim + e] = acc[h][u];
        }
    }
}

// The shares of a row's head brought together, times its gate: workgroups (head, row); the wavefronts take every fourth share.
__global__ __launch_bounds__(256) void heads_combine_kernel(HeadAttention a, Parts parts) {
    __shared__ float weight[kMaxSplits];
    __shared__ float red[3][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, splits = parts.splits;
    const int64_t r = blockIdx.y, seen = past_of(a) + r % a.s + 1, share = share_of(seen, splits);
    const int live = (int)((seen + share - 1) / share);  // shares that have keys
    const float* ml = parts.ml + (r * splits * a.heads + h) * 2;
    const float* po = parts.o + (r * splits * a.heads + h) * a.vdim;
    const int64_t mstep = (int64_t)a.heads * 2, ostep = (int64_t)a.heads * a.vdim;
    if (wave == 0) {
        float top = -__builtin_inff();
        for (int s = lane; s < live; s += 64) top = fmaxf(top, ml[s * mstep]);
        top = wave_max(top);
        float sum = 0.f;
        for (int s = lane; s < live; s += 64) {
            const float w = expf(ml[s * mstep] - top);
            weight[s] = w;
            sum = fmaf(ml[s * mstep + 1], w, sum);
        }
        const float f = gate_of(a, r, h) / wave_sum(sum);
        for (int s = lane; s < live; s += 64) weight[s] *= f;
    }
    __syncthreads();
    for (int e0 = 0; e0 < a.vdim; e0 += 64) {
        const int e = e0 + lane;
        float v = 0.f;
        if (e < a.vdim) {
#pragma unroll 8
            for (int s = wave; s < live; s += 4) v = fmaf(po[s * ostep + e], weight[s], v);
        }
        if (wave > 0) red[wave - 1][lane] = v;
        __syncthreads();
        if (wave == 0 && e < a.vdim) put(parts, r * parts.ldo + (int64_t)h * a.vdim + e, (v + red[0][lane]) + (red[1][lane] + red[2][lane]));
        __syncthreads();
    }
}

// ---- many query rows ------------------------------------------------------------------------
// A wavefront owns 32 query rows of one head and walks the keys in tiles of 64. Both products are computed transposed
// (scores^T = K Q^T, result^T = V^T P^T), so that a row's scores and results lie in one lane and its partner 32 lanes on,
// and the weights go from the exponential straight into the second product's operand, as the sum of two bfloat16. Four
// wavefronts with consecutive rows share a tile of keys and values in LDS, which goes there straight from the cache while the
// tile before is used; a row's pieces of sixteen bytes are exchanged so that the reads of 32 rows spread over the banks.
// Products are issued between the exponentials of the other half of the tile: a wavefront's MFMAs run beside its own
// vector instructions, which take longer.
//
// The queries come times scale log2(e) (a capped score's: 2 scale / cap log2(e)). A capped score is
// cap (1 - 2 / (exp(2 s / cap) + 1)), at most cap: where exp(-2 cap) is far from float32's smallest number the weights are
// taken relative to exp(cap), and no running maximum is needed (CAP 1; CAP 2 keeps one, CAP 0 has no cap).

// 16 bytes a lane from a wavefront's address and a lane's offset into LDS (load_to_lds, gemm_nt_tile.h).
__device__ __forceinline__ void load_to_lds(const void* g, uint32_t offset, uint32_t lds_base) {
    asm volatile("s_mov_b32 m0, %0\n\tglobal_load_lds_dwordx4 %1, %2" ::"s"(lds_base), "v"(offset), "s"(g) : "memory");
}
__device__ __forceinline__ f32x16 mfma_bf16(u32x4 a, u32x4 b, f32x16 c) { return Bf16Element::mfma(a, b, c); }

struct PromptArgs {
    HeadAttention a;
    const uint16_t* q;
    uint16_t* out;
    int64_t ldo;
    int past, s, fold;
    float cap2, inv_cap2;  // 2 cap log2(e), and -1 over it
};

constexpr int kPromptRows = 128;

// DT: sixteenths of dim, rounded up to a multiple of four; VT: 32nds of vdim, rounded up.
template <int DT, int VT, int CAP>
__global__ __launch_bounds__(256, DT > 8 ? 1 : 2) void heads_prompt_kernel(PromptArgs p) {
    constexpr int P = DT * 2;  // pieces of a key's row in LDS
    constexpr int kKeyBytes = kKeys * P * 16, kValBytes = VT * 32 * 128, kStage = kKeyBytes + kValBytes;
    constexpr int NK = DT / 2, NV = VT;  // loads of 1 KB a wavefront issues a tile
    extern __shared__ __align__(1024) char lds_prompt[];
    const HeadAttention& a = p.a;
    const int tid = threadIdx.x, lane = tid & 63, r32 = lane & 31, hi = lane >> 5;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    // heads of different groups beside each other: with as many groups as dies, a group's workgroups share a die's cache
    const int per = a.heads / a.kv_heads, hk = blockIdx.x % a.kv_heads, h = hk * per + blockIdx.x / a.kv_heads;
    // the last rows first: they see the most keys. Where all workgroups fit the device at once, two a compute unit, the
    // second half goes the other way, so that long ones and short ones share a unit.
    const int nb = gridDim.y, by = blockIdx.y;
    const int first = (p.fold && by >= (nb + 1) / 2 ? by - (nb + 1) / 2 : nb - 1 - by) * kPromptRows;
    const int64_t b = blockIdx.z;
    const int row = first + wave * 32 + r32, pos = p.past + row;  // sees keys 0 .. pos
    const int last_wg = first + kPromptRows < p.s ? first + kPromptRows : p.s;
    const int seen_wg = p.past + last_wg;
    const int seen_wave = first + wave * 32 < p.s ? (p.past + (first + wave * 32 + 32 < p.s ? first + wave * 32 + 32 : p.s)) : 0;

    // where this lane's pieces of a tile come from: offsets that are the same for every tile
    uint32_t kfrom[NK], vfrom[NV];
    const char* keys = (const char*)((const uint16_t*)a.keys + key_row(a, b, hk, 0));
    const char* values = (const char*)((const uint16_t*)a.values + value_row(a, b, hk, 0));
    const uint32_t lds0 = (uint32_t)(uintptr_t)lds_prompt + wave * 1024;
#pragma unroll
    for (int n = 0; n < NK; n++) {
        const int item = (wave + 4 * n) * 64 + lane, r = item / P, piece = item % P ^ (P % 16 == 0 ? r & 15 : r >> 1 & 7);
        kfrom[n] = (uint32_t)(r * a.ldk + (piece * 8 < a.ldk ? piece * 8 : 0)) * 2;  // pieces past the last feature meet zeros of q
    }
#pragma unroll
    for (int n = 0; n < NV; n++) {
        const int item = (wave + 4 * n) * 64 + lane, r = item >> 3, piece = (item & 7) ^ (r >> 1 & 7);
        vfrom[n] = (uint32_t)((r < a.vdim ? r : a.vdim - 1) * a.context + piece * 8) * 2;
    }
    auto fetch = [&](uint32_t stage) {
#pragma unroll
        for (int n = 0; n < NK; n++) load_to_lds(keys, kfrom[n], __builtin_amdgcn_readfirstlane(stage + n * 4096));
#pragma unroll
        for (int n = 0; n < NV; n++) load_to_lds(values, vfrom[n], __builtin_amdgcn_readfirstlane(stage + kKeyBytes + n * 4096));
        keys += kKeys * a.ldk * 2;
        values += kKeys * 2;
    };
    u32x4 q[DT];
    {
        const uint16_t* qr = p.q + ((b * p.s + (row < p.s ? row : p.s - 1)) * a.heads + h) * a.ldk;
#pragma unroll
        for (int k = 0; k < DT; k++) {
            const int d = k * 16 + hi * 8;
            q[k] = u32x4{0, 0, 0, 0};
            if (d < a.ldk) q[k] = *(const u32x4*)(qr + d);
        }
    }
    f32x16 o[VT];
#pragma unroll
    for (int t = 0; t < VT; t++)
#pragma unroll
        for (int i = 0; i < 16; i++) o[t][i] = 0.f;
    float m = -__builtin_inff(), l = 0.f;  // the running maximum (in units of log2; not with CAP 1); the sum over the keys this half of the lanes holds
    const int kswz = P % 16 == 0 ? r32 & 15 : r32 >> 1 & 7, vswz = r32 >> 1 & 7;

    fetch(lds0);
    int stage = 0;
    for (int j0 = 0; j0 < seen_wg; j0 += kKeys, stage ^= 1) {
        wait_loads();   // this wavefront's part of the tile has landed
        lds_barrier();  // everyone's has, and everyone has read the other stage
        if (j0 + kKeys < seen_wg) fetch(lds0 + (stage ^ 1) * kStage);
        if (j0 >= seen_wave) continue;
        const char* ks = lds_prompt + stage * kStage;
        const char* vs = ks + kKeyBytes;
        const bool whole = j0 + kKeys - 1 <= p.past + first + wave * 32;  // every row of the wavefront sees the whole tile
        f32x16 sc[2];
        u32x4 high[2], low[2];
        auto key = [&](int c, int k) { return *(const u32x4*)(ks + ((c * 32 + r32) * P + ((2 * k + hi) ^ kswz)) * 16); };
        // all fragments of the keys are requested first, those of the values (a half of the tile's) before its weights are split
        u32x4 kf[2][DT], vf[2][VT];
        if constexpr (DT <= 8) {
#pragma unroll
            for (int c = 0; c < 2; c++)
#pragma unroll
                for (int k = 0; k < DT; k++) kf[c][k] = key(c, k);
            __builtin_amdgcn_sched_barrier(0);
        }
        auto multiply_keys = [&](int c, int k) { sc[c] = mfma_bf16(DT <= 8 ? kf[c][k] : key(c, k), q[k], sc[c]); };
        auto hide = [&](int c, float v) {  // what stands for keys that a row does not see
            if (whole) return;
#pragma unroll
            for (int i = 0; i < 16; i++) sc[c][i] = j0 + c * 32 + (i & 3) + 8 * (i >> 2) + 4 * hi > pos ? v : sc[c][i];
        };
        auto weight = [&](int c, int i) {  // of a score, in its place
            if constexpr (CAP == 1) sc[c][i] = __builtin_amdgcn_exp2f(__builtin_amdgcn_rcpf(fmaf(__builtin_amdgcn_exp2f(sc[c][i]), p.inv_cap2, p.inv_cap2)));
            else sc[c][i] = __builtin_amdgcn_exp2f(sc[c][i] - m);
        };
        auto split = [&](int c, int half) {  // eight weights as the sum of two bfloat16
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const float x = sc[c][half * 8 + 2 * i], y = sc[c][half * 8 + 2 * i + 1];
                l += x + y;
                high[half][i] = pack_bf16(x, y);
                low[half][i] = pack_bf16(x - __uint_as_float(high[half][i] << 16), y - __uint_as_float(high[half][i] & 0xffff0000u));
            }
        };
        auto fetch_values = [&](int c) {
#pragma unroll
            for (int half = 0; half < 2; half++)
#pragma unroll
                for (int t = 0; t < VT; t++) vf[half][t] = *(const u32x4*)(vs + (t * 32 + r32) * 128 + ((c * 4 + half * 2 + hi) ^ vswz) * 16);
            __builtin_amdgcn_sched_barrier(0);
        };
#pragma unroll
        for (int c = 0; c < 2; c++)
#pragma unroll
            for (int i = 0; i < 16; i++) sc[c][i] = 0.f;
#pragma unroll
        for (int k = 0; k < DT; k++) multiply_keys(0, k);
        if constexpr (CAP == 1) {
#pragma unroll
            for (int k = 0; k < DT; k++) {
                multiply_keys(1, k);
#pragma unroll
                for (int i = 16 * k / DT; i < 16 * (k + 1) / DT; i++) weight(0, i);
            }
            hide(0, 0.f);
        } else {
#pragma unroll
            for (int k = 0; k < DT; k++) multiply_keys(1, k);
            if constexpr (CAP == 2) {  // capped scores less their cap
#pragma unroll
                for (int c = 0; c < 2; c++)
#pragma unroll
                    for (int i = 0; i < 16; i++) sc[c][i] = __builtin_amdgcn_rcpf(fmaf(__builtin_amdgcn_exp2f(sc[c][i]), p.inv_cap2, p.inv_cap2));
            }
            hide(0, -__builtin_inff());
            hide(1, -__builtin_inff());
            float top = -__builtin_inff();
#pragma unroll
            for (int c = 0; c < 2; c++)
#pragma unroll
                for (int i = 0; i < 16; i++) top = fmaxf(top, sc[c][i]);
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
            for (int i = 0; i < 16; i++) weight(0, i);
        }
#pragma unroll
        for (int c = 0; c < 2; c++) {
            fetch_values(c);
            split(c, 0);
            split(c, 1);
#pragma unroll
            for (int half = 0; half < 2; half++) {
#pragma unroll
                for (int part = 0; part < 2; part++)
#pragma unroll
                    for (int t = 0; t < VT; t++) {
                        o[t] = mfma_bf16(vf[half][t], part ? low[half] : high[half], o[t]);
                        if (c == 0) {  // the other half's weights between these
                            const int at = (half * 2 + part) * VT + t;
#pragma unroll
                            for (int i = 16 * at / (4 * VT); i < 16 * (at + 1) / (4 * VT); i++) weight(1, i);
                        }
                    }
            }
            if (CAP == 1 && c == 0) hide(1, 0.f);
        }
    }
    const float sum = l + __shfl_xor(l, 32);
    if (row >= p.s) return;
    const float f = gate_of(a, b * p.s + row, h) / sum;
    uint16_t* out = p.out + (b * p.s + row) * p.ldo + (int64_t)h * a.vdim;
    const bool wide = a.vdim % 4 == 0 && p.ldo % 4 == 0 && ((uintptr_t)p.out & 7) == 0;
#pragma unroll
    for (int t = 0; t < VT; t++)
#pragma unroll
        for (int g = 0; g < 4; g++) {
            const int e = t * 32 + 8 * g + 4 * hi;
            if (wide) {
                if (e < a.vdim) *(u32x2*)(out + e) = u32x2{pack_bf16(o[t][4 * g] * f, o[t][4 * g + 1] * f), pack_bf16(o[t][4 * g + 2] * f, o[t][4 * g + 3] * f)};
                continue;
            }
#pragma unroll
            for (int i = 0; i < 4; i++)
                if (e + i < a.vdim) out[e + i] = round_bf16(o[t][4 * g + i] * f);
        }
}

template <int DT, int VT, int CAP>
hipError_t launch_prompt(PromptArgs p, hipStream_t st) {
    constexpr size_t lds = 2 * ((size_t)kKeys * DT * 32 + VT * 32 * 128);
    static_assert(lds <= 160 * 1024, "a compute unit's LDS");
    hipError_t e = hipFuncSetAttribute((const void*)heads_prompt_kernel<DT, VT, CAP>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
    const dim3 grid((unsigned)p.a.heads, (unsigned)((p.s + kPromptRows - 1) / kPromptRows), (unsigned)p.a.batch);
    p.fold = (int64_t)grid.x * grid.y * grid.z <= 512;
    hipLaunchKernelGGL((heads_prompt_kernel<DT, VT, CAP>), grid, dim3(256), lds, st, p);
    return hipGetLastError();
}
template <int DT, int VT>
hipError_t launch_prompt(const PromptArgs& p, hipStream_t st) {
    if (p.a.softcap <= 0.f) return launch_prompt<DT, VT, 0>(p, st);
    return p.cap2 <= 90.f ? launch_prompt<DT, VT, 1>(p, st) : launch_prompt<DT, VT, 2>(p, st);  // weights of 2^-90 and more
}

bool attend_mfma_ok(const HeadAttention& a) { return a.cache_bf16 && a.dim <= 256 && a.vdim <= 256; }

template <int KS, int VT>
void launch_attend(const HeadAttention& a, const float* q32, const Parts& parts, dim3 grid, bool step, hipStream_t st) {
    if (step) hipLaunchKernelGGL((heads_attend_kernel<KS, VT, true>), grid, dim3(256), 0, st, a, q32, parts);
    else hipLaunchKernelGGL((heads_attend_kernel<KS, VT, false>), grid, dim3(256), 0, st, a, q32, parts);
}
template <typename T>
void launch_attend_any(const HeadAttention& a, const float* q32, const Parts& parts, dim3 grid, hipStream_t st) {
    const size_t lds = ((size_t)a.ldk * kHeads + kKeys * kHeads + kHeads) * 4;
    if (a.vdim <= 256) hipLaunchKernelGGL((heads_attend_any_kernel<T, 1>), grid, dim3(256), lds, st, a, q32, parts);
    else hipLaunchKernelGGL((heads_attend_any_kernel<T, 4>), grid, dim3(256), lds, st, a, q32, parts);
}

hipError_t prepare(const HeadAttention& a, uint16_t* q16, float* q32, float q_scale, hipStream_t st) {
    const int lanes = !head_fours_ok(a) ? 0 : a.dim <= 64 ? 16 : a.dim <= 128 ? 32 : 64, at_once = lanes ? 256 / lanes : 4;
    const int64_t heads = a.batch * a.s * ((a.heads + a.kv_heads + at_once - 1) / at_once);
    const dim3 grid((unsigned)(heads + a.batch * ((a.s + 63) / 64) * (((int64_t)a.kv_heads * a.vdim + 63) / 64)));
    if (lanes == 16) hipLaunchKernelGGL(heads_prepare_kernel<16>, grid, dim3(256), 0, st, a, q16, q32, q_scale);
    else if (lanes == 32) hipLaunchKernelGGL(heads_prepare_kernel<32>, grid, dim3(256), 0, st, a, q16, q32, q_scale);
    else if (lanes == 64) hipLaunchKernelGGL(heads_prepare_kernel<64>, grid, dim3(256), 0, st, a, q16, q32, q_scale);
    else hipLaunchKernelGGL(heads_prepare_kernel<0>, grid, dim3(256), 0, st, a, q16, q32, q_scale);
    return hipGetLastError();
}

// By the capacity, not by how many positions are held: a recorded step keeps its grid.
int splits_of(const HeadAttention& a) {
    const int per = a.heads / a.kv_heads;
    const int64_t wgs = (int64_t)a.batch * a.s * a.kv_heads * ((per + kHeads - 1) / kHeads), most = (a.context + kKeys - 1) / kKeys;
    const int64_t want = (kMaxSplits + wgs - 1) / wgs;
    return (int)(want < most ? want : most);
}

}  // namespace

// rows * splits <= kMaxSplits + rows
size_t heads_attend_ws_floats(const HeadAttention& a, int64_t rows) {
    return (size_t)rows * a.heads * a.dim + (size_t)(kMaxSplits + rows) * a.heads * (a.vdim + 2);
}

hipError_t heads_attend(const HeadAttention& a, float* ws, float* out_f32, uint16_t* out_bf16, int64_t ldo, hipStream_t st) {
    const int64_t rows = (int64_t)a.batch * a.s;
    if (rows == 0) return hipSuccess;
    if (a.dim > kHeadAttentionMax || a.vdim > kHeadAttentionMax || rows > 65535 || a.ldk % 8 || a.context % kKeys || a.heads % a.kv_heads) return hipErrorInvalidValue;
    const int per = a.heads / a.kv_heads;
    Parts parts;
    parts.splits = splits_of(a);
    parts.o = ws + (size_t)rows * a.heads * a.dim;
    parts.ml = parts.o + (size_t)rows * parts.splits * a.heads * a.vdim;
    parts.out_f32 = out_f32; parts.out_bf16 = out_bf16; parts.ldo = ldo;
    const dim3 grid((unsigned)parts.splits, (unsigned)(a.kv_heads * ((per + kHeads - 1) / kHeads)), (unsigned)rows);
    const bool mfma = attend_mfma_ok(a), step = mfma && a.s == 1;
    if (!step)
        if (hipError_t e = prepare(a, nullptr, ws, a.scale, st)) return e;
    if (mfma) {
        if (a.dim <= 64 && a.vdim <= 64) launch_attend<2, 1>(a, ws, parts, grid, step, st);
        else if (a.dim <= 128 && a.vdim <= 128) launch_attend<4, 2>(a, ws, parts, grid, step, st);
        else launch_attend<8, 4>(a, ws, parts, grid, step, st);
    } else if (a.cache_bf16) {
        launch_attend_any<uint16_t>(a, ws, parts, grid, st);
    } else {
        launch_attend_any<float>(a, ws, parts, grid, st);
    }
    if (hipError_t e = hipGetLastError()) return e;
    if (parts.splits > 1) hipLaunchKernelGGL(heads_combine_kernel, dim3((unsigned)a.heads, (unsigned)rows), dim3(256), 0, st, a, parts);
    return hipGetLastError();
}

bool heads_prompt_ok(const HeadAttention& a) {
    return attend_mfma_ok(a) && a.vdim * a.context < 1ll << 30 && a.past + a.s < 1 << 30 && !a.past_dev && a.batch <= 65535 && a.s <= (int64_t)65535 * kPromptRows;
}

hipError_t heads_prompt(const HeadAttention& a, uint16_t* q, uint16_t* out, int64_t ldo, hipStream_t st) {
    if (a.batch * a.s == 0) return hipSuccess;
    if (!heads_prompt_ok(a) || a.ldk % 8 || a.context % kKeys || a.past + a.s > a.context || a.heads % a.kv_heads) return hipErrorInvalidValue;
    constexpr float kLog2e = 1.4426950408889634f;
    if (hipError_t e = prepare(a, q, nullptr, a.softcap > 0.f ? 2.f * a.scale / a.softcap * kLog2e : a.scale * kLog2e, st)) return e;
    PromptArgs p;
    p.a = a;
    p.q = q; p.out = out; p.ldo = ldo;
    p.past = (int)a.past; p.s = (int)a.s; p.fold = 0;
    p.cap2 = 2.f * a.softcap * kLog2e;
    p.inv_cap2 = -1.f / p.cap2;
    if (a.dim <= 64 && a.vdim <= 64) return launch_prompt<4, 2>(p, st);
    if (a.dim <= 128 && a.vdim <= 128) return launch_prompt<8, 4>(p, st);
    return launch_prompt<16, 8>(p, st);
}

}  // namespace mimir
