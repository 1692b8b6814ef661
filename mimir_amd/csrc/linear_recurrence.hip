// Linear recurrences with a matrix state per head, S [dim, vdim] <- decay S + k v^T, o = S^T q, in the two forms that
// stack_ops.h describes (struct Recurrence): with learned, stabilized input and forget gates and a normalizer (mLSTM),
// and with a constant decay per head (lightning attention).
//
// recurrence_scan goes position by position: a workgroup owns 32 columns of one head's S, in registers for the whole
// call (a thread holds one column's rows dg * DPT ..), so a decoding step reads and writes the state once. The columns'
// workgroups each keep n and m for themselves (a copy per slice in memory), so none waits for another.
#include "device_util.h"
#include "stack_ops.h"

namespace mimir {

namespace {

constexpr int kCols = 32, kGroups = 8;

__device__ __forceinline__ float load_act(const void* p, int64_t i, bool bf16) {
    return bf16 ? bf16_bits_to_f32(((const uint16_t*)p)[i]) : ((const float*)p)[i];
}

// min(z, 0) - log(1 + exp(-|z|))
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float capped(float z, float cap) { return cap * tanhf(z / cap); }

template <bool GATED, int DPT>
__global__ __launch_bounds__(256) void recurrence_scan_kernel(Recurrence r) {
    __shared__ float kk[kRecurrenceMaxDim], qq[kRecurrenceMaxDim], vv[kCols];
    __shared__ float red[kGroups][kCols + 1], red_n[4];
    const int tid = threadIdx.x, col = tid & 31, dg = tid >> 5, lane = tid & 63, wave = tid >> 6;
    const int slice = blockIdx.x, h = blockIdx.y, b = blockIdx.z, slices = gridDim.x;
    const int D = r.dim, E = r.vdim, e = slice * kCols + col;
    const bool live = e < E;
    const int64_t head = (int64_t)b * r.heads + h;
    float* S = r.S + head * D * E;
    float s[DPT];
#pragma unroll
    for (int i = 0; i < DPT; i++) {
        const int d = dg * DPT + i;
        s[i] = live && d < D ? S[(int64_t)d * E + e] : 0.f;
    }
    float* np = GATED ? r.n + (head * slices + slice) * D : nullptr;
    float n = GATED && tid < D ? np[tid] : 0.f;
    float m = GATED ? r.m[head * slices + slice] : 0.f;
    const float bi = GATED ? r.bias_i[h] : 0.f, bf = GATED ? r.bias_f[h] : 0.f;
    const float decay = GATED ? 0.f : r.decay[h];
    for (int64_t t = 0; t < r.s; t++) {
        const int64_t row = b * r.s + t;
        // zeros beyond the head's features: what the threads hold there stays zero
        kk[tid] = tid < D ? load_act(r.k, row * r.ld + (int64_t)h * D + tid, r.bf16) : 0.f;
        qq[tid] = tid < D ? load_act(r.q, row * r.ld + (int64_t)h * D + tid, r.bf16) * r.q_scale : 0.f;
        if (tid < kCols) vv[tid] = slice * kCols + tid < E ? load_act(r.v, row * r.ld + (int64_t)h * E + slice * kCols + tid, r.bf16) : 0.f;
        float keep = decay, take = 1.f;
        if (GATED) {
            const float li = capped(r.gates[row * r.ldg + h] + bi, r.cap);
            const float lf = log_sigmoid(capped(r.gates[row * r.ldg + r.heads + h] + bf, r.cap));
            const float next = fmaxf(lf + m, li);
            keep = expf(lf + m - next);
            take = expf(li - next);
            m = next;
        }
        __syncthreads();
        const float tv = take * vv[col];
        float o = 0.f;
#pragma unroll
        for (int i = 0; i < DPT; i++) {
            const int d = dg * DPT + i;
            s[i] = fmaf(kk[d], tv, keep * s[i]);
            o = fmaf(s[i], qq[d], o);
        }
        red[dg][col] = o;
        if (GATED) {
            float nq = 0.f;
            if (tid < D) {
                n = fmaf(take, kk[tid], keep * n);
                nq = n * qq[tid];
            }
            nq = wave_sum(nq);
            if (lane == 0) red_n[wave] = nq;
        }
        __syncthreads();
        if (tid < kCols && live) {
            float sum = 0.f;
#pragma unroll
            for (int g = 0; g < kGroups; g++) sum += red[g][tid];
            if (GATED) sum = sum / (fmaxf(fabsf((red_n[0] + red_n[1]) + (red_n[2] + red_n[3])), expf(-m)) + 1e-6f);
            r.out[row * r.ldo + (int64_t)h * E + e] = sum;
        }
    }
#pragma unroll
    for (int i = 0; i < DPT; i++) {
        const int d = dg * DPT + i;
        if (live && d < D) S[(int64_t)d * E + e] = s[i];
    }
    if (GATED) {
        if (tid < D) np[tid] = n;
        if (tid == 0) r.m[head * slices + slice] = m;
    }
}

template <bool GATED>
void launch_scan(const Recurrence& r, hipStream_t st) {
    const dim3 grid((unsigned)recurrence_slices(r.vdim), (unsigned)r.heads, (unsigned)r.batch);
    if (r.dim <= 4 * kGroups) hipLaunchKernelGGL((recurrence_scan_kernel<GATED, 4>), grid, dim3(256), 0, st, r);
    else if (r.dim <= 8 * kGroups) hipLaunchKernelGGL((recurrence_scan_kernel<GATED, 8>), grid, dim3(256), 0, st, r);
    else if (r.dim <= 16 * kGroups) hipLaunchKernelGGL((recurrence_scan_kernel<GATED, 16>), grid, dim3(256), 0, st, r);
    else hipLaunchKernelGGL((recurrence_scan_kernel<GATED, 32>), grid, dim3(256), 0, st, r);
}

// ---- prompts in chunks ---------------------------------------------------------------------
// A chunk of C = 64 positions in matrix products. With b_t the sum of the chunk's log decays up to t, position t sees
// position s <= t of its chunk with weight exp(b_t - b_s + i_s - m_t) and the state S at the chunk's start with
// exp(b_t + m - m_t); since m_t = b_t + M_t with M_t = max(m, max over s <= t of a_s) and a_s = i_s - b_s, these are
// exp(a_s - M_t) and exp(m - M_t), none above 1. A constant decay gives decay^(t - s) and decay^(t + 1).
// Three launches, chunks side by side in the first and the last:
//   chunk_states   each chunk's own sum of weighted v k^T (and of k), relative to its largest a_s
//   chunk_carry    S at every chunk's start, chunk after chunk, and the state behind the last
//   chunk_outputs  o of the chunk's positions from S and from the chunk itself
// Operands that are not q, k, v (weighted keys, weights, S) go to the matrix cores as the sum of two bfloat16. The states
// between the launches lie as their operand does: blocks of 32 values by 16 features, 512 floats each; value e, features
// 8 p .. 8 p + 7 belong to lane e + 32 p (p 0 or 1), whose first four floats are at 4 lane and whose others 256 behind. In
// their place chunk_carry leaves the eight high and the eight low bfloat16 parts.

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

constexpr int kC = kRecurrenceChunk;
constexpr int kRow = kC + 8;     // elements between rows of a transposed tile in LDS
constexpr int kValueTile = 128;  // rows of S (values) a workgroup

__device__ __forceinline__ f32x16 mfma_bf16(u32x4 a, u32x4 b, f32x16 c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

struct ChunkWs {
    float* states;   // [chunks, batch * heads, ep / 32, dp / 16, 512]
    float* norms;    // [chunks, batch * heads, dp]: the sums of k, then n at the chunk's start
    float* gates;    // [chunks, batch * heads, 2]: the chunk's log decay, its largest a_s
    float* m_start;  // [chunks, batch * heads]
    int dp, ep;      // dim to a multiple of 16, vdim to one of 32
    int chunks;
};

// Lane s holds position s of the chunk: its a_s, b_s and the maximum of a up to s. Positions past the end: a = -inf.
__device__ __forceinline__ void chunk_gates(const Recurrence& r, int64_t row0, int n, int h, int lane, float* a, float* b, float* top) {
    float li = -__builtin_inff(), lf = 0.f;
    if (lane < n) {
        const float* g = r.gates + (row0 + lane) * r.ldg + h;
        li = capped(g[0] + r.bias_i[h], r.cap);
        lf = log_sigmoid(capped(g[r.heads] + r.bias_f[h], r.cap));
    }
    float sum = lf;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const float up = __shfl_up(sum, o);
        if (lane >= o) sum += up;
    }
    float most = li - sum;
    *a = most;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const float up = __shfl_up(most, o);
        if (lane >= o) most = fmaxf(most, up);
    }
    *b = sum;
    *top = most;
}

// Columns [c0, c0 + cols) of the chunk's rows of src (n of them, the rest zero), transposed into dst [cols_padded][kRow]; with `w`
// (LDS, by position) scaled and split into dst (high) and low. cols, cols_padded: multiples of 8.
__device__ __forceinline__ void stage_transposed(const uint16_t* __restrict__ src, int64_t ld, int n, int cols, int cols_padded, uint16_t* dst,
                                                 uint16_t* low, const float* w) {
    const int pieces = cols_padded / 8;
    for (int item = threadIdx.x; item < pieces * (kC / 4); item += 256) {
        const int p = item % pieces, s0 = (item / pieces) * 4;
        u32x4 v[4];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            v[i] = u32x4{0, 0, 0, 0};
            if (s0 + i < n && p * 8 < cols) v[i] = *(const u32x4*)(src + (int64_t)(s0 + i) * ld + p * 8);
        }
#pragma unroll
        for (int e = 0; e < 8; e++) {
            uint32_t bits[4];
#pragma unroll
            for (int i = 0; i < 4; i++) bits[i] = e & 1 ? v[i][e >> 1] >> 16 : v[i][e >> 1] & 0xffffu;
            uint16_t* at = dst + (p * 8 + e) * kRow + s0;
            if (!w) {
                *(u32x2*)at = u32x2{bits[0] | bits[1] << 16, bits[2] | bits[3] << 16};
            } else {
                float f[4];
#pragma unroll
                for (int i = 0; i < 4; i++) f[i] = __uint_as_float(bits[i] << 16) * w[s0 + i];
                *(u32x2*)at = u32x2{pack_bf16(f[0], f[1]), pack_bf16(f[2], f[3])};
                *(u32x2*)(low + (p * 8 + e) * kRow + s0) = u32x2{pack_bf16(low_part(f[0]), low_part(f[1])), pack_bf16(low_part(f[2]), low_part(f[3]))};
            }
        }
    }
}

template <bool GATED>
__global__ __launch_bounds__(256) void chunk_states_kernel(Recurrence r, ChunkWs ws) {
    extern __shared__ __align__(16) uint16_t lds_chunk[];
    __shared__ float weight[kC];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r32 = lane & 31, hi = lane >> 5;
    const int chunk = blockIdx.x, h = blockIdx.y, vt = (r.vdim + kValueTile - 1) / kValueTile, b = blockIdx.z / vt, e0 = (blockIdx.z % vt) * kValueTile;
    const int dp32 = (ws.dp + 31) / 32 * 32;
    uint16_t* vT = lds_chunk;                // [kValueTile][kRow]
    uint16_t* kH = vT + kValueTile * kRow;   // [dp32][kRow], high parts
    uint16_t* kL = kH + dp32 * kRow;         // low parts
    const int64_t row0 = b * r.s + (int64_t)chunk * kC;
    const int n = r.s - (int64_t)chunk * kC < kC ? (int)(r.s - (int64_t)chunk * kC) : kC;
    const int64_t head = (int64_t)(chunk * r.batch + b) * r.heads + h;
    if (wave == 0) {
        if (GATED) {
            float a, bs, top;
            chunk_gates(r, row0, n, h, lane, &a, &bs, &top);
            const float most = __shfl(top, n - 1);
            weight[lane] = lane < n ? expf(a - most) : 0.f;
            if (lane == n - 1 && e0 == 0) {
                ws.gates[head * 2] = bs;
                ws.gates[head * 2 + 1] = most;
            }
        } else {
            weight[lane] = lane < n ? r.decay_pow[h * (kC + 1) + n - 1 - lane] : 0.f;
        }
    }
    const int cols = r.vdim - e0 < kValueTile ? r.vdim - e0 : kValueTile;
    stage_transposed((const uint16_t*)r.v + row0 * r.ld + (int64_t)h * r.vdim + e0, r.ld, n, cols, kValueTile, vT, nullptr, nullptr);
    __syncthreads();
    stage_transposed((const uint16_t*)r.k + row0 * r.ld + (int64_t)h * r.dim, r.ld, n, r.dim, dp32, kH, kL, weight);
    __syncthreads();
    const int e = wave * 32;
    if (e < cols) {
        float* out = ws.states + (head * (ws.ep / 32) + (e0 + e) / 32) * (ws.dp / 16) * 512;
        u32x4 v[kC / 16];
#pragma unroll
        for (int k = 0; k < kC / 16; k++) v[k] = *(const u32x4*)(vT + (e + r32) * kRow + k * 16 + hi * 8);
        for (int d = 0; d < dp32; d += 32) {
            f32x16 acc;
#pragma unroll
            for (int i = 0; i < 16; i++) acc[i] = 0.f;
#pragma unroll
            for (int k = 0; k < kC / 16; k++) {
                acc = mfma_bf16(*(const u32x4*)(kH + (d + r32) * kRow + k * 16 + hi * 8), v[k], acc);
                acc = mfma_bf16(*(const u32x4*)(kL + (d + r32) * kRow + k * 16 + hi * 8), v[k], acc);
            }
            // a lane holds value r32 and features d + 8 g + 4 hi .. + 3 for g = 0 .. 3
#pragma unroll
            for (int g = 0; g < 4; g++)
                if (d + 8 * g < ws.dp)
                    *(f32x4*)(out + (d / 16 + g / 2) * 512 + hi * 256 + (r32 + 32 * (g & 1)) * 4) =
                        f32x4{acc[4 * g], acc[4 * g + 1], acc[4 * g + 2], acc[4 * g + 3]};
        }
    }
    if (GATED && e0 == 0)
        for (int d = tid; d < ws.dp; d += 256) {
            float sum = 0.f;
            for (int s = 0; s < kC; s++) sum += bf16_bits_to_f32(kH[d * kRow + s]) + bf16_bits_to_f32(kL[d * kRow + s]);
            ws.norms[head * ws.dp + d] = sum;
        }
}

// A thread carries eight features of one value's row of S (or of n, behind them) through the chunks.
template <bool GATED>
__global__ __launch_bounds__(256) void chunk_carry_kernel(Recurrence r, ChunkWs ws) {
    const int h = blockIdx.y, b = blockIdx.z, per = ws.dp / 8, total = ws.ep * per;
    const int item = blockIdx.x * 256 + threadIdx.x;
    const bool is_n = GATED && item >= total && item < total + per;
    if (item >= total && !is_n) return;
    const int block = item / 64, lane = item % 64;
    const int e = is_n ? 0 : block / (ws.dp / 16) * 32 + lane % 32, d0 = is_n ? (item - total) * 8 : block % (ws.dp / 16) * 16 + lane / 32 * 8;
    const int64_t head = (int64_t)b * r.heads + h, heads = (int64_t)r.batch * r.heads;
    const int slices = (r.vdim + kCols - 1) / kCols;
    float s[8];
#pragma unroll
    for (int i = 0; i < 8; i++)
        s[i] = d0 + i >= r.dim || e >= r.vdim ? 0.f : is_n ? r.n[head * slices * r.dim + d0 + i] : r.S[(head * r.dim + d0 + i) * r.vdim + e];
    float m = GATED ? r.m[head * slices] : 0.f;
    float* at = is_n ? ws.norms + head * ws.dp + d0 : ws.states + head * ws.ep * ws.dp + block * 512 + lane * 4;
    const int64_t step = is_n ? heads * ws.dp : heads * ws.ep * ws.dp, second = is_n ? 4 : 256;  // floats to the other four
    const int last = (int)(r.s - (int64_t)(ws.chunks - 1) * kC);
    f32x4 x[2], y[2];  // the next chunk's sums are requested before this chunk's are used
    x[0] = *(const f32x4*)at;
    x[1] = *(const f32x4*)(at + second);
    for (int c = 0; c < ws.chunks; c++, at += step) {
        if (c + 1 < ws.chunks) {
            y[0] = *(const f32x4*)(at + step);
            y[1] = *(const f32x4*)(at + step + second);
        }
        float keep, take = 1.f;
        if (GATED) {
            const int64_t g = c * heads + head;
            const float own = ws.gates[g * 2 + 1], top = fmaxf(m, own);
            keep = expf(m - top);
            take = expf(own - top);
            if (item == 0) ws.m_start[g] = m;
            m = ws.gates[g * 2] + top;
        } else {
            keep = r.decay_pow[h * (kC + 1) + (c + 1 < ws.chunks ? kC : last)];
        }
        if (is_n) {
            ((f32x4*)at)[0] = f32x4{s[0], s[1], s[2], s[3]};
            ((f32x4*)at)[1] = f32x4{s[4], s[5], s[6], s[7]};
        } else {
            u32x4 high, low;
#pragma unroll
            for (int i = 0; i < 4; i++) {
                high[i] = pack_bf16(s[2 * i], s[2 * i + 1]);
                low[i] = pack_bf16(low_part(s[2 * i]), low_part(s[2 * i + 1]));
            }
            *(u32x4*)at = high;
            *(u32x4*)(at + second) = low;
        }
#pragma unroll
        for (int i = 0; i < 8; i++) s[i] = fmaf(take, x[i >> 2][i & 3], keep * s[i]);
        x[0] = y[0];
        x[1] = y[1];
    }
#pragma unroll
    for (int i = 0; i < 8; i++) {
        if (d0 + i >= r.dim || e >= r.vdim) continue;
        if (is_n)
            for (int k = 0; k < slices; k++) r.n[(head * slices + k) * r.dim + d0 + i] = s[i];
        else
            r.S[(head * r.dim + d0 + i) * r.vdim + e] = s[i];
    }
    // m is read by every workgroup of the head and written by none here: chunk_outputs' launch does it
}

// Both products transposed: scores^T = K Q^T and o^T = S^T-part + V^T P^T, so that a lane holds one position's scores and
// its results. Two wavefronts a half of the chunk's positions, each with ET tiles of 32 values.
template <bool GATED, int DT, int ET>
__global__ __launch_bounds__(256) void chunk_outputs_kernel(Recurrence r, ChunkWs ws) {
    constexpr int kKey = DT * 16 + 8;
    __shared__ __align__(16) uint16_t ks[kC * kKey];
    __shared__ __align__(16) uint16_t qs[DT <= 8 ? kC * kKey : 1];  // up to 128 features; more would not leave room for two workgroups
    __shared__ __align__(16) uint16_t vT[2 * ET * 32 * kRow];
    __shared__ float as[kC], bs[kC], tops[kC], n0[DT * 16], pw[kC + 1];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r32 = lane & 31, hi = lane >> 5;
    constexpr int kTile = 2 * ET * 32;
    const int chunk = blockIdx.x, h = blockIdx.y, vt = (r.vdim + kTile - 1) / kTile, b = blockIdx.z / vt, e0 = (blockIdx.z % vt) * kTile;
    const int64_t row0 = b * r.s + (int64_t)chunk * kC;
    const int n = r.s - (int64_t)chunk * kC < kC ? (int)(r.s - (int64_t)chunk * kC) : kC;
    const int64_t head = (int64_t)(chunk * r.batch + b) * r.heads + h;
    const float m0 = GATED ? ws.m_start[head] : 0.f;
    const int cols = r.vdim - e0 < kTile ? r.vdim - e0 : kTile;
    if (GATED) {
        if (wave == 0) {
            float a, bb, top;
            chunk_gates(r, row0, n, h, lane, &a, &bb, &top);
            as[lane] = a;
            bs[lane] = bb;
            tops[lane] = fmaxf(m0, top);
            if (lane == n - 1 && chunk == ws.chunks - 1 && e0 == 0) {  // m behind the last position
                const int slices = (r.vdim + kCols - 1) / kCols;
                for (int k = 0; k < slices; k++) r.m[((int64_t)b * r.heads + h) * slices + k] = bb + fmaxf(m0, top);
            }
        }
        for (int d = tid; d < DT * 16; d += 256) n0[d] = d < ws.dp ? ws.norms[head * ws.dp + d] : 0.f;
    } else if (tid <= kC) {
        pw[tid] = r.decay_pow[h * (kC + 1) + tid];
    }
    {
        const uint16_t* k = (const uint16_t*)r.k + row0 * r.ld + (int64_t)h * r.dim;
        for (int item = tid; item < kC * DT * 2; item += 256) {
            const int s = item / (DT * 2), p = item % (DT * 2);
            u32x4 v = {0, 0, 0, 0};
            if (s < n && p * 8 < r.dim) v = *(const u32x4*)(k + (int64_t)s * r.ld + p * 8);
            *(u32x4*)(ks + s * kKey + p * 8) = v;
            if constexpr (DT <= 8) {
                v = u32x4{0, 0, 0, 0};
                if (s < n && p * 8 < r.dim) v = *(const u32x4*)((const uint16_t*)r.q + (row0 + s) * r.ld + (int64_t)h * r.dim + p * 8);
                *(u32x4*)(qs + s * kKey + p * 8) = v;
            }
        }
    }
    stage_transposed((const uint16_t*)r.v + row0 * r.ld + (int64_t)h * r.vdim + e0, r.ld, n, cols, kTile, vT, nullptr, nullptr);
    const int t = (wave >> 1) * 32 + r32, e1 = (wave & 1) * ET * 32;  // this lane's position; the wavefront's first value
    u32x4 q[DT];
    if constexpr (DT > 8) {
        const uint16_t* qr = (const uint16_t*)r.q + (row0 + (t < n ? t : n - 1)) * r.ld + (int64_t)h * r.dim + hi * 8;
#pragma unroll
        for (int k = 0; k < DT; k++) {
            q[k] = u32x4{0, 0, 0, 0};
            if (k * 16 + hi * 8 < r.dim) q[k] = *(const u32x4*)(qr + k * 16);
        }
    }
    __syncthreads();
    if constexpr (DT <= 8) {
#pragma unroll
        for (int k = 0; k < DT; k++) q[k] = *(const u32x4*)(qs + t * kKey + k * 16 + hi * 8);
    }
    const float inter = (GATED ? expf(m0 - tops[t]) : pw[t + 1]) * r.q_scale;
    f32x16 acc[ET];
#pragma unroll
    for (int et = 0; et < ET; et++)
#pragma unroll
        for (int i = 0; i < 16; i++) acc[et][i] = 0.f;
    // from the state at the chunk's start
#pragma unroll
    for (int et = 0; et < ET; et++) {
        const int block = (e0 + e1 + et * 32) / 32;
        if (block >= ws.ep / 32) break;
        const float* S = ws.states + (head * (ws.ep / 32) + block) * (ws.dp / 16) * 512 + lane * 4;
#pragma unroll
        for (int k = 0; k < DT; k++) {
            if (k * 16 < ws.dp) {  // dp is a multiple of 16
                acc[et] = mfma_bf16(*(const u32x4*)(S + k * 512), q[k], acc[et]);
                acc[et] = mfma_bf16(*(const u32x4*)(S + k * 512 + 256), q[k], acc[et]);
            }
        }
#pragma unroll
        for (int i = 0; i < 16; i++) acc[et][i] *= inter;
    }
    // from the chunk's own positions, 32 at a time
    float nq = 0.f;
#pragma unroll
    for (int sb = 0; sb < 2; sb++) {
        if (sb > (wave >> 1)) break;  // later than all of this wavefront's positions
        f32x16 sc;
#pragma unroll
        for (int i = 0; i < 16; i++) sc[i] = 0.f;
#pragma unroll
        for (int k = 0; k < DT; k++) sc = mfma_bf16(*(const u32x4*)(ks + (sb * 32 + r32) * kKey + k * 16 + hi * 8), q[k], sc);
        float p[16];
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const int s = sb * 32 + (i & 3) + 8 * (i >> 2) + 4 * hi;
            const float w = s > t ? 0.f : GATED ? expf(as[s] - tops[t]) : pw[t - s];
            p[i] = sc[i] * r.q_scale * w;
            nq += p[i];
        }
#pragma unroll
        for (int half = 0; half < 2; half++) {  // sixteen positions each, in the order the registers hold them
            u32x4 high, low;
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const float x = p[half * 8 + 2 * i], y = p[half * 8 + 2 * i + 1];
                high[i] = pack_bf16(x, y);
                low[i] = pack_bf16(low_part(x), low_part(y));
            }
#pragma unroll
            for (int et = 0; et < ET; et++) {
                const uint16_t* v = vT + (e1 + et * 32 + r32) * kRow + sb * 32 + half * 16 + hi * 4;
                const u32x2 v0 = *(const u32x2*)v, v1 = *(const u32x2*)(v + 8);
                const u32x4 a = {v0[0], v0[1], v1[0], v1[1]};
                acc[et] = mfma_bf16(a, high, acc[et]);
                acc[et] = mfma_bf16(a, low, acc[et]);
            }
        }
    }
    float inv = 1.f;
    if (GATED) {
        float n_q = 0.f;
#pragma unroll
        for (int k = 0; k < DT; k++)
#pragma unroll
            for (int i = 0; i < 8; i++) {
                const uint32_t w = q[k][i >> 1];
                n_q = fmaf(n0[k * 16 + hi * 8 + i], __uint_as_float(i & 1 ? w & 0xffff0000u : w << 16), n_q);
            }
        nq = fmaf(n_q, inter, nq);
        nq += __shfl_xor(nq, 32);
        inv = 1.f / (fmaxf(fabsf(nq), expf(-(bs[t] + tops[t]))) + 1e-6f);
    }
    if (t >= n) return;
    float* out = r.out + (row0 + t) * r.ldo + (int64_t)h * r.vdim + e0;
#pragma unroll
    for (int et = 0; et < ET; et++)
#pragma unroll
        for (int g = 0; g < 4; g++) {
            const int e = e1 + et * 32 + 8 * g + 4 * hi;
            if (e >= cols) continue;  // cols is a multiple of 8
            *(f32x4*)(out + e) = f32x4{acc[et][4 * g] * inv, acc[et][4 * g + 1] * inv, acc[et][4 * g + 2] * inv, acc[et][4 * g + 3] * inv};
        }
}

template <bool GATED, int DT>
void launch_outputs(const Recurrence& r, const ChunkWs& ws, hipStream_t st) {
    if (r.vdim <= 64)
        hipLaunchKernelGGL((chunk_outputs_kernel<GATED, DT, 1>), dim3((unsigned)ws.chunks, (unsigned)r.heads, (unsigned)r.batch), dim3(256), 0, st, r, ws);
    else
        hipLaunchKernelGGL((chunk_outputs_kernel<GATED, DT, 2>), dim3((unsigned)ws.chunks, (unsigned)r.heads, (unsigned)(r.batch * ((r.vdim + 127) / 128))),
                           dim3(256), 0, st, r, ws);
}

template <bool GATED>
hipError_t launch_chunks(const Recurrence& r, const ChunkWs& ws, hipStream_t st) {
    const size_t lds = (size_t)(kValueTile + 2 * ((ws.dp + 31) / 32 * 32)) * kRow * 2;
    if (lds > 64 * 1024) {
        hipError_t e = hipFuncSetAttribute((const void*)chunk_states_kernel<GATED>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    const unsigned vt = (unsigned)((r.vdim + kValueTile - 1) / kValueTile);
    hipLaunchKernelGGL(chunk_states_kernel<GATED>, dim3((unsigned)ws.chunks, (unsigned)r.heads, (unsigned)r.batch * vt), dim3(256), lds, st, r, ws);
    const int items = (ws.ep + (GATED ? 1 : 0)) * ws.dp / 8;
    hipLaunchKernelGGL(chunk_carry_kernel<GATED>, dim3((unsigned)((items + 255) / 256), (unsigned)r.heads, (unsigned)r.batch), dim3(256), 0, st, r, ws);
    if (ws.dp <= 32) launch_outputs<GATED, 2>(r, ws, st);
    else if (ws.dp <= 64) launch_outputs<GATED, 4>(r, ws, st);
    else if (ws.dp <= 128) launch_outputs<GATED, 8>(r, ws, st);
    else launch_outputs<GATED, 16>(r, ws, st);
    return hipGetLastError();
}

int chunk_dp(int dim) { return (dim + 15) / 16 * 16; }

}  // namespace

int recurrence_slices(int vdim) { return (vdim + kCols - 1) / kCols; }

hipError_t recurrence_scan(const Recurrence& r, hipStream_t st) {
    if (r.batch * r.s == 0) return hipSuccess;
    if (r.dim > kRecurrenceMaxDim) return hipErrorInvalidValue;
    if (r.gates) launch_scan<true>(r, st);
    else launch_scan<false>(r, st);
    return hipGetLastError();
}

bool recurrence_chunks_ok(const Recurrence& r) {
    auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    return r.bf16 && r.dim % 8 == 0 && r.vdim % 8 == 0 && r.ld % 8 == 0 && r.ldo % 4 == 0 && r.dim <= kRecurrenceMaxDim && aligned(r.q) && aligned(r.k) &&
           aligned(r.v) && aligned(r.out) && (r.s + kC - 1) / kC < 65536;
}

size_t recurrence_chunk_ws_floats(int batch, int heads, int dim, int vdim, int64_t s) {
    const int64_t dp = chunk_dp(dim);
    return (size_t)((s + kC - 1) / kC) * batch * heads * ((vdim + 31) / 32 * 32 * dp + dp + 4) + 64;
}

hipError_t recurrence_chunks(const Recurrence& r, hipStream_t st) {
    if (r.batch * r.s == 0) return hipSuccess;
    if (!recurrence_chunks_ok(r) || !r.ws) return hipErrorInvalidValue;
    ChunkWs ws;
    ws.dp = chunk_dp(r.dim);
    ws.chunks = (int)((r.s + kC - 1) / kC);
    const size_t heads = (size_t)ws.chunks * r.batch * r.heads;
    ws.states = r.ws;
    ws.ep = (r.vdim + 31) / 32 * 32;
    ws.norms = ws.states + heads * ws.ep * ws.dp;
    ws.gates = ws.norms + heads * ws.dp;
    ws.m_start = ws.gates + heads * 2;
    return r.gates ? launch_chunks<true>(r, ws, st) : launch_chunks<false>(r, ws, st);
}

}  // namespace mimir
