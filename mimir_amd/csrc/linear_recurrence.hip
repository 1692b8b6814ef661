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

}  // namespace

int recurrence_slices(int vdim) { return (vdim + kCols - 1) / kCols; }

hipError_t recurrence_scan(const Recurrence& r, hipStream_t st) {
    if (r.batch * r.s == 0) return hipSuccess;
    if (r.dim > kRecurrenceMaxDim) return hipErrorInvalidValue;
    if (r.gates) launch_scan<true>(r, st);
    else launch_scan<false>(r, st);
    return hipGetLastError();
}

}  // namespace mimir
