// One tile of Y = X . P^T for two 16-bit operands whose rows run along K, on the matrix cores: the body that the products
// over a binary16 panel (qgemm_f16_panel.hip) and over bfloat16 weights (gemm_bf16.hip) share. What happens to a result
// is the caller's (a store object); the operands' element type is a parameter.
//
// A workgroup is eight wavefronts; steps of 64 along K go through two stages of LDS. Both operands go from global memory
// straight into LDS (global_load_lds_dwordx4: no registers, no vector arithmetic in the wavefronts that share a SIMD with
// the MFMAs); a row of a stage is 128 bytes and its eight 16-byte pieces are placed at piece ^ (row / 2 mod 8), which the
// loading lane undoes in the address it reads from, so that the fragment reads of v_mfma_f32_32x32x16 (32 rows, the
// same piece) spread over all banks. The loads of the next step are issued in two parts with the first two of a step's
// four groups of MFMAs (issued later they had not landed by the step's end, issued all at once they hold the wavefront
// up), and the fragments of the next group are read while the current group multiplies.
#pragma once
#include "device_util.h"

namespace mimir {

namespace {

typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr int kStep = 64;              // of K a step
constexpr int kRowBytes = kStep * 2;   // a row of a stage in LDS

// A workgroup's tile of Y: WM x (8 / WM) wavefronts of (32 MT) x (32 NT) each.
template <int WM, int MT, int NT>
struct Tile {
    static constexpr int WN = 8 / WM, kMT = MT, kNT = NT;
    static constexpr int BM = WM * 32 * MT, BN = WN * 32 * NT;
    static constexpr int kRows = BM + BN;                // rows of a stage: X's, then P's
    static constexpr int kLoads = kRows / 64;            // 1 KB loads (8 rows) a wavefront issues per step
    static constexpr int kStageBytes = kRows * kRowBytes;
    static_assert(kRows % 64 == 0 && BM % 8 == 0, "whole loads, none across the two operands");
};
using Wide = Tile<2, 4, 2>;    // 256 x 256: the most MFMAs per byte read from LDS (0.75 fragment reads an MFMA)
using Narrow = Tile<4, 2, 3>;  // 256 x 192: three quarters of a Wide tile, to fill a last round that Wide tiles would leave a quarter empty
using Low = Tile<2, 2, 2>;     // 128 x 256: for products with too few Wide tiles for the device
using Tiny = Tile<2, 1, 1>;    // 64 x 128: for those with too few Low tiles

struct F16Element {
    static __device__ __forceinline__ f32x16 mfma(u32x4 a, u32x4 b, f32x16 c) {
        return __builtin_amdgcn_mfma_f32_32x32x16_f16(__builtin_bit_cast(f16x8, a), __builtin_bit_cast(f16x8, b), c, 0, 0, 0);
    }
};
struct Bf16Element {
    static __device__ __forceinline__ f32x16 mfma(u32x4 a, u32x4 b, f32x16 c) {
        return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
    }
};

// 16 bytes a lane from global memory into LDS: lane l's piece lands at lds_base + 16 l. Written out because the
// compiler, given the builtin, waits for every load under way before any LDS access; these loads are counted by hand.
// The instruction takes its LDS base from M0, which the compiler does not let an asm statement name as clobbered: nothing
// else in this kernel uses M0 (no dynamically indexed registers, no LDS-direct reads), and it is set anew before every load.
__device__ __forceinline__ void load_to_lds(const void* g, uint32_t lds_base) {
    asm volatile("s_mov_b32 m0, %0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(lds_base), "v"(g) : "memory");
}
__device__ __forceinline__ void wait_loads() { asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); }
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// Y [m0 .. m0 + BM) x [n0 .. n0 + BN) of X [M, K] (rows ldx apart) by P [N, K] (rows ldp apart), float32 sums; K a
// multiple of 64, rows 16-byte aligned. store.row(m, M) is called once a row (also for rows past M), then
// store(m, n, N, its value, v) with the results of columns n .. n + 3 (n < N; those past N are not to be stored).
// After the first store.first_steps(steps) of the steps of K the sums so far are multiplied by store.mid(n, N) (called for
// columns past N too); a store object without such a factor returns `steps`.
template <class T, class E, class S>
__device__ __forceinline__ void tile_body(const uint16_t* __restrict__ X16, int64_t ldx, const uint16_t* __restrict__ P, int64_t ldp, const S& store, int M,
                                          int N, int K, int m0, int n0, char* lds) {
    constexpr int MT = T::kMT, NT = T::kNT;
    constexpr int kLoads = T::kLoads;
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = wave / T::WN, wn = wave % T::WN;

    // This wavefront's loads: load g = kLoads wave + j brings rows [8 g, 8 g + 8) of the stage, X's below BM and P's
    // from there. Rows past the matrix re-read its last row (their results are not stored).
    const char* from[kLoads];
    uint32_t into[kLoads];
#pragma unroll
    for (int j = 0; j < kLoads; j++) {
        const int first = 8 * (kLoads * wave + j);
        const int row = first + (lane >> 3);
        const int piece = (lane & 7) ^ ((row >> 1) & 7);
        const uint16_t* base;
        if (first < T::BM) {
            const int m = m0 + row < M ? m0 + row : M - 1;
            base = X16 + (size_t)m * ldx;
        } else {
            const int n = n0 + row - T::BM < N ? n0 + row - T::BM : N - 1;
            base = P + (size_t)n * ldp;
        }
        from[j] = (const char*)(base + 8 * piece);
        into[j] = (uint32_t)(first * kRowBytes);
    }
    const uint32_t lds0 = (uint32_t)(uintptr_t)lds;

    const int r32 = lane & 31, hi = lane >> 5;
    const int swz = (r32 >> 1) & 7;
    int piece_off[4];
#pragma unroll
    for (int kk = 0; kk < 4; kk++) piece_off[kk] = ((2 * kk + hi) ^ swz) * 16;
    const int a_row = (wm * 32 * MT + r32) * kRowBytes, b_row = (T::BM + wn * 32 * NT + r32) * kRowBytes;

    f32x16 acc[MT][NT];
#pragma unroll
    for (int mt = 0; mt < MT; mt++)
#pragma unroll
        for (int nt = 0; nt < NT; nt++)
#pragma unroll
            for (int i = 0; i < 16; i++) acc[mt][nt][i] = 0.f;

    const int nk = K / kStep;
#pragma unroll
    for (int j = 0; j < kLoads; j++) {
        load_to_lds(from[j], __builtin_amdgcn_readfirstlane(lds0 + into[j]));
        from[j] += kRowBytes;
    }
    const int first = store.first_steps(nk);
    for (int i = 0; i < nk; i++) {
        if (i == first) {  // the sums over the first steps have a factor of their own (a lane has one column)
#pragma unroll
            for (int nt = 0; nt < NT; nt++) {
                const float f = store.mid(n0 + wn * 32 * NT + nt * 32 + r32, N);
#pragma unroll
                for (int mt = 0; mt < MT; mt++)
#pragma unroll
                    for (int e = 0; e < 16; e++) acc[mt][nt][e] *= f;
            }
        }
        wait_loads();   // this wavefront's part of step i has landed
        lds_barrier();  // everyone's has, and everyone has read the other stage for the last time
        const bool more = i + 1 < nk;
        const uint32_t next = lds0 + ((i + 1) & 1) * T::kStageBytes;
        const char* st = lds + (i & 1) * T::kStageBytes;
        u32x4 a[2][MT], b[2][NT];
#pragma unroll
        for (int mt = 0; mt < MT; mt++) a[0][mt] = *(const u32x4*)(st + a_row + mt * 32 * kRowBytes + piece_off[0]);
#pragma unroll
        for (int nt = 0; nt < NT; nt++) b[0][nt] = *(const u32x4*)(st + b_row + nt * 32 * kRowBytes + piece_off[0]);
#pragma unroll
        for (int kk = 0; kk < 4; kk++) {
            const int c = kk & 1, n = c ^ 1;
            if (more && kk < 2) {  // half of the next step's loads: all of them early in the step, so that they have landed by its end
#pragma unroll
                for (int j = kk * kLoads / 2; j < (kk + 1) * kLoads / 2; j++) {
                    load_to_lds(from[j], __builtin_amdgcn_readfirstlane(next + into[j]));
                    from[j] += kRowBytes;
                }
            }
            if (kk + 1 < 4) {
#pragma unroll
                for (int mt = 0; mt < MT; mt++) a[n][mt] = *(const u32x4*)(st + a_row + mt * 32 * kRowBytes + piece_off[kk + 1]);
#pragma unroll
                for (int nt = 0; nt < NT; nt++) b[n][nt] = *(const u32x4*)(st + b_row + nt * 32 * kRowBytes + piece_off[kk + 1]);
            }
#pragma unroll
            for (int mt = 0; mt < MT; mt++)
#pragma unroll
                for (int nt = 0; nt < NT; nt++) acc[mt][nt] = E::mfma(a[c][mt], b[c][nt], acc[mt][nt]);
            if (kk + 1 < 4) {  // one fragment read between two MFMAs
#pragma unroll
                for (int q = 0; q < MT + NT; q++) {
                    __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
                    __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
                }
                if (MT * NT > MT + NT) __builtin_amdgcn_sched_group_barrier(0x008, MT * NT - MT - NT, 0);
            }
        }
    }

    // An MFMA leaves a lane one column of Y and four consecutive rows per group of four registers; a 4 x 4
    // transposition within each quad of lanes turns that into one row and four consecutive columns a lane, so that a
    // group is stored with one wide store a lane instead of four narrow ones (the stores of the untransposed form took
    // 5 % of the launch).
#pragma unroll
    for (int mt = 0; mt < MT; mt++)
#pragma unroll
        for (int q = 0; q < 4; q++) {
            const int m = m0 + wm * 32 * MT + mt * 32 + q * 8 + hi * 4 + (lane & 3);
            const float of_row = store.row(m, M);
#pragma unroll
            for (int nt = 0; nt < NT; nt++) {
                float v[4] = {acc[mt][nt][4 * q], acc[mt][nt][4 * q + 1], acc[mt][nt][4 * q + 2], acc[mt][nt][4 * q + 3]};
                quad_transpose(v, lane);
                const int n = n0 + wn * 32 * NT + nt * 32 + (r32 & ~3);
                if (m >= M || n >= N) continue;
                store(m, n, N, of_row, v);
            }
        }
}

// A die's workgroups (every eighth, round-robin) take a contiguous range of the tiles, the tile's row of X varying
// fastest: the 32 that run together share 4 column panels of P and the 8 row panels of X through the die's L2.
__device__ __forceinline__ int tile_of(int b, int ntiles) {
    const int per_die = (ntiles + 7) >> 3;
    return (b & 7) * per_die + (b >> 3);
}

}  // namespace

}  // namespace mimir
