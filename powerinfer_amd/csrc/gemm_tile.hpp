// The LDS-tiled matrix-core product of prompt chunks, shared by the dense mat-mul and the grouped one.
#pragma once
#include "kernels_common.hpp"
#include <type_traits>

namespace {

// ---------------------------------------------------------------------------------------------------
// Prompt chunks of any length on the matrix cores with both operands staged in LDS: y[t][row] = epi(W[row] . xn[t]).
// A workgroup of four waves owns BM weight rows x BN tokens; the reduction dimension advances 64 columns at a time through two
// LDS stages, and two more stages travel in registers as 16-byte global loads (one stage of MFMAs lasts about 0.2 us, less than a
// trip to HBM); one barrier per stage.  Both operands are stored row by row with the reduction dimension contiguous, which is
// the matrix cores' operand layout (eight consecutive columns per lane), so a fragment is one ds_read_b128.  A row is 128 bytes;
// its eight 16-byte pieces are stored at piece ^ (row & 7), so that the 16 rows a quarter wave reads the same piece of, and the
// eight pieces of a row that eight neighbouring lanes write, fall on different banks (the bank-conflict counter reads 0; with
// rows padded to 144 bytes instead it read a third of the LDS cycles).  A wave computes (BM/2) x (BN/2) outputs as 16 x 16
// tiles; per 32-column step it reads BM/32 + BN/32 fragments for (BM/32) * (BN/32) MFMAs.  Workgroups are numbered so that the
// token tiles of one row tile run on the same XCD back to back: the row tile's weights cross HBM once and are re-read from that
// XCD's L2.  cols % 64 == 0; rows and T need not fill the tiles (requests past the edge re-read the last row, results are not
// stored).
// ---------------------------------------------------------------------------------------------------
constexpr int kGtBK = 64;                        // columns per stage
constexpr int kGtRow = kGtBK * 2;                // bytes per LDS row
template <typename EL, int BM, int BN, int WGM, int WGN>      // element type, output tile and the waves' grid over it (WGM x WGN waves)
struct GemmTile {
    static constexpr int kThreads = 64 * WGM * WGN;
    static constexpr int WM = BM / WGM, WN = BN / WGN, MT = WM / 16, NT = WN / 16;
    static constexpr int ACH = BM * kGtBK * 2 / 16 / kThreads, BCH = BN * kGtBK * 2 / 16 / kThreads;  // 16-byte chunks per thread and stage
    static constexpr size_t kLds = (size_t)2 * (BM + BN) * kGtRow;
    static_assert(WM % 16 == 0 && WN % 16 == 0 && ACH * kThreads * 16 == BM * kGtBK * 2 && BCH * kThreads * 16 == BN * kGtBK * 2, "tile does not divide among the waves");
    // the tile row (of either operand) chunk j of this thread belongs to, and its first column within a stage
    static __device__ __forceinline__ int chunk_row(int j) { return j * (kThreads / 8) + (int)threadIdx.x / 8; }
    static __device__ __forceinline__ int chunk_col() { return ((int)threadIdx.x % 8) * 8; }

    // ga, gb: where this thread's chunks of the first stage lie; nk stages of kGtBK columns.  acc[m][n][r] belongs to the tile's row
    // wm * WM + m * 16 + 4 g + r and token wn * WN + n * 16 + i (lane = 16 g + i, wave = wn * WGM + wm)
    static __device__ __forceinline__ void run(unsigned char * smem, const EL * const (&ga)[ACH], const EL * const (&gb)[BCH], int nk, pi_f4 (&acc)[MT][NT]) {
        unsigned char * sa = smem;                                     // [2][BM][kGtRow]
        unsigned char * sb = smem + 2 * BM * kGtRow;                   // [2][BN][kGtRow]
        const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
        const int wm = wave % WGM, wn = wave / WGM;
        auto lds_off = [](int r, int kc) { return r * kGtRow + ((kc ^ (r & 7)) * 16); };
        int la[ACH], lb[BCH];
#pragma unroll
        for (int j = 0; j < ACH; ++j) la[j] = lds_off(chunk_row(j), tid % 8);
#pragma unroll
        for (int j = 0; j < BCH; ++j) lb[j] = lds_off(chunk_row(j), tid % 8);
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int n = 0; n < NT; ++n) acc[m][n] = pi_f4{0.0f, 0.0f, 0.0f, 0.0f};
        // Two column stages travel in registers while a third is being multiplied: stage kt sits in LDS half kt & 1, stages kt + 1 and
        // kt + 2 are in flight (one stage of MFMAs is about 0.2 us, less than a trip to HBM).
        pi_u32x4 ra[2][ACH], rb[2][BCH];
        auto fetch = [&](auto slot, int kt) {
            constexpr int S = decltype(slot)::value;
#pragma unroll
            for (int j = 0; j < ACH; ++j) ra[S][j] = pi_ld16(ga[j] + (size_t)kt * kGtBK);
#pragma unroll
            for (int j = 0; j < BCH; ++j) rb[S][j] = pi_ld16(gb[j] + (size_t)kt * kGtBK);
        };
        auto stash = [&](auto slot) {              // registers of slot S -> LDS half S
            constexpr int S = decltype(slot)::value;
            unsigned char * na = sa + S * BM * kGtRow; unsigned char * nb = sb + S * BN * kGtRow;
#pragma unroll
            for (int j = 0; j < ACH; ++j) *reinterpret_cast<pi_u32x4 *>(na + la[j]) = ra[S][j];
#pragma unroll
            for (int j = 0; j < BCH; ++j) *reinterpret_cast<pi_u32x4 *>(nb + lb[j]) = rb[S][j];
        };
        const std::integral_constant<int, 0> c0; const std::integral_constant<int, 1> c1;
        // every fetch and stash below is unconditional (past the last stage the last one is fetched again and stashed where nobody
        // reads): the count of loads in flight is then the same on every path, and the waits name exactly the loads they need
        const int last = nk - 1;
        fetch(c0, 0);
        fetch(c1, min(1, last));
        stash(c0);
        fetch(c0, min(2, last));
        __syncthreads();
        // the lane's two pieces (columns 8g.. of each 32-column step) of fragment row i: every 16-row tile starts on a multiple of 8
        const int koff[2] = {(g ^ (i & 7)) * 16, ((4 + g) ^ (i & 7)) * 16};
        const int frag_a = (wm * WM + i) * kGtRow, frag_b = (wn * WN + i) * kGtRow;
        // The fragments of a stage's first 32 columns are read while the previous stage's second 32 are multiplied, those of its second
        // 32 while its first are: every LDS read has a block of MFMAs between its issue and its use.
        pi_u32x4 f0a[MT], f0b[NT], f1a[MT], f1b[NT];
        auto frags = [&](auto par, auto half, pi_u32x4 * fa, pi_u32x4 * fb) {
            constexpr int P = decltype(par)::value, KS = decltype(half)::value;
            const unsigned char * ca = sa + P * BM * kGtRow + frag_a + koff[KS];
            const unsigned char * cb = sb + P * BN * kGtRow + frag_b + koff[KS];
#pragma unroll
            for (int m = 0; m < MT; ++m) fa[m] = *reinterpret_cast<const pi_u32x4 *>(ca + m * 16 * kGtRow);
#pragma unroll
            for (int n = 0; n < NT; ++n) fb[n] = *reinterpret_cast<const pi_u32x4 *>(cb + n * 16 * kGtRow);
        };
        auto mfmas = [&](const pi_u32x4 * fa, const pi_u32x4 * fb) {
#pragma unroll
            for (int m = 0; m < MT; ++m)
#pragma unroll
                for (int n = 0; n < NT; ++n)
                    acc[m][n] = mma16<EL>(fa[m], fb[n], acc[m][n]);
        };
        frags(c0, c0, f0a, f0b);
        auto step = [&](auto par, int kt) {
            constexpr int P = decltype(par)::value;
            const std::integral_constant<int, P ^ 1> other;
            frags(par, c1, f1a, f1b);
            __builtin_amdgcn_sched_barrier(0);
            mfmas(f0a, f0b);
            stash(other);
            fetch(other, min(kt + 3, last));
            __builtin_amdgcn_sched_barrier(0);
            __syncthreads();
            __builtin_amdgcn_sched_barrier(0);
            frags(other, c0, f0a, f0b);           // past the last stage: the re-stashed last stage, read and not used
            __builtin_amdgcn_sched_barrier(0);
            mfmas(f1a, f1b);
            __builtin_amdgcn_sched_barrier(0);
        };
        int kt = 0;
        for (; kt + 1 < nk; kt += 2) { step(c0, kt); step(c1, kt + 1); }
        if (kt < nk) step(c0, kt);
    }
};

}  // namespace
