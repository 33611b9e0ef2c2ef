// The wavefront-specialised 128 x 128 x 64 tile product, shared by the f16 kernel of gemm.hip and the segmented kernels of
// seg_gemm.hip.  A 512-thread workgroup holds four LOADER wavefronts and four
// MULTIPLIER wavefronts, one of each per SIMD, so the hardware interleaves their instruction streams:
//   * loaders copy the operand tiles global -> LDS with buffer_load_dwordx4 ... lds (every lane names a 16-byte source,
//     the 64 destinations are consecutive in LDS; no registers are spent on staging).  DMA_STAGES - 1 k-tiles (96 KiB) are
//     in flight per workgroup.  The XOR swizzle moves to the source side: the lane that fills physical granule pg of row
//     r fetches logical granule pg ^ ((r >> 1) & 7).  A wavefront's loads retire in order, so "at most 8*n outstanding"
//     means its part of the tile n behind the newest has landed.
//   * multipliers only read operand slices from LDS and issue MFMAs, software pipelined across slices and k-tiles.
// One barrier per k-tile, executed by all eight wavefronts, publishes tile kt+1 (loaders arrive once it has landed) and
// frees the buffer of tile kt (multipliers arrive once they have read it); the loaders then refill that buffer.
// The tile moves 32 KiB per k-tile for 16 MFMAs per SIMD (0.26 us at the ~2 GHz the clock settles at under MFMA load),
// i.e. needs ~125 B/ns from the CU's load path, which is about what that path delivers from the L2.
// Needs K % 16 == 0: a partial last k-tile runs fewer 16-wide steps; what its copies fetch beyond K is never multiplied.
// Both roles must run their function in the same workgroup with the same n_ktiles (>= 1): they meet at its barriers.
#pragma once
#include "gemm_common.hpp"

namespace {

constexpr int DMA_STAGES = 4;
constexpr int DMA_THREADS = 512;
constexpr size_t DMA_LDS_BYTES = size_t(DMA_STAGES) * 2 * TILE_HALFS * sizeof(half_t);

// The matrix core's 16-bit element types: operands travel as eight 16-bit patterns per lane either way.
struct MfmaF16 {
    static __device__ __forceinline__ float16_t mul(const half8_t &a, const half8_t &b, const float16_t &c) {
        return __builtin_amdgcn_mfma_f32_32x32x16_f16(a, b, c, 0, 0, 0);
    }
};
struct MfmaBf16 {
    static __device__ __forceinline__ float16_t mul(const half8_t &a, const half8_t &b, const float16_t &c) {
        return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
    }
};

// What a loader wavefront copies: both operands as buffers, a 32-bit byte offset per lane and instruction (at k = 0, fixed over
// the k-tiles), and how many bytes one k of the second operand is (2 for [N, K], 2 N for [K, N]).
struct DmaSource {
    const void *a, *w;
    int a_bytes, w_bytes;
    int off_a[4], off_w[4];
    int w_k_bytes;
};

// The loader's rows: this wavefront fills rows [32*role_wave, +32) of both tiles, 8 rows per instruction.
__device__ __forceinline__ int dma_row(int role_wave, int j, int lane) { return 32 * role_wave + 8 * j + (lane >> 3); }

// The copies use the buffer form: a scalar descriptor of the whole operand, one 32-bit offset register per lane (fixed over
// the k-tiles) and a scalar offset for the k-tile.  With 64-bit addresses in registers (two per lane) the copies of a wavefront
// whose SIMD also feeds the matrix core ran at half their rate (measured 66 against 117 B/ns per CU).  Reads past
// the end of the operand return zero, so a partial last k-tile needs no clamping (what lies beyond K is never
// multiplied).
__device__ __forceinline__ void dma_load_tiles(const DmaSource &s, half_t *lds_dma, int k_begin, int n_ktiles, int role_wave) {
    auto issue = [&](int kt) {
        half_t *stage = lds_dma + size_t(kt % DMA_STAGES) * 2 * TILE_HALFS;
        // the k-tile enters through the descriptors' base and size: the range check that turns reads past the end of the
        // operand into zeros does not see an instruction's scalar offset
        const int k_off = (k_begin + kt * BK) * 2;
        const int kw_off = (k_begin + kt * BK) * s.w_k_bytes; // (rows of [K, N] past K lie past the end: zeros)
        const __amdgpu_buffer_rsrc_t rs_a =
            __builtin_amdgcn_make_buffer_rsrc(const_cast<char *>(reinterpret_cast<const char *>(s.a)) + k_off, 0, s.a_bytes - k_off, 0x00020000);
        const __amdgpu_buffer_rsrc_t rs_w =
            __builtin_amdgcn_make_buffer_rsrc(const_cast<char *>(reinterpret_cast<const char *>(s.w)) + kw_off, 0, s.w_bytes - kw_off, 0x00020000);
#pragma unroll
        for (int j = 0; j < 4; j++) {
            __builtin_amdgcn_raw_ptr_buffer_load_lds(rs_a, (__attribute__((address_space(3))) void *)(stage + (32 * role_wave + 8 * j) * BK), 16,
                                                     s.off_a[j], 0, 0, 0);
            __builtin_amdgcn_raw_ptr_buffer_load_lds(
                rs_w, (__attribute__((address_space(3))) void *)(stage + TILE_HALFS + (32 * role_wave + 8 * j) * BK), 16, s.off_w[j], 0, 0, 0);
        }
    };
    int issued = 0; // k-tiles whose copies have been issued
    // this wavefront's part of tile kt has landed once at most 8 * (issued - 1 - kt) of its copies are outstanding
    auto wait_tile = [&](int kt) {
        const int newer = issued - 1 - kt;
        if (newer >= 2) wait_vmcnt<16>();
        else if (newer == 1) wait_vmcnt<8>();
        else wait_vmcnt<0>();
    };
    for (; issued < DMA_STAGES - 1 && issued < n_ktiles; issued++) issue(issued);
    wait_tile(0);
    lds_barrier(); // tile 0 is visible
    for (int kt = 0; kt < n_ktiles; kt++) {
        // past the barrier that published tile kt nobody reads tile kt-1 any more: its buffer takes tile kt + DMA_STAGES - 1
        if (issued < n_ktiles) {
            issue(issued);
            issued++;
        }
        if (kt + 1 < n_ktiles) {
            wait_tile(kt + 1);
            lds_barrier(); // publishes tile kt+1
        }
    }
}

// Two neighbouring stages (32768 halfs from the returned one on) that the last k-tile does not occupy: free for an epilogue as
// soon as the products are done (every copy into them has landed).
__device__ __forceinline__ half_t *dma_free_stages(half_t *lds_dma, int n_ktiles) {
    const int last = (n_ktiles - 1) % DMA_STAGES, free0 = last == 0 ? 1 : last == 1 ? 2 : 0;
    return lds_dma + size_t(free0) * 2 * TILE_HALFS;
}

// A multiplier wavefront's 64 x 64 sub-tile of the product: acc[ni][mi], element v of lane l is
// n = 32 ni + 8 (v / 4) + 4 (l / 32) + v % 4, m = 32 mi + l % 32.
// BKN: the second operand is [K, N] (hgemm.zig's layout) and is read as it lies.  Its tile sits in LDS as [k][128 n]; a
// loader instruction copies four k-rows of 256 bytes, the 16-byte granules of row r XOR-ed with 2 * (r & 3) on the source
// side, and the multipliers fetch their operand slices with the transposing LDS load (ds_read_b64_tr_b16: the 16 lanes of a
// quarter-wavefront name a 4 x 16 block, four halfs each, and lane i receives column i of its four rows), two per slice in
// place of one 16-byte read.  Same products in the same order as with the [N, K] operand: the same bits.  Needs N % 8 == 0.
template <class Op, bool BKN>
__device__ __forceinline__ void dma_multiply_tiles(float16_t (&acc)[2][2], int k_begin, int k_end, int n_ktiles, int wm, int wn, int lane) {
    const int frag_row = lane & 31, frag_g = lane >> 5;
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int v = 0; v < 16; v++) acc[i][j][v] = 0.0f;

    // LDS byte offsets (within a stage) of this lane's operand slices: [16-wide step][row block]
    unsigned off_a[BK / 16][2], off_w[BK / 16][2];
#pragma unroll
    for (int s = 0; s < BK / 16; s++)
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const int rm = wm * 64 + i * 32 + frag_row;
            const int rn = wn * 64 + i * 32 + frag_row;
            off_a[s][i] = (rm * BK + swz(rm, 2 * s + frag_g) * 8) * 2;
            off_w[s][i] = (TILE_HALFS + rn * BK + swz(rn, 2 * s + frag_g) * 8) * 2;
        }
    // BKN: where this lane points the transposing loads of n-block ni, for the first four k of its slice of step 0 (step s and
    // the second four add (16 s + 4 q) rows of 256 bytes): row 8 * frag_g + i / 4, columns 4 * (i % 4) .. + 3 of the 16 the
    // lane's quarter-wavefront covers, i = lane % 16
    unsigned off_wk[2];
#pragma unroll
    for (int ni = 0; ni < 2; ni++) {
        const int i = lane & 15, row = 8 * frag_g + (i >> 2);
        const int c = wn * 8 + ni * 4 + ((lane >> 4) & 1) * 2 + ((i & 3) >> 1); // 16-byte granule of the row
        off_wk[ni] = (TILE_HALFS + row * BN + (c ^ (2 * (row & 3))) * 8 + (i & 1) * 4) * 2;
    }
    // The operand reads and the waits for them are written out by hand.  Left to the compiler the reads sink below the
    // MFMAs of the step before (into the registers those just consumed) and are waited for at once, and the wait at the
    // head of the loop is for everything outstanding, so the LDS latency is paid several times per k-tile with the matrix
    // core idle.  The compiler does not count reads issued from asm statements, so it adds no waits of its own for them;
    // each wait statement names the registers it guards as operands, which keeps their use behind it.
    constexpr unsigned STAGE_BYTES = 2 * TILE_HALFS * sizeof(half_t);
    // (BKN: fw[ni] arrives as two 8-byte halves, wk[ni][0..1])
    struct Frag {
        half8_t fa[2], fw[2];
        half4_t wk[2][2];
    };
    auto read_frags = [&](int kt, int s, Frag &f) {
        const unsigned sb = unsigned(kt % DMA_STAGES) * STAGE_BYTES;
#pragma unroll
        for (int i = 0; i < 2; i++) {
            asm volatile("ds_read_b128 %0, %1" : "=v"(f.fa[i]) : "v"(sb + off_a[s][i]));
            if (!BKN) asm volatile("ds_read_b128 %0, %1" : "=v"(f.fw[i]) : "v"(sb + off_w[s][i]));
            else {
#pragma unroll
                for (int q = 0; q < 2; q++)
                    asm volatile("ds_read_b64_tr_b16 %0, %1" : "=v"(f.wk[i][q]) : "v"(sb + off_wk[i] + unsigned(16 * s + 4 * q) * (BN * 2)));
            }
        }
    };
    // all but the newest group of reads (the one issued last: four reads, six with BKN) have landed; f belongs to an older group
    auto wait_older = [&](Frag &f) {
        if (!BKN) asm volatile("s_waitcnt lgkmcnt(4)" : "+v"(f.fa[0]), "+v"(f.fa[1]), "+v"(f.fw[0]), "+v"(f.fw[1])::"memory");
        else
            asm volatile("s_waitcnt lgkmcnt(6)" : "+v"(f.fa[0]), "+v"(f.fa[1]), "+v"(f.wk[0][0]), "+v"(f.wk[0][1]), "+v"(f.wk[1][0]), "+v"(f.wk[1][1])::"memory");
    };
    auto wait_all = [&](Frag &f) {
        if (!BKN) asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(f.fa[0]), "+v"(f.fa[1]), "+v"(f.fw[0]), "+v"(f.fw[1])::"memory");
        else
            asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(f.fa[0]), "+v"(f.fa[1]), "+v"(f.wk[0][0]), "+v"(f.wk[0][1]), "+v"(f.wk[1][0]), "+v"(f.wk[1][1])::"memory");
    };
    auto multiply = [&](const Frag &f) {
#pragma unroll
        for (int ni = 0; ni < 2; ni++) {
            const half8_t w = BKN ? __builtin_shufflevector(f.wk[ni][0], f.wk[ni][1], 0, 1, 2, 3, 4, 5, 6, 7) : f.fw[ni];
#pragma unroll
            for (int mi = 0; mi < 2; mi++) acc[ni][mi] = Op::mul(w, f.fa[mi], acc[ni][mi]);
        }
    };

    Frag fr[2];
    lds_barrier(); // tile 0 is visible
    read_frags(0, 0, fr[0]);
    // At the top of a k-tile the reads of its first slice into fr[0] are in flight.  Every slice is requested one
    // step (four MFMAs) before it is multiplied; the barrier that publishes tile kt+1 (and hands the buffer of tile kt
    // back to the loaders, hence the wait for this wavefront's last reads of it) is passed with the MFMAs of the third
    // slice queued, and the first slice of tile kt+1 is fetched under the MFMAs of the fourth.
    // Full k-tiles with a successor first, in a loop of one basic block; then the last tile, full or partial (with the
    // partial tile as a second path inside the loop the accumulators end up in different registers on the two paths and
    // are copied, 64 registers each way, every iteration, with the matrix core drained in between).  The scheduling
    // fences keep the MFMAs of a step where they are written: between the reads of the next slice and the wait for it.
    const int last_steps = ((k_end - k_begin) - (n_ktiles - 1) * BK) / 16; // 16-wide steps of the last k-tile (1..4)
    auto first_three = [&](int kt) {
        read_frags(kt, 1, fr[1]);
        wait_older(fr[0]);
        multiply(fr[0]);
        __builtin_amdgcn_sched_barrier(0);
        read_frags(kt, 2, fr[0]);
        wait_older(fr[1]);
        multiply(fr[1]);
        __builtin_amdgcn_sched_barrier(0);
        read_frags(kt, 3, fr[1]);
        wait_older(fr[0]);
        multiply(fr[0]);
        __builtin_amdgcn_sched_barrier(0);
    };
    for (int kt = 0; kt + 1 < n_ktiles; kt++) {
        first_three(kt);
        wait_all(fr[1]);
        __builtin_amdgcn_s_barrier();
        read_frags(kt + 1, 0, fr[0]);
        multiply(fr[1]);
        __builtin_amdgcn_sched_barrier(0);
    }
    if (last_steps == BK / 16) {
        first_three(n_ktiles - 1);
        wait_all(fr[1]);
        multiply(fr[1]);
    } else { // fr[0] will hold its first slice
        wait_all(fr[0]);
        multiply(fr[0]);
        for (int s = 1; s < last_steps; s++) {
            read_frags(n_ktiles - 1, s, fr[0]);
            wait_all(fr[0]);
            multiply(fr[0]);
        }
    }
}

} // namespace
