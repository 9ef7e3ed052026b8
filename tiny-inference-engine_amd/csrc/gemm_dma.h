// One tile of a bfloat16 product whose operand slices go global memory -> LDS directly (buffer loads with the
// lds flag: no registers, no LDS write instructions), for K % 32 == 0.
//
// A workgroup of four waves (one per SIMD, 512 registers each) owns a 256 x BN tile, BN = 256 or 128; a wave owns
// 128 x BN/2 of it, so that every byte read from LDS feeds twice the flops it does with the 64-wide
// wave tiles above. k advances in slices of 32 through a ring of four LDS stages: while slice t is
// multiplied, slices t+1 and t+2 are landing or landed and the loads of t+2 (its w rows) and t+3 (its x rows) are
// issued, a few between the matrix instructions of each half slice so that neither the texture
// path nor the in-order instruction stream of the one wave backs up. One barrier a slice: it sits
// after the first half's matrix instructions, when the fragments of the second half are in
// registers already, so that the stage is free and the next slice's first fragments can be read
// while the second half multiplies.
//
// A staged row is 64 bytes, unpadded; 16-byte chunk c of row r sits at chunk c ^ ((r >> 1) & 3), which
// spreads the 32 rows a fragment read touches over the banks. Rows beyond M or N are clamped to the
// last row (their products land in output rows or columns that are never stored). With PW the weight
// comes in packed blocks of 16 rows x 32 k (1 KB in the matrix cores' operand order, as the decode
// product reads it): one load instruction stages one block, and the 16 lanes that LDS serves in a
// cycle read 256 consecutive bytes of it.
//
// The matrix instructions take w's fragment as their first operand: the tile comes out transposed,
// a lane holding 4 consecutive columns of one output row, which it stores as one 8- or 16-byte piece.
#pragma once
#include "common.h"
#include <type_traits>

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8_t;
typedef __attribute__((__vector_size__(16 * sizeof(float)))) float floatx16;
typedef __attribute__((ext_vector_type(4))) float floatx4_t;
typedef __attribute__((address_space(3))) void lds_void_t;

#define GD_BK 32
#define GD_STAGES 4
// Fourth word of a raw buffer descriptor on gfx9-family GPUs: 32-bit float data format, destination
// selects x, y, z, w; no swizzle, no stride (the compiler's own default for raw buffers on this target).
#define GD_RSRC_FLAGS 0x27000

#define GD_LDS_BYTES(BM, BN) (sizeof(bf16_t) * GD_STAGES * ((BM) + (BN)) * GD_BK)

#if defined(__HIP_DEVICE_COMPILE__)
__device__ __forceinline__ int gd_stage_row(int lane, int wave) { return wave * 16 + (lane >> 2); }
__device__ __forceinline__ int gd_stage_chunk(int lane, int row) { return (lane & 3) ^ ((row >> 1) & 3); }

// acc = x w^T over `k_tiles` slices of 32, for a workgroup of four waves (2 x 2; a wave BM / 2 rows and BN / 2 columns).
// BM: 256, 128 or 64 rows of x. x's rows: byte offsets `a_off` into a_rsrc of the 16-byte chunk that this lane stages
// in wave instruction p (row 64 p + gd_stage_row, chunk gd_stage_chunk of it); w's rows: `b_off` likewise or, with
// PW, lane * 16 with `b_tile_off` the byte offset of block row 4 p + wave. A lane ends with, in acc[i][j], row
// wm BM / 2 + 32 i + lane % 32 and in word 4 g + v column wn BN / 2 + 32 j + 8 g + 4 (lane / 32) + v, wm = wave / 2 and
// wn = wave % 2.
template <int BM, int BN, bool PW>
__device__ __forceinline__ void gemm_dma_tile(bf16_t* lds, const __amdgpu_buffer_rsrc_t a_rsrc,
                                              const unsigned (&a_off)[BM / 64], const __amdgpu_buffer_rsrc_t b_rsrc,
                                              const unsigned (&b_off)[BN / 64], const unsigned (&b_tile_off)[BN / 64],
                                              int k_tiles, floatx16 (&acc)[BM / 64][BN / 64]) {
  constexpr int BK = GD_BK;
  constexpr int TN = BN / 64;                   // 32-column MFMA tiles of a wave
  constexpr int TM = BM / 64;                   // 32-row MFMA tiles of a wave
  constexpr int PA = BM / 64;                   // wave instructions that stage x's rows (16 rows each, 4 waves)
  constexpr int PB = BN / 64;                   // wave instructions that stage w's rows likewise
  static_assert(BM == 256 || BM == 128 || BM == 64, "rows of a tile");
  constexpr int BUF = (BM + BN) * BK;           // elements of one stage
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int wm = wave >> 1, wn = wave & 1;
  const int fr = lane & 31;
  const int fk = lane >> 5;

  auto stage = [&](int kt) { return lds + (kt & (GD_STAGES - 1)) * BUF; };
  auto issue_x = [&](int kt) {
    bf16_t* buf = stage(kt);
#pragma unroll
    for (int p = 0; p < PA; ++p)
      __builtin_amdgcn_raw_ptr_buffer_load_lds(a_rsrc, (lds_void_t*)(buf + (p * 64 + wave * 16) * BK), 16, a_off[p],
                                               kt * BK * 2, 0, 0);
  };
  auto issue_w = [&](int kt) {
    bf16_t* buf = stage(kt);
#pragma unroll
    for (int p = 0; p < PB; ++p)
      __builtin_amdgcn_raw_ptr_buffer_load_lds(b_rsrc, (lds_void_t*)(buf + (BM + p * 64 + wave * 16) * BK), 16,
                                               b_off[p], PW ? b_tile_off[p] + kt * 1024 : kt * BK * 2, 0, 0);
  };

#pragma unroll
  for (int i = 0; i < TM; ++i)
#pragma unroll
    for (int j = 0; j < TN; ++j)
#pragma unroll
      for (int v = 0; v < 16; ++v) acc[i][j][v] = 0.f;

  // Fragment addresses. x's stage rows are swizzled (above); w's are too unless packed, where the
  // 16-byte piece of (row r of block t, k-chunk c) sits at t * 1 KB + (16 c + r) * 16 bytes: the 16 lanes
  // that one LDS cycle serves read 256 consecutive bytes.
  const int sw = (fr >> 1) & 3;
  const int koff0 = ((0 + fk) ^ sw) * 8, koff1 = ((2 + fk) ^ sw) * 8;
  const int a_row = (wm * (BM / 2) + fr) * BK;
  const int b_row = PW ? BM * BK + (wn * (BN / 32) + (fr >> 4)) * 512 + (fr & 15) * 8
                       : (BM + wn * (BN / 2) + fr) * BK;

  bf16x8_t fa[2][TM], fb[2][TN];
  auto load_frags = [&](const bf16_t* buf, int ks, int set) {
    const int koff = ks ? koff1 : koff0;
    const int koff_w = PW ? (ks * 2 + fk) * 128 : koff;
#pragma unroll
    for (int i = 0; i < TM; ++i) fa[set][i] = *reinterpret_cast<const bf16x8_t*>(buf + a_row + i * 32 * BK + koff);
#pragma unroll
    for (int j = 0; j < TN; ++j) fb[set][j] = *reinterpret_cast<const bf16x8_t*>(buf + b_row + j * 32 * BK + koff_w);
  };
  auto mfma_step = [&](int set) {
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
      for (int j = 0; j < TN; ++j)
        acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fb[set][j], fa[set][i], acc[i][j], 0, 0, 0);
  };

  // A stage is free once every wave has passed the barrier of the slice that read it, which stands in the
  // middle of that slice (its last fragments are in registers by then). Slice j's x rows are asked for right
  // after the barrier of slice j - 4, into the stage that slice has just left, and its w rows before the barrier
  // of slice j - 3: the loads of two to three slices are in flight at any time (64 to 96 KB a workgroup of 256 x 256), which is what
  // the latency of L2 asks for at a slice every 0.4 us. (One slice less ahead - 32 to 64 KB - the matrix cores
  // waited a third of the time.) The first slices here; the host gives every range of K at least three.
  issue_x(0);
  issue_w(0);
  issue_x(1);
  issue_w(1);
  issue_x(2);
  issue_w(2);
  // s_waitcnt vmcnt(n) [lgkmcnt(0)], then the barrier (gfx9 encoding: vmcnt in bits 3:0 and 15:14, expcnt 6:4,
  // lgkmcnt 11:8; a counter at its maximum is not waited for).
  auto wait_barrier = [&](auto loads, auto lds_too) {
    constexpr int n = decltype(loads)::value;
    static_assert(n >= 0 && n < 64, "vmcnt has six bits");
    __builtin_amdgcn_sched_barrier(0);
    __builtin_amdgcn_s_waitcnt((n & 15) | ((n >> 4) << 14) | (7 << 4) | ((decltype(lds_too)::value ? 0 : 15) << 8));
    asm volatile("s_barrier" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
  };
  using One = std::integral_constant<int, PA + PB>;
  using Two = std::integral_constant<int, 2 * (PA + PB)>;
  using None = std::integral_constant<int, 0>;
  // Slice 0 has landed when at most the loads of slices 1 and 2 are outstanding.
  wait_barrier(Two{}, std::false_type{});
  load_frags(stage(0), 0, 0);
  if (3 < k_tiles) issue_x(3);

  // One slice; its first fragments are in set 0 already. STEADY: slices up to kt + 4 exist, so the loads
  // sit in straight-line code and exactly those of slices kt + 2 and kt + 3 may still be in flight at the barrier.
  auto slice = [&](int kt, auto steady_tag) {
    constexpr bool STEADY = decltype(steady_tag)::value;
    load_frags(stage(kt), 1, 1);
    if (STEADY || kt + 3 < k_tiles) issue_w(kt + 3);
    mfma_step(0);
    if (STEADY && BM == 256) {
#pragma unroll
      for (int q = 0; q < (4 + TN) / 2; ++q) {
        __builtin_amdgcn_sched_group_barrier(0x008, TN / 2, 0);
        __builtin_amdgcn_sched_group_barrier(0x100, 2, 0);
      }
#pragma unroll
      for (int q = 0; q < PB; ++q) {
        __builtin_amdgcn_sched_group_barrier(0x008, 2, 0);
        __builtin_amdgcn_sched_group_barrier(0x020, 1, 0);
      }
    }
    // My share of slice kt + 1 has landed and my reads of this stage are in registers; after the
    // barrier that holds for every wave.
    if (STEADY || kt + 3 < k_tiles) wait_barrier(Two{}, std::true_type{});
    else if (kt + 2 < k_tiles) wait_barrier(One{}, std::true_type{});
    else wait_barrier(None{}, std::true_type{});
    if (STEADY || kt + 1 < k_tiles) load_frags(stage(kt + 1), 0, 0);
    if (STEADY || kt + 4 < k_tiles) issue_x(kt + 4);
    mfma_step(1);
    if (STEADY && BM == 256) {
#pragma unroll
      for (int q = 0; q < (4 + TN) / 2; ++q) {
        __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
        __builtin_amdgcn_sched_group_barrier(0x100, 2, 0);
      }
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        __builtin_amdgcn_sched_group_barrier(0x008, TN / 2, 0);
        __builtin_amdgcn_sched_group_barrier(0x020, 1, 0);
      }
    }
    __builtin_amdgcn_sched_barrier(0);
  };

  int kt = 0;
  for (; kt + 7 < k_tiles; kt += 4) {
    slice(kt, std::true_type{});
    slice(kt + 1, std::true_type{});
    slice(kt + 2, std::true_type{});
    slice(kt + 3, std::true_type{});
  }
  for (; kt < k_tiles; ++kt) slice(kt, std::false_type{});
}
#endif
