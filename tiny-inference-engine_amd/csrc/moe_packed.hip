// The experts' products (see moe.hip) over weights in packed blocks, bfloat16 on the matrix cores.
//
// All experts' matrices stand one behind the other as one [real * N][K] matrix in blocks of 16 rows x 32 k, 1 KB each, in
// the matrix cores' operand order (block (tile, k-block) at (tile * K / 32 + k-block) * 1 KB; inside it chunk c of 8 k of
// row r at (16 c + r) * 16 bytes). A gated expert's gate and up rows are interleaved in blocks of 8, so that one block
// row holds the gates and the ups of the same 8 outputs. N % 16 == 0, K % 32 == 0 and K >= 96.
//
// Row tiles of 16 (few rows an expert: decode steps): a workgroup takes one row tile and NT block rows; its four waves
// take every fourth k-block each and add their sums through LDS in wave order. A weight load of a wave is one block, 1 KB
// of consecutive memory, and DEPTH k-blocks are asked for before the first is used.
// Row tiles of 64, 128 or 256 (many rows an expert): the dense product's tile (gemm_dma.h), x's rows gathered by slot on
// their way into LDS. Which tiles exist is known on the device only; the grid covers the most there can be, and the
// workgroups that have one are numbered so that each of the 8 XCDs works on a contiguous run of tiles (an expert's row
// tiles and columns), whose weights and rows its L2 then holds once.
#include "expert_activation.h"
#include "gemm_dma.h"

struct MoeRows {
  const int* offsets;      // [real + 1]: places of each expert's slots
  const int* slot_at;      // [slots]
  const int* tiles;        // [max_tiles][2]: expert, first place
  const int* num_tiles;
  int top;
};

// MODE as in moe.hip; MODE 0 reads rows by place and writes float32, the others gather rows by slot and write bfloat16.
template <int MODE, int NT>
__global__ __launch_bounds__(256) void moe_packed_few_rows_kernel(const bf16_t* __restrict__ x,
                                                                  const bf16_t* __restrict__ w, void* __restrict__ out,
                                                                  MoeRows rw, int N, int K, GateParams gp) {
  constexpr bool GATED = MODE == 1 || MODE == 3 || MODE == 4;
  constexpr bool GATHER = MODE != 0;
  const int tile = blockIdx.x;
  if (tile >= *rw.num_tiles) return;                         // the whole workgroup leaves
  __shared__ floatx4_t sums[NT][4][TIE_WAVE];
  const int lane = threadIdx.x & (TIE_WAVE - 1);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / TIE_WAVE);
  const int r16 = lane & 15, quad = lane >> 4;
  const int e = rw.tiles[2 * tile], place0 = rw.tiles[2 * tile + 1];
  const int rows = min(16, rw.offsets[e + 1] - place0);
  const int place = place0 + (r16 < rows ? r16 : 0);         // rows beyond the tile's end: computed, never stored
  const size_t src = GATHER ? static_cast<size_t>(rw.slot_at[place] / rw.top) : static_cast<size_t>(place);
  const bf16_t* xr = x + src * K + quad * 8;
  const int kblocks = K / 32, block_rows = N / 16;
  const int b0 = blockIdx.y * NT;
  const bf16_t* wr[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
    wr[nt] = w + (static_cast<size_t>(e) * block_rows + min(b0 + nt, block_rows - 1)) * kblocks * 512 + lane * 8;
  floatx4_t acc[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) acc[nt] = floatx4_t{0.f, 0.f, 0.f, 0.f};
  int kb = wave;
  auto blocks = [&](auto depth) {                            // DEPTH of this wave's k-blocks, every load before the first use
    constexpr int DEPTH = decltype(depth)::value;
    uint4 xf[DEPTH], wf[NT][DEPTH];
#pragma unroll
    for (int i = 0; i < DEPTH; ++i) {
      xf[i] = *reinterpret_cast<const uint4*>(xr + (kb + 4 * i) * 32);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) wf[nt][i] = *reinterpret_cast<const uint4*>(wr[nt] + static_cast<size_t>(kb + 4 * i) * 512);
    }
#pragma unroll
    for (int i = 0; i < DEPTH; ++i)
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
        acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(&wf[nt][i]),
                                                          *reinterpret_cast<const bf16x8_t*>(&xf[i]), acc[nt], 0, 0, 0);
    kb += 4 * DEPTH;
  };
  while (kb + 28 < kblocks) blocks(std::integral_constant<int, 8>{});
  if (kb + 12 < kblocks) blocks(std::integral_constant<int, 4>{});
  if (kb + 4 < kblocks) blocks(std::integral_constant<int, 2>{});
  if (kb < kblocks) blocks(std::integral_constant<int, 1>{});
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) sums[nt][wave][lane] = acc[nt];
  __syncthreads();
  // wave nt finishes block row nt: lane: x row r16, rows 4 quad .. 4 quad + 3 of the block
  for (int nt = wave; nt < NT; nt += 4) {
    if (b0 + nt >= block_rows) continue;
    floatx4_t v = sums[nt][0][lane];
#pragma unroll
    for (int p = 1; p < 4; ++p) v += sums[nt][p][lane];
    if constexpr (MODE == 4) v *= gp.slot_weights[rw.slot_at[place]];
    if constexpr (GATED) {
      float u[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) u[i] = __shfl_xor(v[i], 32, TIE_WAVE);     // quads 2 and 3 hold the ups
      if (quad < 2 && r16 < rows) {
        uint2 packed;
        packed.x = pack_bf16x2(gated_fast<MODE>(v[0], u[0], gp), gated_fast<MODE>(v[1], u[1], gp));
        packed.y = pack_bf16x2(gated_fast<MODE>(v[2], u[2], gp), gated_fast<MODE>(v[3], u[3], gp));
        *reinterpret_cast<uint2*>(static_cast<bf16_t*>(out) + static_cast<size_t>(place0 + r16) * (N / 2) + (b0 + nt) * 8 +
                                  quad * 4) = packed;
      }
    } else if (r16 < rows) {
      const size_t at = static_cast<size_t>(place0 + r16) * N + (b0 + nt) * 16 + quad * 4;
      if constexpr (MODE == 2) {
        uint2 packed;
        packed.x = pack_bf16x2(relu_squared_f(v[0]), relu_squared_f(v[1]));
        packed.y = pack_bf16x2(relu_squared_f(v[2]), relu_squared_f(v[3]));
        *reinterpret_cast<uint2*>(static_cast<bf16_t*>(out) + at) = packed;
      } else {
        *reinterpret_cast<floatx4_t*>(static_cast<float*>(out) + at) = v;
      }
    }
  }
}

template <int BM, int BN, int MODE>
__global__ __launch_bounds__(256) void moe_packed_many_rows_kernel(const bf16_t* __restrict__ x,
                                                                   const bf16_t* __restrict__ w, void* __restrict__ out,
                                                                   MoeRows rw, int x_rows, int N, int K, int tiles_n,
                                                                   GateParams gp) {
#if defined(__HIP_DEVICE_COMPILE__)
  constexpr bool GATED = MODE == 1 || MODE == 3 || MODE == 4;
  constexpr bool GATHER = MODE != 0;
  constexpr int TN = BN / 64, TM = BM / 64;
  extern __shared__ bf16_t lds[];
  const int total = *rw.num_tiles * tiles_n;
  const int per_xcd = (total + 7) / 8;
  const int id = (blockIdx.x % 8) * per_xcd + blockIdx.x / 8;
  if (static_cast<int>(blockIdx.x / 8) >= per_xcd || id >= total) return;      // the whole workgroup leaves
  const int tile = id / tiles_n, col0 = (id % tiles_n) * BN;
  const int e = rw.tiles[2 * tile], place0 = rw.tiles[2 * tile + 1];
  const int rows = min(BM, rw.offsets[e + 1] - place0);
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int wm = wave >> 1, wn = wave & 1;
  const int fr = lane & 31, fk = lane >> 5;
  const int lr = gd_stage_row(lane, wave), lchunk = gd_stage_chunk(lane, lr);
  const unsigned row_bytes = static_cast<unsigned>(K) * 2;
  const int kblocks = K / 32;
  const __amdgpu_buffer_rsrc_t a_rsrc = __builtin_amdgcn_make_buffer_rsrc(
      const_cast<bf16_t*>(x), 0, static_cast<int>(x_rows * row_bytes), GD_RSRC_FLAGS);
  unsigned a_off[BM / 64], b_off[BN / 64], b_tile_off[BN / 64];
#pragma unroll
  for (int p = 0; p < BM / 64; ++p) {
    const int place = place0 + min(lr + p * 64, rows - 1);     // rows beyond the tile's end: computed, never stored
    const int src = GATHER ? rw.slot_at[place] / rw.top : place;
    a_off[p] = static_cast<unsigned>(src) * row_bytes + lchunk * 16;
  }
  const int tile0 = col0 / 16, last_tile = N / 16 - 1;
  const __amdgpu_buffer_rsrc_t b_rsrc = __builtin_amdgcn_make_buffer_rsrc(
      const_cast<bf16_t*>(w + (static_cast<size_t>(e) * (N / 16) + tile0) * kblocks * 512), 0,
      static_cast<int>(static_cast<unsigned>(min(BN / 16, last_tile + 1 - tile0)) * kblocks * 1024), GD_RSRC_FLAGS);
#pragma unroll
  for (int p = 0; p < BN / 64; ++p) {
    b_off[p] = lane * 16;
    b_tile_off[p] = static_cast<unsigned>(min(p * 4 + wave, last_tile - tile0)) * kblocks * 1024;
  }
  floatx16 acc[TM][TN];
  gemm_dma_tile<BM, BN, true>(lds, a_rsrc, a_off, b_rsrc, b_off, b_tile_off, kblocks, acc);
#pragma unroll
  for (int i = 0; i < TM; ++i) {
    const int m = wm * (BM / 2) + i * 32 + fr;
    if (m >= rows) continue;
    const float sw = MODE == 4 ? gp.slot_weights[rw.slot_at[place0 + m]] : 1.f;
#pragma unroll
    for (int j = 0; j < TN; ++j) {
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int n = col0 + wn * (BN / 2) + j * 32 + 8 * g + 4 * fk;
        if (n >= N) continue;
        float v0 = acc[i][j][4 * g], v1 = acc[i][j][4 * g + 1], v2 = acc[i][j][4 * g + 2], v3 = acc[i][j][4 * g + 3];
        if constexpr (GATED) {
          if (g & 1) continue;                 // the ups of group g are register group g + 1
          float u0 = acc[i][j][4 * g + 4], u1 = acc[i][j][4 * g + 5], u2 = acc[i][j][4 * g + 6], u3 = acc[i][j][4 * g + 7];
          if constexpr (MODE == 4) v0 *= sw, v1 *= sw, v2 *= sw, v3 *= sw, u0 *= sw, u1 *= sw, u2 *= sw, u3 *= sw;
          uint2 packed;
          packed.x = pack_bf16x2(gated_fast<MODE>(v0, u0, gp), gated_fast<MODE>(v1, u1, gp));
          packed.y = pack_bf16x2(gated_fast<MODE>(v2, u2, gp), gated_fast<MODE>(v3, u3, gp));
          *reinterpret_cast<uint2*>(static_cast<bf16_t*>(out) + static_cast<size_t>(place0 + m) * (N / 2) + (n >> 4) * 8 +
                                    4 * fk) = packed;
        } else {
          const size_t at = static_cast<size_t>(place0 + m) * N + n;
          if constexpr (MODE == 2) {
            uint2 packed;
            packed.x = pack_bf16x2(relu_squared_f(v0), relu_squared_f(v1));
            packed.y = pack_bf16x2(relu_squared_f(v2), relu_squared_f(v3));
            *reinterpret_cast<uint2*>(static_cast<bf16_t*>(out) + at) = packed;
          } else {
            *reinterpret_cast<floatx4_t*>(static_cast<float*>(out) + at) = floatx4_t{v0, v1, v2, v3};
          }
        }
      }
    }
  }
#endif
}

// Rows of a row tile by the average number of rows an expert gets (sweeps over 32 experts of 768 x 2048 and 64 of
// 1536 x 4096, 1 to 2048 tokens, four experts each): 256 only where the wider tile still leaves more than one round of
// workgroups for the compute units. inner: an expert's inner size.
extern "C" int tie_moe_packed_tile_rows(int slots, int real, int inner) {
  if (slots < 12L * real) return 16;
  if (slots < 48L * real) return 64;
  return slots >= 96L * real && static_cast<long>(real) * inner >= 128L * 384 ? 256 : 128;
}

template <int BM, int BN, int MODE>
static int launch_many_rows(const void* x, const void* w, void* out, const MoeRows& rw, int max_tiles, int x_rows, int N,
                            int K, GateParams gp, hipStream_t stream) {
  const int tiles_n = (N + BN - 1) / BN;
  const size_t shared = GD_LDS_BYTES(BM, BN);
  static bool raised = false;
  if (!raised) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_packed_many_rows_kernel<BM, BN, MODE>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(shared));
    if (e != hipSuccess) return static_cast<int>(e);
    raised = true;
  }
  const long grid = (static_cast<long>(max_tiles) * tiles_n + 7) / 8 * 8;
  if (grid > 0x7fffffffL) return TIE_BAD_ARGUMENT;
  moe_packed_many_rows_kernel<BM, BN, MODE><<<static_cast<unsigned>(grid), 256, shared, stream>>>(
      static_cast<const bf16_t*>(x), static_cast<const bf16_t*>(w), out, rw, x_rows, N, K, tiles_n, gp);
  return tie_launch_status();
}

// x bfloat16 [x_rows][K]; w packed, [real * N][K] (N counts gate and up rows where gated); mode 1, 3 or 4: out bfloat16
// [slots][N / 2]; mode 2: out bfloat16 [slots][N]; mode 0: x_rows = slots, out float32 [slots][N]. tile_rows (16, 64,
// 128 or 256) as given to tie_moe_align; columns: the columns a workgroup takes (128 or 256; tiles of 64 rows on), or 0
// to choose.
extern "C" int tie_moe_gemm_packed(const void* x, int x_rows, const void* w, void* out, int mode, const int* offsets,
                                   const int* slot_at, const int* tiles, const int* num_tiles, int max_tiles,
                                   int tile_rows, int columns, int top, int N, int K, float limit, float slope,
                                   float shift, const float* slot_weights, hipStream_t stream) {
  if ((mode == 4 && slot_weights == nullptr) || x_rows <= 0 || max_tiles <= 0 || top <= 0 || N <= 0 || N % 16 || K < 96 || K % 32 || mode < 0 || mode > 4 ||
      (columns != 0 && columns != 128 && columns != 256) || static_cast<size_t>(x_rows) * K * 2 > 0x7fffffffu ||
      static_cast<size_t>(K) * 512 > 0x7fffffffu || reinterpret_cast<uintptr_t>(x) % 16 ||
      reinterpret_cast<uintptr_t>(w) % 16 || reinterpret_cast<uintptr_t>(out) % 16)
    return TIE_BAD_ARGUMENT;
  const MoeRows rw{offsets, slot_at, tiles, num_tiles, top};
  const GateParams gp{limit, slope, shift, slot_weights};
  if (tile_rows == 16) {
    const dim3 grid(max_tiles, (N / 16 + 1) / 2);
    if (grid.y > 65535) return TIE_BAD_ARGUMENT;
#define FEW(MODE)                                                                                          \
  moe_packed_few_rows_kernel<MODE, 2><<<grid, 256, 0, stream>>>(static_cast<const bf16_t*>(x),             \
                                                                static_cast<const bf16_t*>(w), out, rw, N, K, gp)
    if (mode == 0) FEW(0);
    else if (mode == 1) FEW(1);
    else if (mode == 2) FEW(2);
    else if (mode == 4) FEW(4);
    else FEW(3);
#undef FEW
    return tie_launch_status();
  }
#define MANY(BM, BN)                                                                                     \
  (mode == 0   ? launch_many_rows<BM, BN, 0>(x, w, out, rw, max_tiles, x_rows, N, K, gp, stream)         \
   : mode == 1 ? launch_many_rows<BM, BN, 1>(x, w, out, rw, max_tiles, x_rows, N, K, gp, stream)         \
   : mode == 2 ? launch_many_rows<BM, BN, 2>(x, w, out, rw, max_tiles, x_rows, N, K, gp, stream)         \
   : mode == 4 ? launch_many_rows<BM, BN, 4>(x, w, out, rw, max_tiles, x_rows, N, K, gp, stream)         \
               : launch_many_rows<BM, BN, 3>(x, w, out, rw, max_tiles, x_rows, N, K, gp, stream))
  if (columns == 0) columns = tile_rows == 64 ? 128 : 256;
  if (tile_rows == 64) return columns == 128 ? MANY(64, 128) : MANY(64, 256);
  if (tile_rows == 128) return columns == 128 ? MANY(128, 128) : MANY(128, 256);
  if (tile_rows == 256) return columns == 128 ? MANY(256, 128) : MANY(256, 256);
#undef MANY
  return TIE_BAD_ARGUMENT;
}
