// The gated delta rule with one decay a head, over long portions: chunks of up to 64 tokens as float32 matrix products.
//
// A token's step is S_i = g_i S_(i-1) + k_i u_i^T with u_i = beta_i (v_i - g_i S_(i-1)^T k_i). Inside a chunk that starts
// from S_0, with b_i the sum of log g over its tokens up to and with i,
//
//   S_i = e^(b_i) S_0 + sum_(j <= i) e^(b_i - b_j) k_j u_j^T
//   (I + A) U = diag(beta) V - diag(beta e^b) K S_0 ,     A_ij = beta_i e^(b_i - b_j) k_i . k_j  for j < i
//   o_i = e^(b_i) S_0^T q_i + sum_(j <= i) P_ij u_j ,      P_ij = e^(b_i - b_j) q_i . k_j        for j <= i
//
// so with U0 = (I + A)^-1 diag(beta) V and W = (I + A)^-1 diag(beta e^b) K, which need no state, U = U0 - W S_0. All
// exponents are differences of a running sum that only falls: no factor exceeds 1. The sums b are kept in double, so
// that the decay between two late tokens of a chunk does not lose the digits an early strong decay takes. Three
// launches:
//   prepare  a workgroup a (chunk, head): K K^T and Q K^T, A, P; forward substitution for U0 and W in blocks of 16 rows
//            (the four diagonal blocks of I + A are inverted by substitution, everything else is matrix products);
//            K scaled by e^(b_end - b_j) and transposed
//   states   a workgroup a (sequence, head, 16 value columns) walks the chunks in order: U = U0 - W S, then
//            S <- e^(b_end) S + K~^T U; leaves every chunk its starting state and the slot the final one
//   outputs  a workgroup a (chunk, head, 64 value columns): O = e^b (Q S_0) + P U
// Every value is float32 and every product v_mfma_f32_16x16x4_f32: a lane gives A[m = lane % 16][slot = lane / 16] and
// B[slot][n = lane % 16] and receives C[4 (lane / 16) + r][lane % 16]. The four slots of instruction i of a block of 16
// along K stand for its elements 4 slot + i: so four consecutive floats of a row feed four instructions, and an
// accumulator block is the next product's B operand as it stands.
//
// What one launch leaves for the next lies in memory in blocks of 16 x 16 elements, 1 KB, in the order in which the reader's
// lanes take them (four consecutive words a lane): a load or a store of a wave is then 1 KB of consecutive memory. A block
// read as an A operand holds element (m, k) at word 4 (16 (k / 4) + m) + k % 4, a block in accumulator layout (read as a B
// operand) element (k, n) at word 4 (16 (k / 4) + n) + k % 4. (Row-major, with 64 bytes of 16 rows a load, the states
// kernel took 101 us of a 2048-token prompt of 16 heads.)
#include "common.h"

#define DC_ROWS 64                 // tokens of a chunk at most
#define DC_THREADS 256
#define DC_AR (DC_ROWS + 4)        // words from one row of A in LDS to the next
#define DC_TR 20                   // ... of an inverted diagonal block

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float dc_floatx4;

__device__ __forceinline__ dc_floatx4 dc_mfma(float a, float b, dc_floatx4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// Four consecutive elements from place i of a vector of n (zeros behind); WIDE: n is a multiple of 4 and the vector lies
// on a 16-byte address, so the four count together and are one load (from an address that exists, whatever i is).
template <bool WIDE>
__device__ __forceinline__ float4 dc_load4(const float* __restrict__ p, int i, int n) {
  if constexpr (WIDE) {
    const float4 v = *reinterpret_cast<const float4*>(p + min(i, n - 4));
    const bool in = i < n;
    return make_float4(in ? v.x : 0.f, in ? v.y : 0.f, in ? v.z : 0.f, in ? v.w : 0.f);
  }
  const float x = p[min(i, n - 1)], y = p[min(i + 1, n - 1)], z = p[min(i + 2, n - 1)], w = p[min(i + 3, n - 1)];
  return make_float4(i < n ? x : 0.f, i + 1 < n ? y : 0.f, i + 2 < n ? z : 0.f, i + 3 < n ? w : 0.f);
}

__device__ __forceinline__ dc_floatx4 dc_mfma4(float4 a, dc_floatx4 b, dc_floatx4 c) {
  c = dc_mfma(a.x, b[0], c);
  c = dc_mfma(a.y, b[1], c);
  c = dc_mfma(a.z, b[2], c);
  return dc_mfma(a.w, b[3], c);
}

// A launch's geometry and the chunks' memory; entry (chunk * heads + head - head0) of each array.
struct DeltaChunks {
  const float* tok;        // rows of delta_prepare: [q (G d) | k (G d) | v (H e) | g (H) | beta (H) | log g (H)]
  int row;
  const int* items;        // [count][3]: sequence, first row, end row
  int G, H, d, e;
  int head0, heads;        // the heads of this launch
  int ep;                  // e rounded up to 16
  int D;                   // d rounded up as the chunks' memory is
  float* u;                // [ep / 16][4] blocks: U0, then U
  float* w;                // [4][D / 16] blocks (A)
  float* kt;               // [D / 16][4] blocks (A): K~ transposed
  float* q;                // [4][D / 16] blocks (A): e^(b_i) q_i
  float* p;                // [4][4] blocks (A), those above the diagonal unused
  float* s0;               // [ep / 16][D / 16] blocks: the state before the chunk
  float* decay;            // [1]: e^(b_end)
};

// WIDE: q and k of every head start on 16-byte addresses and d is a multiple of 4.
template <bool WIDE>
__global__ __launch_bounds__(DC_THREADS) void delta_chunk_prepare_kernel(DeltaChunks g) {
  extern __shared__ __attribute__((aligned(16))) float keys[];             // [64][D + 4]: the chunk's keys
  __shared__ __attribute__((aligned(16))) float A[DC_ROWS * DC_AR];
  __shared__ __attribute__((aligned(16))) float inv[4][16 * DC_TR];        // (I + A_rr)^-1 of the diagonal blocks
  __shared__ double b[DC_ROWS];
  __shared__ __attribute__((aligned(16))) float beta[DC_ROWS];             // all three are 0 behind the chunk's end:
  __shared__ __attribute__((aligned(16))) float beta_eb[DC_ROWS];          // beta_i e^(b_i)
  __shared__ __attribute__((aligned(16))) float to_end[DC_ROWS];           // e^(b_end - b_i)
  __shared__ float eb[DC_ROWS];                                            // e^(b_i)
  const int item = blockIdx.x / g.heads, head = g.head0 + blockIdx.x % g.heads;
  const int kv = head / (g.H / g.G);
  const int t0 = g.items[3 * item + 1], n = g.items[3 * item + 2] - t0;
  const size_t entry = blockIdx.x;
  const float* rows = g.tok + static_cast<size_t>(t0) * g.row;
  const int q_at = kv * g.d, k_at = (g.G + kv) * g.d, v_at = 2 * g.G * g.d + head * g.e;
  const int beta_at = 2 * g.G * g.d + g.H * g.e + g.H + head, log_at = beta_at + g.H;
  const int lane = threadIdx.x % TIE_WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / TIE_WAVE);
  const int r16 = lane & 15, quad = lane >> 4;
  if (wave == 0) {                       // a lane a token: the running sum of log g
    const float* r = rows + static_cast<size_t>(min(lane, n - 1)) * g.row;
    double sum = lane < n ? static_cast<double>(r[log_at]) : 0.0;
    const float bt = lane < n ? r[beta_at] : 0.f;
#pragma unroll
    for (int off = 1; off < TIE_WAVE; off *= 2) {
      const double before = __shfl_up(sum, off, TIE_WAVE);
      if (lane >= off) sum += before;
    }
    const float e_b = expf(static_cast<float>(sum));
    const double end = __shfl(sum, TIE_WAVE - 1, TIE_WAVE);
    b[lane] = sum;
    beta[lane] = bt;
    beta_eb[lane] = bt * e_b;
    eb[lane] = e_b;
    to_end[lane] = lane < n ? expf(static_cast<float>(end - sum)) : 0.f;
    if (lane == TIE_WAVE - 1) g.decay[entry] = e_b;
  }
  const int kr = g.D + 4, quads = g.D / 4, blocks = g.D / 16;
  for (int i = threadIdx.x; i < DC_ROWS * quads; i += DC_THREADS) {      // rows behind the chunk's end: the last one's
    const int t = i / quads, c = (i % quads) * 4;
    *reinterpret_cast<float4*>(keys + t * kr + c) =
        dc_load4<WIDE>(rows + static_cast<size_t>(min(t, n - 1)) * g.row + k_at, c, g.d);
  }
  __syncthreads();
  // rows 16 tile .. of K K^T and Q K^T; which wave has the longest rows turns with the workgroup
  const int tile = (wave + blockIdx.x) & 3;
  dc_floatx4 kk[4], qk[4];
#pragma unroll
  for (int nt = 0; nt < 4; ++nt) kk[nt] = qk[nt] = dc_floatx4{0.f, 0.f, 0.f, 0.f};
  const float* own = rows + static_cast<size_t>(min(tile * 16 + r16, n - 1)) * g.row + q_at;
  const float own_eb = eb[tile * 16 + r16];
  float* qe = g.q + (entry * 4 + tile) * blocks * 256 + lane * 4;
#pragma unroll 2
  for (int kb = 0; kb < blocks; ++kb) {
    const int i0 = kb * 16 + quad * 4;
    const float4 qa = dc_load4<WIDE>(own, i0, g.d);
    const float4 ka = *reinterpret_cast<const float4*>(keys + (tile * 16 + r16) * kr + i0);
    *reinterpret_cast<float4*>(qe + kb * 256) = make_float4(qa.x * own_eb, qa.y * own_eb, qa.z * own_eb, qa.w * own_eb);
#pragma unroll
    for (int nt = 0; nt < 4; ++nt) {
      if (nt > tile) continue;
      const float4 v = *reinterpret_cast<const float4*>(keys + (nt * 16 + r16) * kr + i0);
      const dc_floatx4 kv4 = {v.x, v.y, v.z, v.w};
      kk[nt] = dc_mfma4(ka, kv4, kk[nt]);
      qk[nt] = dc_mfma4(qa, kv4, qk[nt]);
    }
  }
  float* pe = g.p + entry * DC_ROWS * DC_ROWS;
#pragma unroll
  for (int nt = 0; nt < 4; ++nt) {
    const int j = nt * 16 + r16;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = tile * 16 + quad * 4 + r;
      const bool in = i < n && j <= i;
      const float f = in ? expf(static_cast<float>(b[i] - b[j])) : 0.f;
      A[i * DC_AR + j] = in && j < i ? beta[i] * f * kk[nt][r] : 0.f;
      pe[(tile * 4 + nt) * 256 + (r16 / 4) * 64 + (quad * 4 + r) * 4 + r16 % 4] = in ? f * qk[nt][r] : 0.f;
    }
  }
  __syncthreads();
  {     // wave r inverts diagonal block r, a lane a column (the four quads the same ones)
    const float* Ar = A + wave * 16 * DC_AR + wave * 16;
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == r16 ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; j += 4) {
        const float4 a = *reinterpret_cast<const float4*>(Ar + i * DC_AR + j);
        v = fmaf(-a.x, x[j], v);
        if (j + 1 < i) v = fmaf(-a.y, x[j + 1], v);
        if (j + 2 < i) v = fmaf(-a.z, x[j + 2], v);
        if (j + 3 < i) v = fmaf(-a.w, x[j + 3], v);
      }
      x[i] = v;
    }
    if (quad == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) inv[wave][i * DC_TR + r16] = x[i];
    }
  }
  __syncthreads();
  float4 off[4][3], diag[4];             // the blocks of -A below the diagonal and the inverted ones, as A operands
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    diag[r] = *reinterpret_cast<const float4*>(&inv[r][r16 * DC_TR + quad * 4]);
#pragma unroll
    for (int c = 0; c < r; ++c) {
      const float4 a = *reinterpret_cast<const float4*>(A + (r * 16 + r16) * DC_AR + c * 16 + quad * 4);
      off[r][c] = make_float4(-a.x, -a.y, -a.z, -a.w);
    }
  }
  // 16 columns of [diag(beta) V | diag(beta e^b) K] a wave at a time
  for (int nt = wave; nt * 16 < g.ep + g.D; nt += 4) {
    const bool is_k = nt * 16 >= g.ep;
    const int c = nt * 16 - (is_k ? g.ep : 0) + r16;
    const bool live = c < (is_k ? g.d : g.e);
    const float* src = rows + v_at + (live ? c : 0);
    const float* factor = is_k ? beta_eb : beta;
    dc_floatx4 x[4];
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = r * 16 + quad * 4 + i;
        x[r][i] = is_k ? keys[t * kr + c] : src[static_cast<size_t>(min(t, n - 1)) * g.row];
      }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (!live) x[r] = dc_floatx4{0.f, 0.f, 0.f, 0.f};
      if (is_k) {
        const float4 f = *reinterpret_cast<const float4*>(to_end + r * 16 + quad * 4);
        *reinterpret_cast<float4*>(g.kt + ((entry * blocks + c / 16) * 4 + r) * 256 + lane * 4) =
            make_float4(x[r][0] * f.x, x[r][1] * f.y, x[r][2] * f.z, x[r][3] * f.w);
      }
      const float4 f = *reinterpret_cast<const float4*>(factor + r * 16 + quad * 4);
      x[r] = dc_floatx4{x[r][0] * f.x, x[r][1] * f.y, x[r][2] * f.z, x[r][3] * f.w};
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
#pragma unroll
      for (int s = 0; s < r; ++s) x[r] = dc_mfma4(off[r][s], x[s], x[r]);
      x[r] = dc_mfma4(diag[r], x[r], dc_floatx4{0.f, 0.f, 0.f, 0.f});
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (is_k) {
        float* dst = g.w + ((entry * 4 + r) * blocks + c / 16) * 256 + (r16 / 4) * 64 + r16 % 4;
#pragma unroll
        for (int i = 0; i < 4; ++i) dst[(quad * 4 + i) * 4] = x[r][i];
      } else {
        *reinterpret_cast<float4*>(g.u + ((entry * (g.ep / 16) + nt) * 4 + r) * 256 + lane * 4) =
            make_float4(x[r][0], x[r][1], x[r][2], x[r][3]);
      }
    }
  }
}

// What the walk takes of one chunk: a wave's part of W and K~^T and its rows of U0.
template <int TD>
struct DeltaChunkOperands {
  float4 w[4][TD];         // [row block of the chunk][block of the wave's key rows]
  float4 k[TD][4];         // [block of the wave's key rows][row block of the chunk]
  float4 u0;
  float decay;
};

template <int D, int TD>
__device__ __forceinline__ void delta_chunk_fetch(const DeltaChunks& g, size_t entry, int wave, int lane, int slab,
                                                  DeltaChunkOperands<TD>& o) {
  const float* w = g.w + (entry * 4 * (D / 16) + wave * TD) * 256 + lane * 4;
  const float* kt = g.kt + (entry * (D / 16) + wave * TD) * 4 * 256 + lane * 4;
#pragma unroll
  for (int m = 0; m < 4; ++m)
#pragma unroll
    for (int t = 0; t < TD; ++t) {
      o.w[m][t] = *reinterpret_cast<const float4*>(w + (m * (D / 16) + t) * 256);
      o.k[t][m] = *reinterpret_cast<const float4*>(kt + (t * 4 + m) * 256);
    }
  o.u0 = *reinterpret_cast<const float4*>(g.u + ((entry * (g.ep / 16) + slab) * 4 + wave) * 256 + lane * 4);
  o.decay = g.decay[entry];
}

// The four waves share the key rows: wave w holds rows [w D / 4, (w + 1) D / 4) of the 16 columns of S in accumulator
// layout, forms its part of W S for all rows of the chunk and passes it round through LDS (two buffers taking turns,
// one barrier a chunk); every wave then has all of U and updates its own rows of S. The next chunk's operands are on
// their way meanwhile, in the other of two sets of registers.
template <int D>
__global__ __launch_bounds__(DC_THREADS, 1) void delta_chunk_states_kernel(DeltaChunks g, float* __restrict__ state,
                                                                           const int* __restrict__ first_chunk,
                                                                           const int* __restrict__ state_slots,
                                                                           int pairs) {
  constexpr int TD = D / 64;
  __shared__ dc_floatx4 parts[2][4][4][TIE_WAVE];
  const int pair = blockIdx.x % pairs, slab = blockIdx.x / pairs;      // the slabs of a head land on one XCD
  const int s = pair / g.heads, local = pair % g.heads, head = g.head0 + local;
  const int c0 = first_chunk[s], c1 = first_chunk[s + 1];
  if (c0 >= c1) return;                                                // the whole workgroup
  const int lane = threadIdx.x % TIE_WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / TIE_WAVE);
  const int r16 = lane & 15, quad = lane >> 4;
  const int col = slab * 16 + r16;
  const int row0 = wave * (D / 4) + quad * 4;                          // + 16 t + r
  float* slot = state + (static_cast<size_t>(state_slots[s]) * g.H + head) * g.d * g.e + col;
  dc_floatx4 S[TD];
#pragma unroll
  for (int t = 0; t < TD; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = row0 + 16 * t + r;
      S[t][r] = i < g.d && col < g.e ? slot[static_cast<size_t>(i) * g.e] : 0.f;
    }
  DeltaChunkOperands<TD> even, odd;
  auto step = [&](int c, DeltaChunkOperands<TD>& now, DeltaChunkOperands<TD>& next) {
    const size_t entry = static_cast<size_t>(c) * g.heads + local;
    delta_chunk_fetch<D, TD>(g, static_cast<size_t>(min(c + 1, c1 - 1)) * g.heads + local, wave, lane, slab, next);
    __builtin_amdgcn_sched_barrier(0);           // the loads stay ahead of the chunk's products
    float* s0 = g.s0 + ((entry * (g.ep / 16) + slab) * (D / 16) + wave * TD) * 256 + lane * 4;
#pragma unroll
    for (int t = 0; t < TD; ++t) *reinterpret_cast<dc_floatx4*>(s0 + t * 256) = S[t];
    dc_floatx4 acc[4];                         // W S - U0, of the wave's key rows
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      const bool mine = m == wave;
      acc[m] = dc_floatx4{mine ? -now.u0.x : 0.f, mine ? -now.u0.y : 0.f, mine ? -now.u0.z : 0.f, mine ? -now.u0.w : 0.f};
    }
#pragma unroll
    for (int t = 0; t < TD; ++t) {
#pragma unroll
      for (int m = 0; m < 4; ++m) acc[m] = dc_mfma(now.w[m][t].x, S[t][0], acc[m]);
#pragma unroll
      for (int m = 0; m < 4; ++m) acc[m] = dc_mfma(now.w[m][t].y, S[t][1], acc[m]);
#pragma unroll
      for (int m = 0; m < 4; ++m) acc[m] = dc_mfma(now.w[m][t].z, S[t][2], acc[m]);
#pragma unroll
      for (int m = 0; m < 4; ++m) acc[m] = dc_mfma(now.w[m][t].w, S[t][3], acc[m]);
    }
    dc_floatx4 (*buf)[4][TIE_WAVE] = parts[(c - c0) & 1];
#pragma unroll
    for (int m = 0; m < 4; ++m) buf[wave][m][lane] = acc[m];
    __syncthreads();
    dc_floatx4 U[4];
#pragma unroll
    for (int m = 0; m < 4; ++m)
      U[m] = -((buf[0][m][lane] + buf[1][m][lane]) + (buf[2][m][lane] + buf[3][m][lane]));
    *reinterpret_cast<dc_floatx4*>(g.u + ((entry * (g.ep / 16) + slab) * 4 + wave) * 256 + lane * 4) =
        wave == 0 ? U[0] : (wave == 1 ? U[1] : (wave == 2 ? U[2] : U[3]));
#pragma unroll
    for (int t = 0; t < TD; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t][r] *= now.decay;
#pragma unroll
    for (int m = 0; m < 4; ++m) {
#pragma unroll
      for (int t = 0; t < TD; ++t) S[t] = dc_mfma(now.k[t][m].x, U[m][0], S[t]);
#pragma unroll
      for (int t = 0; t < TD; ++t) S[t] = dc_mfma(now.k[t][m].y, U[m][1], S[t]);
#pragma unroll
      for (int t = 0; t < TD; ++t) S[t] = dc_mfma(now.k[t][m].z, U[m][2], S[t]);
#pragma unroll
      for (int t = 0; t < TD; ++t) S[t] = dc_mfma(now.k[t][m].w, U[m][3], S[t]);
    }
  };
  delta_chunk_fetch<D, TD>(g, static_cast<size_t>(c0) * g.heads + local, wave, lane, slab, even);
  for (int c = c0; c < c1; c += 2) {
    step(c, even, odd);
    if (c + 1 >= c1) break;
    step(c + 1, odd, even);
  }
#pragma unroll
  for (int t = 0; t < TD; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = row0 + 16 * t + r;
      if (i < g.d && col < g.e) slot[static_cast<size_t>(i) * g.e] = S[t][r];
    }
}

__global__ __launch_bounds__(DC_THREADS) void delta_chunk_outputs_kernel(DeltaChunks g, float* __restrict__ out,
                                                                         int out_row) {
  const int item = blockIdx.x / g.heads, head = g.head0 + blockIdx.x % g.heads;
  const int t0 = g.items[3 * item + 1], n = g.items[3 * item + 2] - t0;
  const size_t entry = blockIdx.x;
  const int lane = threadIdx.x % TIE_WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / TIE_WAVE);
  const int r16 = lane & 15, quad = lane >> 4;
  const int slab = blockIdx.y * 4 + wave, slabs = g.ep / 16, blocks = g.D / 16;
  if (slab >= slabs) return;                                           // the whole wave; there is no barrier below
  const float* q = g.q + entry * 4 * blocks * 256 + lane * 4;
  const float* s0 = g.s0 + (entry * slabs + slab) * blocks * 256 + lane * 4;
  dc_floatx4 acc[4];
#pragma unroll
  for (int m = 0; m < 4; ++m) acc[m] = dc_floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
  for (int kb = 0; kb < blocks; ++kb) {
    const dc_floatx4 v = *reinterpret_cast<const dc_floatx4*>(s0 + kb * 256);
    float4 a[4];
#pragma unroll
    for (int m = 0; m < 4; ++m) a[m] = *reinterpret_cast<const float4*>(q + (m * blocks + kb) * 256);
#pragma unroll
    for (int m = 0; m < 4; ++m) acc[m] = dc_mfma(a[m].x, v[0], acc[m]);
#pragma unroll
    for (int m = 0; m < 4; ++m) acc[m] = dc_mfma(a[m].y, v[1], acc[m]);
#pragma unroll
    for (int m = 0; m < 4; ++m) acc[m] = dc_mfma(a[m].z, v[2], acc[m]);
#pragma unroll
    for (int m = 0; m < 4; ++m) acc[m] = dc_mfma(a[m].w, v[3], acc[m]);
  }
  const float* pe = g.p + entry * DC_ROWS * DC_ROWS + lane * 4;
  const float* u = g.u + (entry * slabs + slab) * 4 * 256 + lane * 4;
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    const dc_floatx4 v = *reinterpret_cast<const dc_floatx4*>(u + jt * 256);
#pragma unroll
    for (int m = jt; m < 4; ++m) acc[m] = dc_mfma4(*reinterpret_cast<const float4*>(pe + (m * 4 + jt) * 256), v, acc[m]);
  }
  const int col = slab * 16 + r16;
  if (col >= g.e) return;
#pragma unroll
  for (int m = 0; m < 4; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = m * 16 + quad * 4 + r;
      if (i < n) out[static_cast<size_t>(t0 + i) * out_row + head * g.e + col] = acc[m][r];
    }
}

extern "C" int tie_delta_chunk_rows() { return DC_ROWS; }
// Key rows the chunks' memory is padded to.
extern "C" int tie_delta_chunk_dim(int d) { return d <= 64 ? 64 : (d <= 128 ? 128 : (d <= 256 ? 256 : 0)); }
// Floats of the memory of one (chunk, head).
extern "C" int tie_delta_chunk_floats(int d, int e) {
  const int D = tie_delta_chunk_dim(d), ep = (e + 15) / 16 * 16;
  return DC_ROWS * ep + 3 * DC_ROWS * D + DC_ROWS * DC_ROWS + 4 + D * ep;
}

// tok: rows of delta_prepare with one decay a head; out float32 [T][>= H e]; state [slots][H][d][e]; items [count][3]
// (sequence, first row, end row; at most 64 rows each) in the order of the rows, first_chunk [num_seqs + 1]; memory:
// count * heads * tie_delta_chunk_floats(d, e) floats on a 16-byte address. Runs heads head0 .. head0 + heads - 1.
extern "C" int tie_delta_chunks(const float* tok, int row, float* out, int out_row, float* state, const int* state_slots,
                                int num_seqs, const int* items, const int* first_chunk, int count, float* memory, int G,
                                int H, int d, int e, int head0, int heads, hipStream_t stream) {
  if (num_seqs <= 0 || count <= 0 || G <= 0 || H <= 0 || H % G || d <= 0 || d > 256 || e <= 0 || out_row < H * e ||
      row < 2 * G * d + H * e + 3 * H || head0 < 0 || heads <= 0 || head0 + heads > H || !items || !first_chunk ||
      !memory || reinterpret_cast<uintptr_t>(memory) % 16)
    return TIE_BAD_ARGUMENT;
  const int ep = (e + 15) / 16 * 16;
  const size_t entries = static_cast<size_t>(count) * heads;
  if (entries > 0x7fffffffu || static_cast<size_t>(num_seqs) * heads * (ep / 16) > 0x7fffffffu) return TIE_BAD_ARGUMENT;
  DeltaChunks g{};
  g.tok = tok, g.row = row, g.items = items, g.G = G, g.H = H, g.d = d, g.e = e;
  g.head0 = head0, g.heads = heads, g.ep = ep, g.D = tie_delta_chunk_dim(d);
  g.u = memory;
  g.w = g.u + entries * DC_ROWS * ep;
  g.kt = g.w + entries * DC_ROWS * g.D;
  g.q = g.kt + entries * DC_ROWS * g.D;
  g.p = g.q + entries * DC_ROWS * g.D;
  g.s0 = g.p + entries * DC_ROWS * DC_ROWS;
  g.decay = g.s0 + entries * g.D * ep;
  const bool wide = d % 4 == 0 && row % 4 == 0 && reinterpret_cast<uintptr_t>(tok) % 16 == 0;
  const size_t lds = sizeof(float) * DC_ROWS * (g.D + 4);
  static bool raised = false;
  if (!raised) {             // with the rest of its LDS the keys of 256 dimensions exceed the 64 KB of an ordinary launch
    for (const void* kernel : {reinterpret_cast<const void*>(&delta_chunk_prepare_kernel<true>),
                               reinterpret_cast<const void*>(&delta_chunk_prepare_kernel<false>)}) {
      const hipError_t err = hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize,
                                                 static_cast<int>(sizeof(float) * DC_ROWS * (256 + 4)));
      if (err != hipSuccess) return static_cast<int>(err);
    }
    raised = true;
  }
  if (wide) delta_chunk_prepare_kernel<true><<<static_cast<unsigned>(entries), DC_THREADS, lds, stream>>>(g);
  else delta_chunk_prepare_kernel<false><<<static_cast<unsigned>(entries), DC_THREADS, lds, stream>>>(g);
  int rc = tie_launch_status();
  if (rc != TIE_OK) return rc;
  const int pairs = num_seqs * heads;
  const unsigned walks = static_cast<unsigned>(pairs) * (ep / 16);
#define STATES(D) delta_chunk_states_kernel<D><<<walks, DC_THREADS, 0, stream>>>(g, state, first_chunk, state_slots, pairs)
  if (g.D == 64) STATES(64);
  else if (g.D == 128) STATES(128);
  else STATES(256);
#undef STATES
  rc = tie_launch_status();
  if (rc != TIE_OK) return rc;
  const dim3 grid(static_cast<unsigned>(entries), (ep + 63) / 64);
  delta_chunk_outputs_kernel<<<grid, DC_THREADS, 0, stream>>>(g, out, out_row);
  return tie_launch_status();
}
