// A mixer that carries a vector of fixed size from token to token instead of a cache of keys: an element-wise gated
// recurrence (mixers that keep a matrix a head are in matrix_state.hip), and the gated norm of heads' outputs side by side.
// States live in float32 in slots, state[slot][...], one slot a sequence (state_slots[s]); a step reads the state its
// sequence's earlier tokens left, runs the sequence's new rows query_start[s] .. query_start[s+1]-1 in order and writes the
// state back. What a token's output is depends on the tokens before it only, not on how they were cut into steps, beyond
// rounding.
//
// A sequence's tokens are a dependent chain, so a step of single tokens (or short portions) walks each sequence in
// one go (pass 0). A long portion would leave the GPU to a handful of waves; it is cut into chunks of rows
// instead (items = (sequence, first row, one past the last row), listed in the order of the rows) and run in three
// launches, all chunks side by side: pass 1 runs every chunk from a zero state and keeps what it ends with; the
// combine kernel walks a sequence's chunks in order, S <- A_chunk S + L_chunk, leaving every chunk the state it
// starts from and the slot the state after the last; pass 3 runs every chunk again from its true starting state
// and writes the outputs. The recurrence is linear in the state, which is all this needs.
//
// All arithmetic is float32; inputs are the float32 sums of the projections, activations are applied here.
#include "common.h"

#include <math.h>

__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float silu_f(float x) { return x / (1.0f + expf(-x)); }

// --------------------------------------------------- gated norm of the heads' outputs
// out[t] = RMSNorm(o[t]) * w * sigmoid(gate[t]) over rows of n values (all heads side by side); gate rows are
// gate_row floats apart (a view into the projection's rows). Statistics in float32.
template <typename TO>
__global__ void gated_rms_norm_kernel(const float* __restrict__ o, const float* __restrict__ w, float eps,
                                      const float* __restrict__ gate, int gate_row, TO* __restrict__ out, int n) {
  __shared__ float scratch[16];
  const size_t t = blockIdx.x;
  const float* r = o + t * n;
  const float* g = gate + t * gate_row;
  float ss = 0.f;
  for (int c = threadIdx.x; c < n; c += blockDim.x) ss = fmaf(r[c], r[c], ss);
  ss = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / static_cast<float>(n) + eps);
  for (int c = threadIdx.x; c < n; c += blockDim.x)
    store_from_float(out + t * n + c, (r[c] * inv) * w[c] * sigmoid_f(g[c]));
}

extern "C" int tie_gated_rms_norm(const float* o, const float* w, float eps, const float* gate, int gate_row, void* out,
                                  int out_dtype, int T, int n, hipStream_t stream) {
  if (T <= 0 || n <= 0 || gate_row < n) return TIE_BAD_ARGUMENT;
  const int threads = n >= 2048 ? 512 : (n >= 512 ? 256 : 64);
  if (out_dtype == TIE_F32)
    gated_rms_norm_kernel<float><<<T, threads, 0, stream>>>(o, w, eps, gate, gate_row, static_cast<float*>(out), n);
  else if (out_dtype == TIE_BF16)
    gated_rms_norm_kernel<bf16_t><<<T, threads, 0, stream>>>(o, w, eps, gate, gate_row, static_cast<bf16_t*>(out), n);
  else
    return TIE_BAD_ARGUMENT;
  return tie_launch_status();
}

// ------------------------------------------------------------- minimal gated recurrent unit
// Element by element: z = sigmoid(a), c = candidate(u) = u + 1/2 (u >= 0) or sigmoid(u) (u < 0),
// S_t = (1 - z) S_(t-1) + z c, out_t = S_t * silu(g). Row t of `proj` holds [a (n) | u (n) | g (n)]; `bias` (or
// null) holds 3 n values that are added to them here, so that the projection needs no pass of its own for them.
// A thread owns one channel of one sequence and walks its rows; neighbouring threads read neighbouring floats.
// Chunks (see the top): pass 1 leaves a chunk's product of (1 - z) in chunk_a and what it ends with from zero in
// chunk_b; the combine kernel turns chunk_b into the state each chunk starts from; pass 3 writes the outputs.
template <typename TO, int PASS>
__global__ void min_gru_scan_kernel(const float* __restrict__ proj, int row, TO* __restrict__ out,
                                    float* __restrict__ state, const int* __restrict__ query_start,
                                    const int* __restrict__ state_slots, int n, const int* __restrict__ items,
                                    float* __restrict__ chunk_a, float* __restrict__ chunk_b,
                                    const float* __restrict__ bias) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= n) return;
  const float ba = bias ? bias[c] : 0.f, bu = bias ? bias[n + c] : 0.f, bg = bias ? bias[2 * n + c] : 0.f;
  const int s = PASS == 0 ? static_cast<int>(blockIdx.y) : items[blockIdx.y * 3];
  float* sp = PASS == 0 ? state + static_cast<size_t>(state_slots[s]) * n + c
                        : chunk_b + static_cast<size_t>(blockIdx.y) * n + c;
  float st = PASS == 1 ? 0.f : *sp;
  float keep = 1.f;
  const int t0 = PASS == 0 ? query_start[s] : items[blockIdx.y * 3 + 1];
  const int t1 = PASS == 0 ? query_start[s + 1] : items[blockIdx.y * 3 + 2];
  // Eight tokens' values are asked for before the first of them is used: the chain through the state is short
  // arithmetic, and what it would otherwise wait for, token after token, is memory.
  constexpr int AHEAD = 8;
  for (int t = t0; t < t1; t += AHEAD) {
    float a[AHEAD], u[AHEAD], g[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      const float* r = proj + static_cast<size_t>(min(t + j, t1 - 1)) * row + c;
      a[j] = r[0];
      u[j] = r[n];
      g[j] = PASS == 1 ? 0.f : r[2 * static_cast<size_t>(n)];
    }
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      if (t + j >= t1) break;
      const float z = sigmoid_f(a[j] + ba);
      const float x = u[j] + bu;
      const float cand = x >= 0.f ? x + 0.5f : sigmoid_f(x);
      st = fmaf(z, cand, (1.0f - z) * st);
      if (PASS == 1) keep *= 1.0f - z;
      else store_from_float(out + static_cast<size_t>(t + j) * n + c, st * silu_f(g[j] + bg));
    }
  }
  if (PASS == 3) return;
  *sp = st;
  if (PASS == 1) chunk_a[static_cast<size_t>(blockIdx.y) * n + c] = keep;
}

__global__ void min_gru_combine_kernel(const float* __restrict__ chunk_a, float* __restrict__ chunk_b,
                                       float* __restrict__ state, const int* __restrict__ first_item,
                                       const int* __restrict__ state_slots, int n) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= n) return;
  const int s = blockIdx.y;
  float* slot = state + static_cast<size_t>(state_slots[s]) * n + c;
  float S = *slot;
  for (int i = first_item[s]; i < first_item[s + 1]; ++i) {
    const float local = chunk_b[static_cast<size_t>(i) * n + c];
    chunk_b[static_cast<size_t>(i) * n + c] = S;
    S = fmaf(chunk_a[static_cast<size_t>(i) * n + c], S, local);
  }
  *slot = S;
}

// num_items = 0: every sequence in one go; otherwise items, first_item as for the linear attention and chunk_ab
// [2][num_items][n] scratch memory.
extern "C" int tie_min_gru_scan(const float* proj, int row, void* out, int out_dtype, float* state,
                                const int* query_start, const int* state_slots, int S, int n, const int* items,
                                const int* first_item, int num_items, float* chunk_ab, const float* bias,
                                hipStream_t stream) {
  if (S <= 0 || S > 65535 || n <= 0 || row < 3 * n || num_items < 0 || num_items > 65535 ||
      (num_items > 0 && (items == nullptr || first_item == nullptr || chunk_ab == nullptr)) ||
      (out_dtype != TIE_F32 && out_dtype != TIE_BF16))
    return TIE_BAD_ARGUMENT;
  const int threads = n >= 256 ? 256 : 64;
  const unsigned across = (n + threads - 1) / threads;
  float* chunk_a = chunk_ab;
  float* chunk_b = chunk_ab == nullptr ? nullptr : chunk_ab + static_cast<size_t>(num_items) * n;
#define LAUNCH_PASS(TO, PASS, COUNT)                                                                              \
  min_gru_scan_kernel<TO, PASS><<<dim3(across, COUNT), threads, 0, stream>>>(                                     \
      proj, row, static_cast<TO*>(out), state, query_start, state_slots, n, items, chunk_a, chunk_b, bias)
#define LAUNCH(TO)                                                                                                \
  {                                                                                                               \
    if (num_items == 0) {                                                                                         \
      LAUNCH_PASS(TO, 0, S);                                                                                      \
    } else {                                                                                                      \
      LAUNCH_PASS(TO, 1, num_items);                                                                              \
      min_gru_combine_kernel<<<dim3(across, S), threads, 0, stream>>>(chunk_a, chunk_b, state, first_item,        \
                                                                      state_slots, n);                            \
      LAUNCH_PASS(TO, 3, num_items);                                                                              \
    }                                                                                                             \
  }
  if (out_dtype == TIE_F32) LAUNCH(float)
  else LAUNCH(bf16_t)
#undef LAUNCH
#undef LAUNCH_PASS
  return tie_launch_status();
}
