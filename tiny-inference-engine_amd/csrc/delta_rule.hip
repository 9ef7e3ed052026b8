// Short causal convolutions over time with a state per sequence, and the gated delta rule.
//
// Short convolution: y_t[c] = sum_j w[c][j] * u_(t - taps + 1 + j)[c], zeros before a sequence's first token. The
// last taps - 1 inputs u of a sequence live in its state slot `[slots][taps - 1][C]` (the newest last), so a
// sequence may be cut into steps anywhere. The kernels that convolve read the state; `conv_state_update` writes it
// in a launch of its own behind them, so no reader meets a writer.
//
// Gated delta rule, per value head with state S `[key_dim][value_dim]` (float32, in the sequence's slot):
//   S <- diag(g) S ;  u = beta (v - S^T k) ;  S <- S + k u^T ;  o = S^T q
// with q and k unit vectors (q also times key_dim^(-1/2)), beta in (0, 1) and decays in (0, 1): one per head and
// key channel, or one per head. `delta_prepare` makes q, k, v, beta and g of every token of a step, in parallel over tokens;
// `gated_delta_scan` walks each sequence's tokens in order.
#include "common.h"

#define CONV_MAX_TAPS 8

__device__ __forceinline__ float silu_f(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// The same for a sequence's only row of a step, whose channel c no other thread reads: the state takes the row's input.
__device__ __forceinline__ float conv_and_shift(float u, const float* __restrict__ w, float* hist, int taps, int C, int c) {
  float past[CONV_MAX_TAPS - 1];
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS - 1; ++j)
    if (j < taps - 1) past[j] = hist[static_cast<size_t>(j) * C + c];
  float y = 0.f;
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS - 1; ++j)
    if (j < taps - 1) y = fmaf(w[c * taps + j], past[j], y);
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS - 1; ++j)
    if (j < taps - 1) hist[static_cast<size_t>(j) * C + c] = j + 1 < taps - 1 ? past[j + 1 < CONV_MAX_TAPS - 1 ? j + 1 : j] : u;
  return fmaf(w[c * taps + taps - 1], u, y);
}

// The convolution's sum for row t (of the sequence that starts at row `start`), channel c of the C convolved
// columns, whose inputs are columns of `u` rows `row` apart.
__device__ __forceinline__ float conv_at(const float* __restrict__ u, size_t row, const float* __restrict__ w,
                                         const float* __restrict__ hist, int taps, int C, int t, int start, int c) {
  float y = 0.f;
  for (int j = 0; j < taps; ++j) {
    const int src = t - (taps - 1) + j;
    // before the step's first row of the sequence: the state, whose entry i is the input of row start - (taps-1) + i
    const float v = src >= start ? u[static_cast<size_t>(src) * row + c]
                                 : hist[static_cast<size_t>(src - start + taps - 1) * C + c];
    y = fmaf(w[c * taps + j], v, y);
  }
  return y;
}

// ---------------------------------------------------------------- q, k, v of an attention with short convolutions
// Row t of `u` holds [q (nq) | k (nk) | v (nv)] as projected (C = nq + nk + nv columns are convolved). out row:
// the same columns convolved; then, where wq / wk are given, q and k each divided by the root mean square over
// their whole width (all heads together; mean over `count_q` / `count_k` values, which may be fewer than the
// columns where heads carry padding columns of zeros) and multiplied by their weights.
__global__ void conv_qkv_kernel(const float* __restrict__ u, int row, const float* __restrict__ w, int taps,
                                const float* __restrict__ state, const int* __restrict__ state_slots,
                                const int* __restrict__ seq_of_row, const int* __restrict__ query_start,
                                int nq, int nk, int nv, const float* __restrict__ wq, const float* __restrict__ wk,
                                float count_q, float count_k, float eps, float* __restrict__ out, int out_row) {
  extern __shared__ float vals[];
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  const int s = seq_of_row[t];
  const int start = query_start[s];
  const int C = nq + nk + nv;
  const float* hist = state + static_cast<size_t>(state_slots[s]) * (taps - 1) * C;
  // three workgroups a row: q, k and v each on their own (a norm runs over one of them)
  const int lo = blockIdx.y == 0 ? 0 : (blockIdx.y == 1 ? nq : nq + nk);
  const int hi = blockIdx.y == 0 ? nq : (blockIdx.y == 1 ? nq + nk : C);
  float sq = 0.f, sk = 0.f;
  for (int c = lo + threadIdx.x; c < hi; c += blockDim.x) {
    const float y = taps > 1 ? conv_at(u, row, w, hist, taps, C, t, start, c)
                             : w[c] * u[static_cast<size_t>(t) * row + c];
    vals[c] = y;
    if (c < nq) sq = fmaf(y, y, sq);
    else if (c < nq + nk) sk = fmaf(y, y, sk);
  }
  float iq = 1.f, ik = 1.f;
  if (wq && blockIdx.y == 0) iq = 1.0f / sqrtf(block_sum(sq, scratch) / count_q + eps);
  if (wk && blockIdx.y == 1) ik = 1.0f / sqrtf(block_sum(sk, scratch) / count_k + eps);
  __syncthreads();
  float* o = out + static_cast<size_t>(t) * out_row;
  for (int c = lo + threadIdx.x; c < hi; c += blockDim.x) {
    float y = vals[c];
    if (c < nq) { if (wq) y = (y * iq) * wq[c]; }
    else if (c < nq + nk) { if (wk) y = (y * ik) * wk[c - nq]; }
    o[c] = y;
  }
}

extern "C" int tie_conv_qkv(const float* u, int row, const float* w, int taps, const float* state,
                            const int* state_slots, const int* seq_of_row, const int* query_start, int T, int nq,
                            int nk, int nv, const float* wq, const float* wk, float count_q, float count_k, float eps,
                            float* out, int out_row, hipStream_t stream) {
  const int C = nq + nk + nv;
  if (T <= 0 || C <= 0 || taps < 1 || taps > CONV_MAX_TAPS || row < C || out_row < C ||
      static_cast<size_t>(C) * 4 > 65536 || (taps > 1 && !state))
    return TIE_BAD_ARGUMENT;
  // few channels a thread: every one waits for its loads, and a decode step brings few rows
  const int threads = C >= 2048 ? 1024 : (C >= 1024 ? 512 : (C >= 512 ? 256 : 128));
  conv_qkv_kernel<<<dim3(T, 3), threads, static_cast<size_t>(C) * sizeof(float), stream>>>(
      u, row, w, taps, state, state_slots, seq_of_row, query_start, nq, nk, nv, wq, wk, count_q, count_k, eps, out,
      out_row);
  return tie_launch_status();
}

// ---------------------------------------------------------------- the state of a short convolution after a step
// new[i] = input of row end - (taps - 1) + i: a row of this step, or what the old state held for it.
__global__ void conv_state_update_kernel(const float* __restrict__ u, int row, int taps, float* __restrict__ state,
                                         const int* __restrict__ state_slots, const int* __restrict__ query_start,
                                         int C) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= C) return;
  const int s = blockIdx.y;
  const int start = query_start[s], end = query_start[s + 1];
  const int hist = taps - 1;
  float* st = state + static_cast<size_t>(state_slots[s]) * hist * C;
  float keep[CONV_MAX_TAPS];
#pragma unroll
  for (int i = 0; i < CONV_MAX_TAPS - 1; ++i) {
    if (i >= hist) break;
    const int src = end - hist + i;
    keep[i] = src >= start ? u[static_cast<size_t>(src) * row + c]
                           : st[static_cast<size_t>(src - start + hist) * C + c];
  }
#pragma unroll
  for (int i = 0; i < CONV_MAX_TAPS - 1; ++i) {
    if (i >= hist) break;
    st[static_cast<size_t>(i) * C + c] = keep[i];
  }
}

extern "C" int tie_conv_state_update(const float* u, int row, int taps, float* state, const int* state_slots,
                                     const int* query_start, int num_seqs, int C, hipStream_t stream) {
  if (num_seqs <= 0 || C <= 0 || taps < 1 || taps > CONV_MAX_TAPS || row < C) return TIE_BAD_ARGUMENT;
  if (taps == 1) return TIE_OK;
  conv_state_update_kernel<<<dim3((C + 255) / 256, num_seqs), 256, 0, stream>>>(u, row, taps, state, state_slots,
                                                                                query_start, C);
  return tie_launch_status();
}

// ---------------------------------------------------------------- what the delta rule takes of a token
// Row t of `u`: [q (G d) | k (G d) | v (H e) | b (H)], the first C = 2 G d + H e columns convolved, then silu.
// Row t of `a`: the decay's argument (H da), `a_row` apart, da = d or 1 (one decay a head). out row: [q^ | k^ | v |
// g (H da) | beta (H)] and, with one decay a head, the decays' logarithms (H) behind:
//   q^, k^ unit vectors per head (x / sqrt(sum x^2 + 1e-6)), q^ also times d^(-1/2); beta = sigmoid(b);
//   g = exp(-exp(A_log[head]) * softplus(a + dt_bias)).
// SHIFT: every sequence has one row, and the convolution's state is brought up to date here (`shifted` is the state;
// otherwise `state`, which is only read).
template <bool SHIFT>
__global__ void delta_prepare_kernel(const float* __restrict__ u, int row, const float* __restrict__ w, int taps,
                                     const float* __restrict__ state, float* shifted, const int* __restrict__ state_slots,
                                     const int* __restrict__ seq_of_row, const int* __restrict__ query_start,
                                     const float* __restrict__ a, int a_row, const float* __restrict__ A_log,
                                     const float* __restrict__ dt_bias, int G, int H, int d, int e, int da,
                                     float* __restrict__ out, int out_row) {
  extern __shared__ float vals[];
  const int t = blockIdx.x;
  const int s = seq_of_row[t];
  const int start = query_start[s];
  const int C = 2 * G * d + H * e;
  const size_t slot_at = static_cast<size_t>(state_slots[s]) * (taps - 1) * C;
  float* o = out + static_cast<size_t>(t) * out_row;
  // three workgroups a row: q and k with their unit norms, v, and beta with the decays
  if (blockIdx.y == 2) {
    const float* b = u + static_cast<size_t>(t) * row + C;
    for (int h = threadIdx.x; h < H; h += blockDim.x) o[C + H * da + h] = sigmoid_f(b[h]);
    const float* ar = a + static_cast<size_t>(t) * a_row;
    for (int c = threadIdx.x; c < H * da; c += blockDim.x) {
      const float log_g = -expf(A_log[c / da]) * softplus_f(ar[c] + dt_bias[c]);
      o[C + c] = expf(log_g);
      if (da == 1) o[C + 2 * H + c] = log_g;
    }
    return;
  }
  const int lo = blockIdx.y == 0 ? 0 : 2 * G * d, hi = blockIdx.y == 0 ? 2 * G * d : C;
  for (int c = lo + threadIdx.x; c < hi; c += blockDim.x) {
    const float y = taps == 1 ? w[c] * u[static_cast<size_t>(t) * row + c]
                    : SHIFT   ? conv_and_shift(u[static_cast<size_t>(t) * row + c], w, shifted + slot_at, taps, C, c)
                              : conv_at(u, row, w, state + slot_at, taps, C, t, start, c);
    if (blockIdx.y == 0) vals[c] = silu_f(y);
    else o[c] = silu_f(y);
  }
  if (blockIdx.y == 1) return;
  __syncthreads();
  const int lane = threadIdx.x & (TIE_WAVE - 1), wave = threadIdx.x / TIE_WAVE, waves = blockDim.x / TIE_WAVE;
  const float q_scale = 1.0f / sqrtf(static_cast<float>(d));
  for (int head = wave; head < 2 * G; head += waves) {      // q heads, then k heads
    const float* x = vals + head * d;
    float ss = 0.f;
    for (int i = lane; i < d; i += TIE_WAVE) ss = fmaf(x[i], x[i], ss);
    const float inv = 1.0f / sqrtf(wave_sum(ss) + 1e-6f);
    const float f = head < G ? inv * q_scale : inv;
    for (int i = lane; i < d; i += TIE_WAVE) o[head * d + i] = x[i] * f;
  }
}

// The same for many rows: a wave takes the channels of one q or k head, or 64 PER channels of v, and walks
// DELTA_WALK_ROWS rows with the convolution's window in registers, so that an input is read once instead of once a tap;
// lane l holds channels l, l + 64, ... The units behind them make the decays, 64 PER columns each, the first of them beta too.
#define DELTA_WALK_ROWS 16
#define DELTA_WALK_WAVES 4

template <int PER, int TAPS>
__global__ __launch_bounds__(DELTA_WALK_WAVES* TIE_WAVE) void delta_prepare_walk_kernel(
    const float* __restrict__ u, int row, const float* __restrict__ w, const float* __restrict__ state,
    const int* __restrict__ state_slots, const int* __restrict__ seq_of_row, const int* __restrict__ query_start,
    const float* __restrict__ a, int a_row, const float* __restrict__ A_log, const float* __restrict__ dt_bias, int T,
    int G, int H, int d, int e, int da, float* __restrict__ out, int out_row, int units) {
  const int unit = blockIdx.x * DELTA_WALK_WAVES + threadIdx.x / TIE_WAVE, lane = threadIdx.x % TIE_WAVE;
  if (unit >= units) return;                       // the whole wave; there is no barrier below
  const int first = blockIdx.y * DELTA_WALK_ROWS, rows = min(DELTA_WALK_ROWS, T - first);
  const int C = 2 * G * d + H * e;
  const int decays = 2 * G + (H * e + TIE_WAVE * PER - 1) / (TIE_WAVE * PER);        // the first unit of the decays
  if (unit >= decays) {
    const int lo = (unit - decays) * TIE_WAVE * PER, width = min(TIE_WAVE * PER, H * da - lo);
    for (int i = lane; i < rows * width; i += TIE_WAVE) {
      const int t = first + i / width, c = lo + i % width;
      float* o = out + static_cast<size_t>(t) * out_row;
      const float log_g = -expf(A_log[c / da]) * softplus_f(a[static_cast<size_t>(t) * a_row + c] + dt_bias[c]);
      o[C + c] = expf(log_g);
      if (da == 1) o[C + 2 * H + c] = log_g;
    }
    if (unit > decays) return;
    for (int i = lane; i < rows * H; i += TIE_WAVE) {
      const int t = first + i / H, h = i % H;
      out[static_cast<size_t>(t) * out_row + C + H * da + h] = sigmoid_f(u[static_cast<size_t>(t) * row + C + h]);
    }
    return;
  }
  const bool head = unit < 2 * G;                  // a q or k head: a unit vector
  const int c0 = head ? unit * d : 2 * G * d + (unit - 2 * G) * TIE_WAVE * PER;
  const int width = head ? d : min(TIE_WAVE * PER, C - c0);
  const float scale = unit < G ? 1.0f / sqrtf(static_cast<float>(d)) : 1.0f;
  int ch[PER];
  float wt[TAPS][PER], win[TAPS][PER];             // win: the inputs of rows t - TAPS + 1 .. t
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    ch[p] = c0 + min(lane + p * TIE_WAVE, width - 1);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) wt[j][p] = w[ch[p] * TAPS + j];
  }
  int start = 0, left = 0;                         // the first row of t's sequence, rows left in it
  constexpr int AHEAD = 4;                         // rows asked for before they are needed
  float ahead[AHEAD][PER];
#pragma unroll
  for (int r = 0; r < AHEAD; ++r)
#pragma unroll
    for (int p = 0; p < PER; ++p) ahead[r][p] = u[static_cast<size_t>(first + min(r, rows - 1)) * row + ch[p]];
  for (int r = 0; r < rows; ++r) {
    const int t = first + r;
    if (left == 0) {                               // a sequence begins here, or this wave's rows do
      const int s = seq_of_row[t];
      start = query_start[s];
      left = query_start[s + 1] - t;
      const float* hist = state + static_cast<size_t>(state_slots[s]) * (TAPS - 1) * C;
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) {
        const int src = t - (TAPS - 1) + j;
        const float* from = src >= start ? u + static_cast<size_t>(src) * row
                                         : hist + static_cast<size_t>(src - start + TAPS - 1) * C;
#pragma unroll
        for (int p = 0; p < PER; ++p) win[j][p] = from[ch[p]];
      }
    }
    --left;
    float y[PER], ss = 0.f;
#pragma unroll
    for (int p = 0; p < PER; ++p) {
      win[TAPS - 1][p] = ahead[0][p];
#pragma unroll
      for (int j = 0; j + 1 < AHEAD; ++j) ahead[j][p] = ahead[j + 1][p];
      ahead[AHEAD - 1][p] = u[static_cast<size_t>(first + min(r + AHEAD, rows - 1)) * row + ch[p]];
      float v = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) v = fmaf(wt[j][p], win[j][p], v);
      y[p] = silu_f(v);
      if (lane + p * TIE_WAVE < width) ss = fmaf(y[p], y[p], ss);
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) win[j][p] = win[j + 1][p];
    }
    const float f = head ? 1.0f / sqrtf(wave_sum(ss) + 1e-6f) * scale : 1.0f;
    float* o = out + static_cast<size_t>(t) * out_row;
#pragma unroll
    for (int p = 0; p < PER; ++p)
      if (lane + p * TIE_WAVE < width) o[ch[p]] = y[p] * f;
  }
}

#define DELTA_WALK_FROM 128       // rows of a step from which the walk runs

extern "C" int tie_delta_prepare(const float* u, int row, const float* w, int taps, float* state, int shift,
                                 const int* state_slots, const int* seq_of_row, const int* query_start,
                                 const float* a, int a_row, const float* A_log, const float* dt_bias, int T, int G,
                                 int H, int d, int e, int head_decay, float* out, int out_row, hipStream_t stream) {
  const int C = 2 * G * d + H * e;
  const int da = head_decay ? 1 : d;
  if (T <= 0 || G <= 0 || H <= 0 || d <= 0 || e <= 0 || taps < 1 || taps > CONV_MAX_TAPS || row < C + H ||
      out_row < C + H + (head_decay ? 2 * H : H * d) || a_row < H * da || static_cast<size_t>(C) * 4 > 65536 || (taps > 1 && !state))
    return TIE_BAD_ARGUMENT;
  if (T >= DELTA_WALK_FROM && !shift && taps >= 2 && taps <= 4 && d <= 4 * TIE_WAVE) {
    const int per = d <= TIE_WAVE ? 1 : (d <= 2 * TIE_WAVE ? 2 : 4);
    const int per_unit = TIE_WAVE * per;
    const int units = 2 * G + (H * e + per_unit - 1) / per_unit + (H * da + per_unit - 1) / per_unit;
    const dim3 grid((units + DELTA_WALK_WAVES - 1) / DELTA_WALK_WAVES, (T + DELTA_WALK_ROWS - 1) / DELTA_WALK_ROWS);
#define WALK(PER, TAPS)                                                                                            \
  delta_prepare_walk_kernel<PER, TAPS><<<grid, DELTA_WALK_WAVES * TIE_WAVE, 0, stream>>>(                           \
      u, row, w, state, state_slots, seq_of_row, query_start, a, a_row, A_log, dt_bias, T, G, H, d, e, da, out, out_row, \
      units)
#define WALKS(PER)                                                                             \
  {                                                                                            \
    if (taps == 2) WALK(PER, 2); else if (taps == 3) WALK(PER, 3); else WALK(PER, 4);          \
  }
    if (per == 1) WALKS(1) else if (per == 2) WALKS(2) else WALKS(4)
#undef WALKS
#undef WALK
    return tie_launch_status();
  }
  const int threads = C >= 2048 ? 1024 : (C >= 1024 ? 512 : 256);
  const size_t lds = static_cast<size_t>(C) * sizeof(float);
  if (shift && taps > 1)
    delta_prepare_kernel<true><<<dim3(T, 3), threads, lds, stream>>>(u, row, w, taps, nullptr, state, state_slots,
                                                                     seq_of_row, query_start, a, a_row, A_log, dt_bias,
                                                                     G, H, d, e, da, out, out_row);
  else
    delta_prepare_kernel<false><<<dim3(T, 3), threads, lds, stream>>>(u, row, w, taps, state, nullptr, state_slots,
                                                                      seq_of_row, query_start, a, a_row, A_log, dt_bias,
                                                                      G, H, d, e, da, out, out_row);
  return tie_launch_status();
}

// ---------------------------------------------------------------- the recurrence
// A wave owns DELTA_COLS value columns of one (sequence, value head): lane l holds rows [p R, (p + 1) R) of column
// l / 8 in registers, p = l % 8 (R = key rows a lane: an eighth of key_dim rounded up to 4, 8, 16 or 32; rows
// beyond key_dim stay zero), so the two sums over key rows (S^T k, S^T q) meet inside eight neighbouring lanes,
// through three lane permutations each and without a barrier. The DELTA_WAVES waves of a workgroup take columns
// side by side and share the token's k, q and g in LDS, staged NT tokens at a time (the next ones are on their way
// from memory meanwhile, four words a load where the row's layout allows; one decay a head travels with the values
// instead), every p's rows four words behind the
// last one's so that the eight addresses of one read fall into different banks; the lanes of one p read the same
// words. A token's words are in registers before the token before it is done.
#define DELTA_COLS 8
#define DELTA_PARTS 8
#define DELTA_WAVES 4
#define DELTA_THREADS (DELTA_WAVES * TIE_WAVE)

__device__ __forceinline__ float part_sum(float v) {     // over the DELTA_PARTS lanes of a column
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xf, 0xf, false));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x4E, 0xf, 0xf, false));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x141, 0xf, 0xf, false));
  return v;
}

// Where a head's columns lie inside a token's row, and where the sequence's tokens end.
struct DeltaRowPlan {
  int k_at, q_at, g_at, v_at, b_at, first_col, d, e, t1, row;
};

// k, q and g (VECS 3; 2: without g) of the tokens tb .. tb + NT - 1 of the head (padded to DP rows) into registers, W
// words a load: entry (x * DELTA_THREADS + thread) * W of [token][k, q, g][row]. Every load is issued whether it counts or not
// (from an address that exists), so that none waits for a branch.
template <int DP, int NT, int VECS, int W, int PER>
__device__ __forceinline__ void delta_fetch(const float* __restrict__ tok, const DeltaRowPlan pl, int tb,
                                            float (&stage)[PER][W]) {
  const float* first = tok + static_cast<size_t>(tb) * pl.row;
  const int left = pl.t1 - tb;                    // tokens from tb on, at least one
#pragma unroll
  for (int x = 0; x < PER; ++x) {
    const int idx = (x * DELTA_THREADS + static_cast<int>(threadIdx.x)) * W;
    const int tk = idx / (VECS * DP), rest = idx % (VECS * DP), which = rest / DP, i = rest % DP;
    const float* r = first + static_cast<size_t>(min(tk, left - 1)) * pl.row +
                     (which == 0 ? pl.k_at : (which == 1 ? pl.q_at : pl.g_at));
    const float pad = which == 2 ? 1.f : 0.f;      // padding rows: no key, no query, no decay
    if constexpr (W == 4) {                        // d is a multiple of 4: the four rows count together
      const float4 v = *reinterpret_cast<const float4*>(r + min(i, pl.d - 4));
      const bool in = tk < left && i < pl.d;
      stage[x][0] = in ? v.x : pad, stage[x][1] = in ? v.y : pad, stage[x][2] = in ? v.z : pad, stage[x][3] = in ? v.w : pad;
    } else {
      const float v = r[min(i, pl.d - 1)];
      stage[x][0] = (tk < left && i < pl.d) ? v : pad;
    }
  }
}

// The values of the wave's columns and beta (EXTRA 2: and the head's decay) of the same tokens: entry j * 64 + lane of
// [token][columns, beta, decay].
template <int NT, int EXTRA, int VB>
__device__ __forceinline__ void delta_fetch_values(const float* __restrict__ tok, const DeltaRowPlan pl, int tb,
                                                   int lane, float (&stage_vb)[VB]) {
  const float* first = tok + static_cast<size_t>(tb) * pl.row;
  const int left = pl.t1 - tb;
#pragma unroll
  for (int j = 0; j < VB; ++j) {
    const int idx = j * TIE_WAVE + lane;
    const int tk = idx / (DELTA_COLS + EXTRA), x = idx % (DELTA_COLS + EXTRA);
    const float* r = first + static_cast<size_t>(min(tk, left - 1)) * pl.row;
    const float v = r[x == DELTA_COLS ? pl.b_at : (x > DELTA_COLS ? pl.g_at : pl.v_at + min(pl.first_col + x, pl.e - 1))];
    stage_vb[j] = (tk < NT && tk < left && (x >= DELTA_COLS || pl.first_col + x < pl.e)) ? v : 0.f;
  }
}

// One token through the lane's rows: S <- g S; u = beta (v - S^T k); S <- S + k u; returns S^T q. GR = R: a decay a
// row; GR = 1: one for all of them.
template <int R, int GR>
__device__ __forceinline__ float delta_token(float (&S)[R], const float (&kk)[R], const float (&qq)[R],
                                             const float (&gg)[GR], float v, float beta) {
  float dot0 = 0.f, dot1 = 0.f, dot2 = 0.f, dot3 = 0.f;
#pragma unroll
  for (int r = 0; r < R; r += 4) {
    S[r] *= gg[r % GR];
    S[r + 1] *= gg[(r + 1) % GR];
    S[r + 2] *= gg[(r + 2) % GR];
    S[r + 3] *= gg[(r + 3) % GR];
    dot0 = fmaf(S[r], kk[r], dot0);
    dot1 = fmaf(S[r + 1], kk[r + 1], dot1);
    dot2 = fmaf(S[r + 2], kk[r + 2], dot2);
    dot3 = fmaf(S[r + 3], kk[r + 3], dot3);
  }
  const float u = beta * (v - part_sum((dot0 + dot1) + (dot2 + dot3)));
  float o0 = 0.f, o1 = 0.f, o2 = 0.f, o3 = 0.f;
#pragma unroll
  for (int r = 0; r < R; r += 4) {
    S[r] = fmaf(kk[r], u, S[r]);
    S[r + 1] = fmaf(kk[r + 1], u, S[r + 1]);
    S[r + 2] = fmaf(kk[r + 2], u, S[r + 2]);
    S[r + 3] = fmaf(kk[r + 3], u, S[r + 3]);
    o0 = fmaf(S[r], qq[r], o0);
    o1 = fmaf(S[r + 1], qq[r + 1], o1);
    o2 = fmaf(S[r + 2], qq[r + 2], o2);
    o3 = fmaf(S[r + 3], qq[r + 3], o3);
  }
  return part_sum((o0 + o1) + (o2 + o3));
}

// What a launch of the scan walks. Without `items` a workgroup's rows are a sequence's rows of the step and its
// state the sequence's slot. With `items` ([count][3]: sequence, first row, end row) they are one chunk's, and the
// state is entry `item` of `state`. A state has `columns` columns: e, or e + d where the columns from e on carry the
// chunk's transition (they start as the identity and take no values, so they end as the product of the tokens'
// transition matrices, which is what the state before the chunk is multiplied by).
struct DeltaScanMode {
  const int* items;
  int columns;
  int init;      // 0: the state is read; 1: it starts as zeros (and the identity from column e on)
  int store;     // the state is written back at the end
  int outputs;   // outputs are written
};

template <int R, int W, bool HEAD_DECAY>
__global__ __launch_bounds__(DELTA_THREADS) void gated_delta_scan_kernel(
    const float* __restrict__ tok, int row, float* __restrict__ out, int out_row, float* __restrict__ state,
    const int* __restrict__ query_start, const int* __restrict__ state_slots, int G, int H, int d, int e,
    DeltaScanMode mode) {
  constexpr int DP = R * DELTA_PARTS;                 // padded key rows
  constexpr int RP = R + 4;                           // words from one p's rows to the next one's in LDS
  constexpr int NT = 4 * DELTA_THREADS / DP;          // tokens staged at a time: 4 to 32
  constexpr int VECS = HEAD_DECAY ? 2 : 3;            // k, q and, with a decay a key channel, g
  constexpr int GR = HEAD_DECAY ? 1 : R;
  constexpr int VW = DELTA_COLS + (HEAD_DECAY ? 2 : 1);
  constexpr int PER = NT * VECS * DP / (DELTA_THREADS * W);
  constexpr int VB = (NT * VW + TIE_WAVE - 1) / TIE_WAVE;
  __shared__ __attribute__((aligned(16))) float kqg[NT * VECS * DELTA_PARTS * RP];   // [token][k, q, g][p][row]
  __shared__ float vbs[DELTA_WAVES][NT * VW];     // a wave: [token][the values of its columns, beta, one decay]
  const int item = blockIdx.x / H, head = blockIdx.x % H;
  const int kv = head / (H / G);
  const int wave = threadIdx.x / TIE_WAVE, lane = threadIdx.x % TIE_WAVE;
  const int p = lane & (DELTA_PARTS - 1), c = lane / DELTA_PARTS;
  const int first_col = (blockIdx.y * DELTA_WAVES + wave) * DELTA_COLS;
  const int col = first_col + c;
  const int columns = mode.columns;
  const bool live = col < columns;
  int t0, t1, holder;
  if (mode.items) {
    t0 = mode.items[3 * item + 1], t1 = mode.items[3 * item + 2], holder = item;
  } else {
    t0 = query_start[item], t1 = query_start[item + 1], holder = state_slots[item];
  }
  if (t0 >= t1) return;                               // the whole workgroup
  float* sp = state + ((static_cast<size_t>(holder) * H + head) * d) * columns + col;
  float S[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int i = p * R + r;
    if (mode.init) S[r] = (live && col - e == i) ? 1.f : 0.f;
    else S[r] = (live && i < d) ? sp[static_cast<size_t>(i) * columns] : 0.f;
  }
  DeltaRowPlan pl;
  pl.q_at = kv * d;
  pl.k_at = G * d + kv * d;
  pl.v_at = 2 * G * d + head * e;
  pl.g_at = 2 * G * d + H * e + (HEAD_DECAY ? head : head * d);
  pl.b_at = 2 * G * d + H * e + (HEAD_DECAY ? H : H * d) + head;
  pl.first_col = first_col;
  pl.d = d, pl.e = e, pl.t1 = t1, pl.row = row;
  float* vb = vbs[wave];
  const bool writes = mode.outputs && p == 0 && col < e;
  float stage[PER][W], stage_vb[VB];
  delta_fetch<DP, NT, VECS, W, PER>(tok, pl, t0, stage);
  delta_fetch_values<NT, VW - DELTA_COLS, VB>(tok, pl, t0, lane, stage_vb);
  float ka[R], qa[R], ga[GR], kb[R], qb[R], gb[GR];
  auto read = [&](int j, float (&kk)[R], float (&qq)[R], float (&gg)[GR]) {     // token j of the staged ones
    const float* at = kqg + (j * VECS * DELTA_PARTS + p) * RP;
    if constexpr (HEAD_DECAY) gg[0] = vb[j * VW + DELTA_COLS + 1];
#pragma unroll
    for (int r = 0; r < R; r += 4) {
      const float4 k4 = *reinterpret_cast<const float4*>(at + r);
      const float4 q4 = *reinterpret_cast<const float4*>(at + DELTA_PARTS * RP + r);
      kk[r] = k4.x, kk[r + 1] = k4.y, kk[r + 2] = k4.z, kk[r + 3] = k4.w;
      qq[r] = q4.x, qq[r + 1] = q4.y, qq[r + 2] = q4.z, qq[r + 3] = q4.w;
      if constexpr (!HEAD_DECAY) {
        const float4 g4 = *reinterpret_cast<const float4*>(at + 2 * DELTA_PARTS * RP + r);
        gg[r] = g4.x, gg[r + 1] = g4.y, gg[r + 2] = g4.z, gg[r + 3] = g4.w;
      }
    }
  };
  for (int tb = t0; tb < t1; tb += NT) {
    __syncthreads();          // every wave is done with the tokens staged before
#pragma unroll
    for (int x = 0; x < PER; ++x) {                  // [token][which][row] as fetched
      const int idx = (x * DELTA_THREADS + static_cast<int>(threadIdx.x)) * W;
      const int vec = idx / DP, i = idx % DP;
      float* to = kqg + (vec * DELTA_PARTS + i / R) * RP + i % R;
      if constexpr (W == 4) {
        *reinterpret_cast<float4*>(to) = make_float4(stage[x][0], stage[x][1], stage[x][2], stage[x][3]);
      } else {
        *to = stage[x][0];
      }
    }
#pragma unroll
    for (int j = 0; j < VB; ++j) {
      const int idx = j * TIE_WAVE + lane;
      if (idx < NT * VW) vb[idx] = stage_vb[j];
    }
    __syncthreads();
    if (tb + NT < t1) {
      delta_fetch<DP, NT, VECS, W, PER>(tok, pl, tb + NT, stage);
      delta_fetch_values<NT, VW - DELTA_COLS, VB>(tok, pl, tb + NT, lane, stage_vb);
    }
    const int count = min(NT, t1 - tb);
    float* o = out + static_cast<size_t>(tb) * out_row + head * e + col;
    if constexpr (R > 16) {   // too many rows a lane for two tokens' words in registers
      for (int j = 0; j < count; ++j) {
        read(j, ka, qa, ga);
        const float sum = delta_token<R, GR>(S, ka, qa, ga, vb[j * VW + c], vb[j * VW + DELTA_COLS]);
        if (writes) o[static_cast<size_t>(j) * out_row] = sum;
      }
      continue;
    }
    read(0, ka, qa, ga);
    for (int j = 0; j < count; j += 2) {
      if (j + 1 < count) read(j + 1, kb, qb, gb);
      const float first = delta_token<R, GR>(S, ka, qa, ga, vb[j * VW + c], vb[j * VW + DELTA_COLS]);
      if (writes) o[static_cast<size_t>(j) * out_row] = first;
      if (j + 1 < count) {
        if (j + 2 < count) read(j + 2, ka, qa, ga);
        const float second = delta_token<R, GR>(S, kb, qb, gb, vb[(j + 1) * VW + c], vb[(j + 1) * VW + DELTA_COLS]);
        if (writes) o[static_cast<size_t>(j + 1) * out_row] = second;
      }
    }
  }
  if (!mode.store) return;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int i = p * R + r;
    if (live && i < d) sp[static_cast<size_t>(i) * columns] = S[r];
  }
}

// The chunks' states in order: `ends` [count][H][d][e + d] holds what every chunk makes of a zero state (columns
// below e) and its transition P (columns from e on). A workgroup owns COMBINE_COLS columns of a (sequence, head):
// it leaves every chunk the state before its first token (`starts` [count][H][d][e]) and the slot the state behind
// the last one, S <- P S + L chunk after chunk. A thread has a row (two where d > 128) and four columns; the state
// lies in LDS, and P passes through LDS `jt` columns at a time (rows jt + 1 words apart: the rows of a wave meet
// different banks), the next tile on its way into registers meanwhile.
#define COMBINE_COLS 8
#define COMBINE_THREADS 256
#define COMBINE_TILE 8192          // elements of P in LDS at a time
#define COMBINE_PER (COMBINE_TILE / COMBINE_THREADS)

__global__ __launch_bounds__(COMBINE_THREADS) void gated_delta_combine_kernel(
    const float* __restrict__ ends, float* __restrict__ starts, float* __restrict__ state,
    const int* __restrict__ first_chunk, const int* __restrict__ state_slots, int H, int d, int e, int jt) {
  extern __shared__ __attribute__((aligned(16))) float sl[];       // [2][d][COMBINE_COLS], then P's tile [d][jt + 1]
  const int s = blockIdx.x / H, head = blockIdx.x % H;
  const int c0 = first_chunk[s], c1 = first_chunk[s + 1];
  if (c0 >= c1) return;
  const int col0 = blockIdx.y * COMBINE_COLS;
  const int half = threadIdx.x & 1, col = col0 + half * 4;          // this thread's four columns
  const int row0 = threadIdx.x >> 1;                                // its rows: row0, row0 + 128
  float* slot = state + (static_cast<size_t>(state_slots[s]) * H + head) * d * e;
  float* cur = sl;
  float* nxt = sl + d * COMBINE_COLS;
  float* pl = sl + 2 * d * COMBINE_COLS;
  for (int i = row0; i < d; i += COMBINE_THREADS / 2)
#pragma unroll
    for (int x = 0; x < 4; ++x) cur[i * COMBINE_COLS + half * 4 + x] = col + x < e ? slot[static_cast<size_t>(i) * e + col + x] : 0.f;
  const int wide = e + d;
  const int tiles = (d + jt - 1) / jt;
  float ahead[COMBINE_PER];
  // element k * COMBINE_THREADS + thread of a tile is (row, column) = (i0 + k * rows_step, jj0) where jt divides the
  // threads; otherwise a division an element
  const bool regular = COMBINE_THREADS % jt == 0;
  const int i0 = threadIdx.x / jt, jj0 = threadIdx.x % jt, rows_step = COMBINE_THREADS / jt;
  auto fetch = [&](int c, int tile) {            // tile `tile` of chunk c's P into registers
    const float* P = ends + (static_cast<size_t>(c) * H + head) * d * wide + e + tile * jt;
    const int width = min(jt, d - tile * jt);
#pragma unroll
    for (int k = 0; k < COMBINE_PER; ++k) {
      int i = i0 + k * rows_step, jj = jj0;
      if (!regular) i = (k * COMBINE_THREADS + threadIdx.x) / jt, jj = (k * COMBINE_THREADS + threadIdx.x) % jt;
      ahead[k] = (i < d && jj < width) ? P[static_cast<size_t>(i) * wide + jj] : 0.f;
    }
  };
  fetch(c0, 0);
  float acc[2][4];
  for (int c = c0; c < c1; ++c) {
    const float* E = ends + (static_cast<size_t>(c) * H + head) * d * wide;
    float* st = starts + (static_cast<size_t>(c) * H + head) * d * e;
    for (int tile = 0; tile < tiles; ++tile) {
      __syncthreads();                             // the tile before is used up; `cur` is whole
#pragma unroll
      for (int k = 0; k < COMBINE_PER; ++k) {
        int i = i0 + k * rows_step, jj = jj0;
        if (!regular) i = (k * COMBINE_THREADS + threadIdx.x) / jt, jj = (k * COMBINE_THREADS + threadIdx.x) % jt;
        if (i < d) pl[i * (jt + 1) + jj] = ahead[k];
      }
      __syncthreads();
      if (tile + 1 < tiles) fetch(c, tile + 1);
      else if (c + 1 < c1) fetch(c + 1, 0);
      const int width = min(jt, d - tile * jt);
#pragma unroll
      for (int rr = 0; rr < 2; ++rr) {
        const int i = row0 + rr * (COMBINE_THREADS / 2);
        if (i >= d) continue;
        if (tile == 0) {
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            if (col + x < e) st[static_cast<size_t>(i) * e + col + x] = cur[i * COMBINE_COLS + half * 4 + x];
            acc[rr][x] = col + x < e ? E[static_cast<size_t>(i) * wide + col + x] : 0.f;
          }
        }
        const float* pi = pl + i * (jt + 1);
        const float* sj = cur + tile * jt * COMBINE_COLS + half * 4;
        for (int jj = 0; jj < width; ++jj) {
          const float pij = pi[jj];
          const float4 v = *reinterpret_cast<const float4*>(sj + jj * COMBINE_COLS);
          acc[rr][0] = fmaf(pij, v.x, acc[rr][0]);
          acc[rr][1] = fmaf(pij, v.y, acc[rr][1]);
          acc[rr][2] = fmaf(pij, v.z, acc[rr][2]);
          acc[rr][3] = fmaf(pij, v.w, acc[rr][3]);
        }
        if (tile + 1 == tiles) {
#pragma unroll
          for (int x = 0; x < 4; ++x) nxt[i * COMBINE_COLS + half * 4 + x] = acc[rr][x];
        }
      }
    }
    float* t = cur;
    cur = nxt;
    nxt = t;
  }
  __syncthreads();
  for (int i = row0; i < d; i += COMBINE_THREADS / 2)
#pragma unroll
    for (int x = 0; x < 4; ++x)
      if (col + x < e) slot[static_cast<size_t>(i) * e + col + x] = cur[i * COMBINE_COLS + half * 4 + x];
}

// tok: rows of delta_prepare; out: float32 [T][>= H e]; state: [slots][H][d][e].
static int launch_delta_scan(const float* tok, int row, float* out, int out_row, float* state, const int* query_start,
                             const int* state_slots, int num_items, int G, int H, int d, int e, int head_decay,
                             DeltaScanMode mode, hipStream_t stream) {
  constexpr int wg_cols = DELTA_WAVES * DELTA_COLS;
  const dim3 grid(num_items * H, (mode.columns + wg_cols - 1) / wg_cols);
  if (grid.y > 65535) return TIE_BAD_ARGUMENT;
  // four words a load where every head's k, q and g start at a multiple of four words of an aligned row
  const bool wide = d % 4 == 0 && (H * e) % 4 == 0 && row % 4 == 0 && reinterpret_cast<uintptr_t>(tok) % 16 == 0;
#define SCAN_AS(R, W, HD)                                                                                     \
  gated_delta_scan_kernel<R, W, HD><<<grid, DELTA_THREADS, 0, stream>>>(tok, row, out, out_row, state, query_start, \
                                                                        state_slots, G, H, d, e, mode)
#define SCAN(R)                                          \
  do {                                                   \
    if (wide && head_decay) SCAN_AS(R, 4, true);         \
    else if (wide) SCAN_AS(R, 4, false);                 \
    else if (head_decay) SCAN_AS(R, 1, true);            \
    else SCAN_AS(R, 1, false);                           \
  } while (0)
  if (d <= 32) SCAN(4);
  else if (d <= 64) SCAN(8);
  else if (d <= 128) SCAN(16);
  else SCAN(32);
#undef SCAN
#undef SCAN_AS
  return tie_launch_status();
}

extern "C" int tie_gated_delta_scan(const float* tok, int row, float* out, int out_row, float* state,
                                    const int* query_start, const int* state_slots, int num_seqs, int G, int H, int d,
                                    int e, int head_decay, hipStream_t stream) {
  if (num_seqs <= 0 || G <= 0 || H <= 0 || H % G || d <= 0 || d > 256 || e <= 0 || out_row < H * e ||
      row < 2 * G * d + H * e + H + (head_decay ? H : H * d))
    return TIE_BAD_ARGUMENT;
  return launch_delta_scan(tok, row, out, out_row, state, query_start, state_slots, num_seqs, G, H, d, e, head_decay,
                           DeltaScanMode{nullptr, e, 0, 1, 1}, stream);
}

// The same over chunks, in three launches: every chunk from a zero state with its transition beside it (`ends`
// [count][H][d][e + d]), the chunks' states combined in order (`starts` [count][H][d][e]; the slots receive the
// final states), every chunk again from its true start with outputs. items: [count][3] (sequence, first row, end
// row), in the order of the sequences' rows; first_chunk: [num_seqs + 1].
extern "C" int tie_gated_delta_scan_chunked(const float* tok, int row, float* out, int out_row, float* state,
                                            const int* state_slots, int num_seqs, const int* items,
                                            const int* first_chunk, int count, float* ends, float* starts, int G,
                                            int H, int d, int e, hipStream_t stream) {
  if (num_seqs <= 0 || count <= 0 || G <= 0 || H <= 0 || H % G || d <= 0 || d > 256 || e <= 0 || out_row < H * e ||
      row < 2 * G * d + H * e + H + H * d || !items || !first_chunk || !ends || !starts)
    return TIE_BAD_ARGUMENT;
  int rc = launch_delta_scan(tok, row, out, out_row, ends, nullptr, nullptr, count, G, H, d, e, 0,
                             DeltaScanMode{items, e + d, 1, 1, 0}, stream);
  if (rc != TIE_OK) return rc;
  const dim3 grid(num_seqs * H, (e + COMBINE_COLS - 1) / COMBINE_COLS);
  if (grid.y > 65535) return TIE_BAD_ARGUMENT;
  int jt = COMBINE_TILE / d / 4 * 4;           // d <= 256: at least 32
  if (jt > d) jt = d;
  const size_t lds = (2 * static_cast<size_t>(d) * COMBINE_COLS + static_cast<size_t>(d) * (jt + 1)) * sizeof(float);
  gated_delta_combine_kernel<<<grid, COMBINE_THREADS, lds, stream>>>(ends, starts, state, first_chunk, state_slots, H,
                                                                     d, e, jt);
  rc = tie_launch_status();
  if (rc != TIE_OK) return rc;
  return launch_delta_scan(tok, row, out, out_row, starts, nullptr, nullptr, count, G, H, d, e, 0,
                           DeltaScanMode{items, e, 0, 0, 1}, stream);
}

// ---------------------------------------------------------------- the norm of the heads' outputs, gated
// out = o / rms(o over each group of `group` columns) * w[column in group] * sigmoid(gate) (or * silu(gate)), a wave a
// group; the weights of neighbouring groups lie w_group apart (0: one weight for all groups), w null: all 1.
template <typename TO>
__global__ void grouped_gated_rms_norm_kernel(const float* __restrict__ o, int o_row, const float* __restrict__ w,
                                              int w_group, float eps, const float* __restrict__ gate, int gate_row, int silu_gate,
                                              TO* __restrict__ out, int groups, int group) {
  const int lane = threadIdx.x & (TIE_WAVE - 1);
  const int g = blockIdx.y * (blockDim.x / TIE_WAVE) + threadIdx.x / TIE_WAVE;
  if (g >= groups) return;
  const size_t t = blockIdx.x;
  const float* r = o + t * o_row + static_cast<size_t>(g) * group;
  const float* gt = gate + t * gate_row + static_cast<size_t>(g) * group;
  float ss = 0.f;
  for (int c = lane; c < group; c += TIE_WAVE) ss = fmaf(r[c], r[c], ss);
  const float inv = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(group) + eps);
  TO* d = out + (t * groups + g) * group;
  for (int c = lane; c < group; c += TIE_WAVE)
    store_from_float(d + c, (r[c] * inv) * (w ? w[static_cast<size_t>(g) * w_group + c] : 1.f) * (silu_gate ? silu_f(gt[c]) : sigmoid_f(gt[c])));
}

// The same for groups of up to 4 LANES columns in whole aligned pieces of four: LANES lanes a group, four columns a lane, the
// groups of all rows one behind the other.
template <typename TO, int LANES>
__global__ __launch_bounds__(256) void grouped_gated_rms_norm_piece_kernel(
    const float* __restrict__ o, int o_row, const float* __restrict__ w, int w_group, float eps,
    const float* __restrict__ gate, int gate_row, int silu_gate, TO* __restrict__ out, int groups, int group, long total) {
  const long at = static_cast<long>(blockIdx.x) * (256 / LANES) + threadIdx.x / LANES;
  const int c = (threadIdx.x % LANES) * 4;
  const bool in = at < total && c < group;
  const long t = in ? at / groups : 0;
  const int g = in ? static_cast<int>(at - t * groups) : 0;
  float4 v = make_float4(0.f, 0.f, 0.f, 0.f), z = v, s = make_float4(1.f, 1.f, 1.f, 1.f);
  if (in) {
    v = *reinterpret_cast<const float4*>(o + t * o_row + static_cast<size_t>(g) * group + c);
    z = *reinterpret_cast<const float4*>(gate + t * gate_row + static_cast<size_t>(g) * group + c);
    if (w) s = *reinterpret_cast<const float4*>(w + static_cast<size_t>(g) * w_group + c);
  }
  float ss = (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
#pragma unroll
  for (int off = LANES / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, TIE_WAVE);
  if (!in) return;
  const float inv = 1.0f / sqrtf(ss / static_cast<float>(group) + eps);
  auto act = [&](float x) { return silu_gate ? silu_f(x) : sigmoid_f(x); };
  const float r0 = (v.x * inv) * s.x * act(z.x), r1 = (v.y * inv) * s.y * act(z.y);
  const float r2 = (v.z * inv) * s.z * act(z.z), r3 = (v.w * inv) * s.w * act(z.w);
  TO* d = out + (t * groups + g) * group + c;
  if constexpr (sizeof(TO) == 2)
    *reinterpret_cast<uint2*>(d) = make_uint2(pack_bf16x2(r0, r1), pack_bf16x2(r2, r3));
  else
    *reinterpret_cast<float4*>(d) = make_float4(r0, r1, r2, r3);
}

extern "C" int tie_grouped_gated_rms_norm(const float* o, int o_row, const float* w, int w_group, float eps, const float* gate,
                                          int gate_row, int silu_gate, void* out, int out_dtype, int T, int groups,
                                          int group, hipStream_t stream) {
  if (T <= 0 || groups <= 0 || group <= 0 || o_row < groups * group || gate_row < groups * group)
    return TIE_BAD_ARGUMENT;
  if (group % 4 == 0 && group <= 256 && o_row % 4 == 0 && gate_row % 4 == 0 && w_group % 4 == 0 &&
      (out_dtype == TIE_F32 || out_dtype == TIE_BF16) &&
      (reinterpret_cast<uintptr_t>(o) | reinterpret_cast<uintptr_t>(w) | reinterpret_cast<uintptr_t>(gate) |
       reinterpret_cast<uintptr_t>(out)) % 16 == 0) {
    const long total = static_cast<long>(T) * groups;
#define PIECE(TO, LANES)                                                                                              \
  grouped_gated_rms_norm_piece_kernel<TO, LANES>                                                                      \
      <<<static_cast<unsigned>((total + 256 / LANES - 1) / (256 / LANES)), 256, 0, stream>>>(                         \
          o, o_row, w, w_group, eps, gate, gate_row, silu_gate, static_cast<TO*>(out), groups, group, total)
#define PIECES(LANES)                              \
  {                                                \
    if (out_dtype == TIE_F32) PIECE(float, LANES); \
    else PIECE(bf16_t, LANES);                     \
  }
    if (group <= 32) PIECES(8)
    else if (group <= 64) PIECES(16)
    else if (group <= 128) PIECES(32)
    else PIECES(64)
#undef PIECES
#undef PIECE
    return tie_launch_status();
  }
  const int waves = groups >= 4 ? 4 : groups;
  const dim3 grid(T, (groups + waves - 1) / waves);
  if (out_dtype == TIE_F32)
    grouped_gated_rms_norm_kernel<float><<<grid, waves * TIE_WAVE, 0, stream>>>(
        o, o_row, w, w_group, eps, gate, gate_row, silu_gate, static_cast<float*>(out), groups, group);
  else if (out_dtype == TIE_BF16)
    grouped_gated_rms_norm_kernel<bf16_t><<<grid, waves * TIE_WAVE, 0, stream>>>(
        o, o_row, w, w_group, eps, gate, gate_row, silu_gate, static_cast<bf16_t*>(out), groups, group);
  else
    return TIE_BAD_ARGUMENT;
  return tie_launch_status();
}
