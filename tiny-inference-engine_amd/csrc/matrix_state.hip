// Mixers whose memory is one matrix a head, S [d][e] in float32, that takes in an outer product a token:
//
//   decay    S_t = decay_h S_(t-1) + k_t v_t^T                                   o_t = S_t^T q_t
//   memory   gates from the token:  i = cap tanh((z_i + b_i) / cap),   f = log sigmoid(cap tanh((z_f + b_f) / cap))
//            m_t = max(f + m_(t-1), i),   keep = exp(f + m_(t-1) - m_t),   take = exp(i - m_t)
//            S_t = keep S_(t-1) + take k_t v_t^T,    n_t = keep n_(t-1) + take k_t
//            o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)
//
// q may be scaled, and q, k, v may pass SiLU; in `decay` q and k may be rotated by position (the walk does it itself,
// long portions are rotated by rotate_heads beforehand). States live in slots, state[slot][H][d][e]; `memory` also keeps
// [slot][H][blocks][d + 1] = (n, m), one copy for each block of WALK_COLS value columns, because the workgroups of a head
// own a block of columns each and none may read what another one writes. All of it starts as zeros.
//
// A sequence's tokens are a dependent chain. Steps of single tokens and short portions walk it (state_walk_kernel): a
// workgroup holds d x 32 of the state in registers and moves down the tokens. A long portion is cut into chunks of up to 64
// rows (items = (sequence, first row, one past the last row), in the order of the rows), and three launches run all chunks
// side by side as float32 matrix products (v_mfma_f32_32x32x2_f32: operands and sums in 32 bits throughout):
//   1. chunk_state      L = K'^T V, what a chunk ends with when it starts from zero; row j of K' is k_j times what is left of
//                       token j at the chunk's end
//   2. combine_chunks   the chunks of a sequence in order: S <- keep S + take L; a chunk's L is replaced by the state it
//                       starts from, the slot receives the last one
//   3. chunk_output     O = diag(r) Q S + ((Q K^T) (.) D) V,  r_i what is left of the starting state at token i, D_ij what is
//                       left there of token j <= i; `memory` divides by the same sums over n
// In `memory` with b the running sum of f inside a chunk, a_j = i_j - b_j and M_i = max(m_start, a_1 .. a_i): m_i = b_i + M_i,
// r_i = exp(m_start - M_i), D_ij = exp(a_j - M_i). No factor exceeds 1. b, a and M are kept in double: they grow with the
// chunk, and only their small differences count.
#include "common.h"

#include <math.h>

#define KIND_DECAY 0
#define KIND_MEMORY 1

#define WALK_COLS 32       // value columns of a workgroup of the walk
#define WALK_TOKENS 8      // tokens staged at a time
#define STATE_MAX_D 512
#define CHUNK_ROWS 64

struct StateInputs {
  const float* proj;                // float32 sums of the projections, rows `row` apart
  int row;
  int q_col, k_col, v_col;          // head h: columns + h d, + h d, + h e
  int activation;                   // 1: SiLU on q, k and v
  float q_scale;
  const float* angles;              // walk: [T][rot] = cos | sin of the rot / 2 angles of a row (or null)
  int rot;
  int H, d, e;
};

struct StateFactors {
  const float* decay;               // decay: [H]
  const float *i_bias, *f_bias;     // memory: [H] each; z_i and z_f are columns i_col + h, f_col + h of a row
  int i_col, f_col;
  float cap;
};

__device__ __forceinline__ float state_silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float gate_in(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float gate_forget(float z, float cap) {
  const float x = cap * tanhf(z / cap);
  return fminf(x, 0.f) - log1pf(expf(-fabsf(x)));                     // log sigmoid(x)
}

// ------------------------------------------------------------------ the walk
// A workgroup owns the 32 value columns block * 32 .. of one (sequence, head). Thread = 4 columns (tid % 8) x the rows
// i * 32 + tid / 8 of the state, i < RPT: eight lanes read 128 consecutive bytes of a row. A token costs a thread 8 RPT
// multiply-adds; the partial outputs of the 32 row groups meet by shuffles inside a wave and through LDS across the four.
template <int KIND, int RPT>
__global__ __launch_bounds__(256) void state_walk_kernel(StateInputs in, StateFactors fa, float* __restrict__ out,
                                                         float* __restrict__ state, float* __restrict__ norm_state,
                                                         const int* __restrict__ query_start,
                                                         const int* __restrict__ state_slots) {
  constexpr int MAXD = 32 * RPT;
  constexpr int ROW = 2 * MAXD + WALK_COLS;
  constexpr int REGS = (WALK_TOKENS * ROW + 255) / 256;
  __shared__ __attribute__((aligned(16))) float kqv_s[WALK_TOKENS][ROW];
  __shared__ __attribute__((aligned(16))) float o_s[WALK_TOKENS][4][WALK_COLS];
  __shared__ float nq_s[WALK_TOKENS][4], gate_s[WALK_TOKENS][2], floor_s[WALK_TOKENS];
  const int tid = threadIdx.x, wave = tid / TIE_WAVE, lane = tid & (TIE_WAVE - 1);
  const int quad = tid & 7, group = tid >> 3;
  const int block = blockIdx.x, h = blockIdx.y, s = blockIdx.z;
  const int H = in.H, d = in.d, e = in.e;
  const int first = block * WALK_COLS, col = first + quad * 4;
  const size_t slot = state_slots[s];
  float* S = state + (slot * H + h) * d * e;
  float* nm = KIND == KIND_MEMORY ? norm_state + ((slot * H + h) * gridDim.x + block) * (d + 1) : nullptr;
  const bool whole = (e & 3) == 0;                      // four columns of a row are one aligned piece (or none at all)
  float st[RPT][4], nst[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = i * 32 + group;
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (r < d && col < e) {
      const float* p = S + static_cast<size_t>(r) * e + col;
      if (whole) {
        v = *reinterpret_cast<const float4*>(p);
      } else {
        v.x = p[0];
        if (col + 1 < e) v.y = p[1];
        if (col + 2 < e) v.z = p[2];
        if (col + 3 < e) v.w = p[3];
      }
    }
    st[i][0] = v.x, st[i][1] = v.y, st[i][2] = v.z, st[i][3] = v.w;
    nst[i] = (KIND == KIND_MEMORY && r < d) ? nm[r] : 0.f;
  }
  float m = KIND == KIND_MEMORY ? nm[d] : 0.f;
  const float lam = KIND == KIND_DECAY ? fa.decay[h] : 0.f;

  const int t0 = query_start[s], t1 = query_start[s + 1];
  float regs[REGS], gate_reg = 0.f;
  auto fetch = [&](int tb) {
    const int count = min(WALK_TOKENS, t1 - tb);
#pragma unroll
    for (int r = 0; r < REGS; ++r) {
      const int idx = tid + r * 256;
      const int tok = idx / ROW, j = idx % ROW;
      const float* p = in.proj + static_cast<size_t>(tb + tok) * in.row;
      regs[r] = 0.f;
      if (tok < count) {
        if (j < MAXD) {
          if (j < d) regs[r] = p[in.k_col + h * d + j];
        } else if (j < 2 * MAXD) {
          if (j - MAXD < d) regs[r] = p[in.q_col + h * d + j - MAXD];
        } else if (first + j - 2 * MAXD < e) {
          regs[r] = p[in.v_col + h * e + first + j - 2 * MAXD];
        }
      }
    }
    if (KIND == KIND_MEMORY && tid < 2 * count)
      gate_reg = in.proj[static_cast<size_t>(tb + (tid >> 1)) * in.row + ((tid & 1) ? fa.f_col : fa.i_col) + h];
  };
  auto publish = [&](int count) {
#pragma unroll
    for (int r = 0; r < REGS; ++r) {
      const int idx = tid + r * 256;
      const int tok = idx / ROW, j = idx % ROW;
      if (tok < count) {
        float v = in.activation ? state_silu(regs[r]) : regs[r];
        if (j >= MAXD && j < 2 * MAXD) v *= in.q_scale;
        kqv_s[tok][j] = v;
      }
    }
    if (KIND == KIND_MEMORY && tid < 2 * count)
      gate_s[tid >> 1][tid & 1] = (tid & 1) ? gate_forget(gate_reg + fa.f_bias[h], fa.cap)
                                            : gate_in(gate_reg + fa.i_bias[h], fa.cap);
  };
  if (t0 < t1) fetch(t0);
  for (int tb = t0; tb < t1; tb += WALK_TOKENS) {       // uniform for the workgroup
    const int count = min(WALK_TOKENS, t1 - tb);
    publish(count);
    __syncthreads();
    if (tb + WALK_TOKENS < t1) fetch(tb + WALK_TOKENS); // in flight during the arithmetic below
    if (KIND == KIND_DECAY && in.angles != nullptr) {   // pairs (i, i + rot / 2) of k, then of q
      const int half = in.rot / 2;
      for (int p = tid; p < count * in.rot; p += 256) {
        const int tok = p / in.rot, j = p - tok * in.rot;
        const int i = j < half ? j : j - half;
        const float* a = in.angles + static_cast<size_t>(tb + tok) * in.rot;
        float* at = &kqv_s[tok][(j < half ? 0 : MAXD) + i];
        const float u = at[0], v = at[half], cs = a[i], sn = a[half + i];
        at[0] = u * cs - v * sn;
        at[half] = v * cs + u * sn;
      }
      __syncthreads();
    }
    for (int tok = 0; tok < count; ++tok) {
      float keep = lam, take = 1.f;
      if (KIND == KIND_MEMORY) {
        const float li = gate_s[tok][0], lf = gate_s[tok][1] + m;
        m = fmaxf(lf, li);
        keep = expf(lf - m);
        take = expf(li - m);
      }
      const float4 v4 = *reinterpret_cast<const float4*>(&kqv_s[tok][2 * MAXD + quad * 4]);
      const float v[4] = {take * v4.x, take * v4.y, take * v4.z, take * v4.w};
      float o[4] = {0.f, 0.f, 0.f, 0.f}, nq = 0.f;
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        const float k = kqv_s[tok][i * 32 + group], q = kqv_s[tok][MAXD + i * 32 + group];
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          st[i][c] = fmaf(keep, st[i][c], k * v[c]);
          o[c] = fmaf(st[i][c], q, o[c]);
        }
        if (KIND == KIND_MEMORY) {
          nst[i] = fmaf(keep, nst[i], take * k);
          nq = fmaf(nst[i], q, nq);
        }
      }
#pragma unroll
      for (int off = 8; off < TIE_WAVE; off *= 2) {
#pragma unroll
        for (int c = 0; c < 4; ++c) o[c] += __shfl_xor(o[c], off, TIE_WAVE);
        if (KIND == KIND_MEMORY) nq += __shfl_xor(nq, off, TIE_WAVE);
      }
      if (lane < 8) *reinterpret_cast<float4*>(&o_s[tok][wave][quad * 4]) = make_float4(o[0], o[1], o[2], o[3]);
      if (KIND == KIND_MEMORY) {
        if (lane == 0) nq_s[tok][wave] = nq;
        if (tid == 0) floor_s[tok] = expf(-m);
      }
    }
    __syncthreads();
    for (int j = tid; j < count * WALK_COLS; j += 256) {
      const int tok = j / WALK_COLS, c = j % WALK_COLS;
      if (first + c >= e) continue;
      float v = ((o_s[tok][0][c] + o_s[tok][1][c]) + o_s[tok][2][c]) + o_s[tok][3][c];
      if (KIND == KIND_MEMORY) {
        const float nq = ((nq_s[tok][0] + nq_s[tok][1]) + nq_s[tok][2]) + nq_s[tok][3];
        v /= fmaxf(fabsf(nq), floor_s[tok]) + 1e-6f;
      }
      out[(static_cast<size_t>(tb + tok) * H + h) * e + first + c] = v;
    }
    // what was read here is overwritten behind the barrier of the next round's publish at the earliest: kqv_s is not
    // read after the barrier above, and o_s, nq_s, floor_s are written again only behind the next one
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = i * 32 + group;
    if (r < d && col < e) {
      float* p = S + static_cast<size_t>(r) * e + col;
      if (whole) {
        *reinterpret_cast<float4*>(p) = make_float4(st[i][0], st[i][1], st[i][2], st[i][3]);
      } else {
        p[0] = st[i][0];
        if (col + 1 < e) p[1] = st[i][1];
        if (col + 2 < e) p[2] = st[i][2];
        if (col + 3 < e) p[3] = st[i][3];
      }
    }
    if (KIND == KIND_MEMORY && quad == 0 && r < d) nm[r] = nst[i];
  }
  if (KIND == KIND_MEMORY && tid == 0) nm[d] = m;
}

// One token a sequence (decode steps): the same layout, keys, queries and values straight from memory into the threads that
// need them, everything asked for before the first use, one barrier.
template <int KIND, int RPT>
__global__ __launch_bounds__(256) void state_step_kernel(StateInputs in, StateFactors fa, float* __restrict__ out,
                                                         float* __restrict__ state, float* __restrict__ norm_state,
                                                         const int* __restrict__ query_start,
                                                         const int* __restrict__ state_slots) {
  __shared__ __attribute__((aligned(16))) float o_s[4][WALK_COLS];
  __shared__ float nq_s[4];
  const int tid = threadIdx.x, wave = tid / TIE_WAVE, lane = tid & (TIE_WAVE - 1);
  const int quad = tid & 7, group = tid >> 3;
  const int block = blockIdx.x, h = blockIdx.y, s = blockIdx.z;
  const int H = in.H, d = in.d, e = in.e;
  const int first = block * WALK_COLS, col = first + quad * 4;
  const size_t slot = state_slots[s];
  const size_t t = query_start[s];
  float* S = state + (slot * H + h) * d * e;
  float* nm = KIND == KIND_MEMORY ? norm_state + ((slot * H + h) * gridDim.x + block) * (d + 1) : nullptr;
  const float* p = in.proj + t * in.row;
  const bool whole = (e & 3) == 0;
  float st[RPT][4], nst[RPT], k[RPT], q[RPT], v[4];
  float m = 0.f, zi = 0.f, zf = 0.f;
  if (KIND == KIND_MEMORY) {
    m = nm[d];
    zi = p[fa.i_col + h] + fa.i_bias[h];
    zf = p[fa.f_col + h] + fa.f_bias[h];
  }
#pragma unroll
  for (int c = 0; c < 4; ++c) v[c] = col + c < e ? p[in.v_col + h * e + col + c] : 0.f;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = i * 32 + group;
    const bool has = r < d;
    k[i] = has ? p[in.k_col + h * d + r] : 0.f;
    q[i] = has ? p[in.q_col + h * d + r] : 0.f;
    nst[i] = (KIND == KIND_MEMORY && has) ? nm[r] : 0.f;
    float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
    if (has && col < e) {
      const float* at = S + static_cast<size_t>(r) * e + col;
      if (whole) {
        x = *reinterpret_cast<const float4*>(at);
      } else {
        x.x = at[0];
        if (col + 1 < e) x.y = at[1];
        if (col + 2 < e) x.z = at[2];
        if (col + 3 < e) x.w = at[3];
      }
    }
    st[i][0] = x.x, st[i][1] = x.y, st[i][2] = x.z, st[i][3] = x.w;
  }
  if (KIND == KIND_DECAY && in.angles != nullptr) {     // dimension r turns with r + rot / 2 (or r - rot / 2)
    const int half = in.rot / 2;
    const float* a = in.angles + t * in.rot;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int r = i * 32 + group;
      if (r >= in.rot) continue;
      const bool low = r < half;
      const int other = low ? r + half : r - half, pair = low ? r : r - half;
      const float cs = a[pair], sn = low ? -a[half + pair] : a[half + pair];
      k[i] = k[i] * cs + p[in.k_col + h * d + other] * sn;
      q[i] = q[i] * cs + p[in.q_col + h * d + other] * sn;
    }
  }
  if (in.activation) {
#pragma unroll
    for (int c = 0; c < 4; ++c) v[c] = state_silu(v[c]);
#pragma unroll
    for (int i = 0; i < RPT; ++i) k[i] = state_silu(k[i]), q[i] = state_silu(q[i]);
  }
  float keep = 1.f, take = 1.f;
  if (KIND == KIND_MEMORY) {
    const float li = gate_in(zi, fa.cap), lf = gate_forget(zf, fa.cap) + m;
    m = fmaxf(lf, li);
    keep = expf(lf - m);
    take = expf(li - m);
#pragma unroll
    for (int c = 0; c < 4; ++c) v[c] *= take;
  } else {
    keep = fa.decay[h];
  }
  float o[4] = {0.f, 0.f, 0.f, 0.f}, nq = 0.f;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const float qs = q[i] * in.q_scale;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      st[i][c] = fmaf(keep, st[i][c], k[i] * v[c]);
      o[c] = fmaf(st[i][c], qs, o[c]);
    }
    if (KIND == KIND_MEMORY) {
      nst[i] = fmaf(keep, nst[i], take * k[i]);
      nq = fmaf(nst[i], qs, nq);
    }
  }
#pragma unroll
  for (int off = 8; off < TIE_WAVE; off *= 2) {
#pragma unroll
    for (int c = 0; c < 4; ++c) o[c] += __shfl_xor(o[c], off, TIE_WAVE);
    if (KIND == KIND_MEMORY) nq += __shfl_xor(nq, off, TIE_WAVE);
  }
  if (lane < 8) *reinterpret_cast<float4*>(&o_s[wave][quad * 4]) = make_float4(o[0], o[1], o[2], o[3]);
  if (KIND == KIND_MEMORY && lane == 0) nq_s[wave] = nq;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = i * 32 + group;
    if (r < d && col < e) {
      float* at = S + static_cast<size_t>(r) * e + col;
      if (whole) {
        *reinterpret_cast<float4*>(at) = make_float4(st[i][0], st[i][1], st[i][2], st[i][3]);
      } else {
        at[0] = st[i][0];
        if (col + 1 < e) at[1] = st[i][1];
        if (col + 2 < e) at[2] = st[i][2];
        if (col + 3 < e) at[3] = st[i][3];
      }
    }
    if (KIND == KIND_MEMORY && quad == 0 && r < d) nm[r] = nst[i];
  }
  __syncthreads();                                      // every thread has read nm[d] by now
  if (tid < WALK_COLS && first + tid < e) {
    float x = ((o_s[0][tid] + o_s[1][tid]) + o_s[2][tid]) + o_s[3][tid];
    if (KIND == KIND_MEMORY) x /= fmaxf(fabsf(((nq_s[0] + nq_s[1]) + nq_s[2]) + nq_s[3]), expf(-m)) + 1e-6f;
    out[(t * H + h) * e + first + tid] = x;
  }
  if (KIND == KIND_MEMORY && tid == 0) nm[d] = m;
}

// ------------------------------------------------------------------ chunks
typedef float state_f16_t __attribute__((ext_vector_type(16)));

struct ChunkPlan {
  const int* items;                 // [count][3]
  const int* first_item;            // [S + 1]
  float* states;                    // [count][heads][per]: d e values of S, then (memory) d of n
  double* sums;                     // memory: [count][heads][2] = (b at the chunk's end, max of a)
  float* starts;                    // memory: [count][heads] = m where the chunk starts
  int h_first, heads, per;          // the heads of this pass
};

__device__ __forceinline__ double shfl_up_d(double v, int off) {
  int2 w = *reinterpret_cast<int2*>(&v);
  w.x = __shfl_up(w.x, off, TIE_WAVE);
  w.y = __shfl_up(w.y, off, TIE_WAVE);
  return *reinterpret_cast<double*>(&w);
}
__device__ __forceinline__ double shfl_d(double v, int from) {
  int2 w = *reinterpret_cast<int2*>(&v);
  w.x = __shfl(w.x, from, TIE_WAVE);
  w.y = __shfl(w.y, from, TIE_WAVE);
  return *reinterpret_cast<double*>(&w);
}
__device__ __forceinline__ double wave_running_sum(double v, int lane) {
#pragma unroll
  for (int off = 1; off < TIE_WAVE; off *= 2) {
    const double up = shfl_up_d(v, off);
    if (lane >= off) v += up;
  }
  return v;
}
__device__ __forceinline__ double wave_running_max(double v, int lane) {
#pragma unroll
  for (int off = 1; off < TIE_WAVE; off *= 2) {
    const double up = shfl_up_d(v, off);
    if (lane >= off) v = fmax(v, up);
  }
  return v;
}

// One wave, a lane a token of the chunk t0 .. t0 + n - 1: b (running sum of f) and a = i - b; beyond the chunk f = 0, a = -inf.
__device__ __forceinline__ void chunk_gates(const StateInputs& in, const StateFactors& fa, int h, int t0, int n, int lane,
                                            double& b, double& a) {
  float li = 0.f, lf = 0.f;
  if (lane < n) {
    const float* p = in.proj + static_cast<size_t>(t0 + lane) * in.row;
    li = gate_in(p[fa.i_col + h] + fa.i_bias[h], fa.cap);
    lf = gate_forget(p[fa.f_col + h] + fa.f_bias[h], fa.cap);
  }
  b = wave_running_sum(static_cast<double>(lf), lane);
  a = lane < n ? static_cast<double>(li) - b : -INFINITY;
}

__device__ __forceinline__ float decay_power(float log2_lam, int m) {   // m = 0 apart: a decay of zero gives 1, then 0
  return m > 0 ? exp2f(static_cast<float>(m) * log2_lam) : 1.f;
}

__device__ __forceinline__ float4 f4_map(float4 v, bool silu, float scale) {
  if (silu) v = make_float4(state_silu(v.x), state_silu(v.y), state_silu(v.z), state_silu(v.w));
  return make_float4(v.x * scale, v.y * scale, v.z * scale, v.w * scale);
}

// Four columns c .. c + 3 of a row of n values: one 16-byte load where rows are made of whole aligned pieces (WHOLE).
template <bool WHOLE>
__device__ __forceinline__ float4 load_piece(const float* row, int c, int n, bool in) {
  float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
  if (!in || c >= n) return v;
  if (WHOLE) return *reinterpret_cast<const float4*>(row + c);
  v.x = row[c];
  if (c + 1 < n) v.y = row[c + 1];
  if (c + 2 < n) v.z = row[c + 2];
  if (c + 3 < n) v.w = row[c + 3];
  return v;
}

// Launch 1. A workgroup owns 128 rows x 128 columns of one (chunk, head): 32 tokens of keys and values at a time in LDS, wave
// w the rows 32 w .. of four tiles of 32 columns, two tokens an instruction (lane l hands over token l / 32). The
// accumulators hold, in lane l, column l % 32 and the rows 8 (r / 4) + 4 (l / 32) + r % 4 of register r.
template <int KIND, bool WHOLE>
__global__ __launch_bounds__(256) void chunk_state_kernel(StateInputs in, StateFactors fa, ChunkPlan plan,
                                                          const float* __restrict__ norm_state,
                                                          const int* __restrict__ state_slots, int blocks_e, int copies) {
  __shared__ __attribute__((aligned(16))) float k_s[32][128];
  __shared__ __attribute__((aligned(16))) float v_s[32][128];
  __shared__ float weight_s[CHUNK_ROWS];
  const int tid = threadIdx.x, wave = tid / TIE_WAVE, lane = tid & (TIE_WAVE - 1);
  const int hl = blockIdx.y, h = plan.h_first + hl, item = blockIdx.z;
  const int d = in.d, e = in.e;
  const int d_first = (blockIdx.x / blocks_e) * 128, e_first = (blockIdx.x % blocks_e) * 128;
  const int t0 = plan.items[item * 3 + 1], n = plan.items[item * 3 + 2] - t0;
  const float* kp = in.proj + static_cast<size_t>(t0) * in.row + in.k_col + h * d;
  const float* vp = in.proj + static_cast<size_t>(t0) * in.row + in.v_col + h * e;
  float4 kr[4], vr[4];
  const int i4 = (tid & 31) * 4;                         // the four columns a thread stages, of the tokens tid / 32 + 8 u
  auto fetch = [&](int from) {
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int j = from + (tid >> 5) + 8 * u;
      const size_t at = static_cast<size_t>(min(j, n - 1)) * in.row;
      kr[u] = load_piece<WHOLE>(kp + at, d_first + i4, d, j < n);
      vr[u] = load_piece<WHOLE>(vp + at, e_first + i4, e, j < n);
    }
  };
  fetch(0);
  if (wave == 0) {
    if (KIND == KIND_MEMORY) {
      double b, a;
      chunk_gates(in, fa, h, t0, n, lane, b, a);
      const double top = shfl_d(wave_running_max(a, lane), TIE_WAVE - 1), b_end = shfl_d(b, TIE_WAVE - 1);
      weight_s[lane] = lane < n ? expf(static_cast<float>(a - top)) : 0.f;
      if (blockIdx.x == 0 && lane == 0) {
        const size_t at = static_cast<size_t>(item) * plan.heads + hl;
        plan.sums[2 * at] = b_end;
        plan.sums[2 * at + 1] = top;
        const int s = plan.items[item * 3];
        if (item == plan.first_item[s])
          plan.starts[at] = norm_state[(static_cast<size_t>(state_slots[s]) * in.H + h) * copies * (d + 1) + d];
      }
    } else {
      weight_s[lane] = lane < n ? decay_power(log2f(fa.decay[h]), n - 1 - lane) : 0.f;
    }
  }
  __syncthreads();
  state_f16_t acc[4];
#pragma unroll
  for (int c = 0; c < 4; ++c)
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[c][r] = 0.f;
  const int half = lane >> 5, l32 = lane & 31;
  const bool sums_n = KIND == KIND_MEMORY && e_first == 0 && tid < 128;
  float n_sum = 0.f;
  for (int from = 0; from < n; from += 32) {            // uniform for the workgroup
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int j = (tid >> 5) + 8 * u;
      *reinterpret_cast<float4*>(&k_s[j][i4]) = f4_map(kr[u], in.activation, weight_s[from + j]);
      *reinterpret_cast<float4*>(&v_s[j][i4]) = f4_map(vr[u], in.activation, 1.f);
    }
    __syncthreads();
    if (from + 32 < n) fetch(from + 32);                // in flight during the products
    const int steps = (min(32, n - from) + 1) / 2;       // a token beyond the chunk is a row of zeros
    for (int st = 0; st < steps; ++st) {
      const int j = 2 * st + half;
      const float a = k_s[j][wave * 32 + l32];
#pragma unroll
      for (int c = 0; c < 4; ++c)
        acc[c] = __builtin_amdgcn_mfma_f32_32x32x2f32(a, v_s[j][c * 32 + l32], acc[c], 0, 0, 0);
    }
    if (sums_n)
      for (int j = 0; j < 32; ++j) n_sum += k_s[j][tid];
    __syncthreads();
  }
  float* L = plan.states + (static_cast<size_t>(item) * plan.heads + hl) * plan.per;
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    const int col = e_first + c * 32 + l32;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int rw = d_first + wave * 32 + 8 * (r / 4) + 4 * half + (r % 4);
      if (rw < d && col < e) L[static_cast<size_t>(rw) * e + col] = acc[c][r];
    }
  }
  if (sums_n && d_first + tid < d) L[static_cast<size_t>(d) * e + d_first + tid] = n_sum;
}

// Launch 2. One thread a value of (S, n) of a head; the factors of 64 chunks at a time are formed by one wave. In `memory`,
// with B the sum of the chunks' b before chunk c and u_c = max a_c - B_c: m where c starts = B_c + G_c, G_c the largest of
// the sequence's m and the u of the chunks before, and keep = exp(G_c - max(G_c, u_c)), take = exp(u_c - max(G_c, u_c)).
template <int KIND>
__global__ __launch_bounds__(256) void combine_chunks_kernel(ChunkPlan plan, StateFactors fa, float* __restrict__ state,
                                                             float* __restrict__ norm_state,
                                                             const int* __restrict__ state_slots, int H, int d, int e,
                                                             int blocks_per_head, int copies) {
  __shared__ float keep_s[TIE_WAVE], take_s[TIE_WAVE];
  const int tid = threadIdx.x, lane = tid & (TIE_WAVE - 1);
  const int hl = blockIdx.x / blocks_per_head, h = plan.h_first + hl, part = blockIdx.x % blocks_per_head;
  const int s = blockIdx.y, idx = part * 256 + tid;
  const size_t slot = state_slots[s];
  const int matrix = d * e;
  const int first = plan.first_item[s], last = plan.first_item[s + 1];
  if (first >= last) return;
  const bool live = idx < plan.per;
  float* S = state + (slot * H + h) * matrix + idx;
  float* nm = KIND == KIND_MEMORY ? norm_state + (slot * H + h) * copies * (d + 1) : nullptr;
  float v = 0.f;
  if (live) v = idx < matrix ? *S : nm[idx - matrix];
  double m = KIND == KIND_MEMORY ? static_cast<double>(plan.starts[static_cast<size_t>(first) * plan.heads + hl]) : 0.0;
  constexpr int AHEAD = 8;                              // chunks whose values are asked for before the chain needs them
  for (int c0 = first; c0 < last; c0 += TIE_WAVE) {     // uniform for the workgroup
    const int count = min(TIE_WAVE, last - c0);
    if (KIND == KIND_MEMORY) {
      if (tid < TIE_WAVE) {
        double b = 0.0, top = -INFINITY;
        const size_t at = static_cast<size_t>(c0 + lane) * plan.heads + hl;
        if (lane < count) {
          b = plan.sums[2 * at];
          top = plan.sums[2 * at + 1];
        }
        const double b_after = wave_running_sum(b, lane), before = b_after - b;
        const double u = top - before;
        const double most = fmax(m, wave_running_max(u, lane));
        double g = shfl_up_d(most, 1);
        if (lane == 0) g = m;
        keep_s[lane] = expf(static_cast<float>(g - most));
        take_s[lane] = expf(static_cast<float>(u - most));
        if (part == 0 && lane < count && c0 + lane > first) plan.starts[at] = static_cast<float>(before + g);
        m = shfl_d(b_after, count - 1) + shfl_d(most, count - 1);
      }
    } else if (tid < count) {
      keep_s[tid] = powf(fa.decay[h], static_cast<float>(plan.items[(c0 + tid) * 3 + 2] - plan.items[(c0 + tid) * 3 + 1]));
      take_s[tid] = 1.f;
    }
    __syncthreads();
    if (live) {
      float* at = plan.states + (static_cast<size_t>(c0) * plan.heads + hl) * plan.per + idx;
      const size_t stride = static_cast<size_t>(plan.heads) * plan.per;
      for (int c = 0; c < count; c += AHEAD) {
        float local[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) local[u] = at[stride * min(c + u, count - 1)];
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) {
          if (c + u >= count) break;
          at[stride * (c + u)] = v;
          v = fmaf(keep_s[c + u], v, take_s[c + u] * local[u]);
        }
      }
    }
    __syncthreads();
  }
  if (live) {
    if (idx < matrix) {
      *S = v;
    } else {
      for (int c = 0; c < copies; ++c) nm[static_cast<size_t>(c) * (d + 1) + idx - matrix] = v;
    }
  }
  // m is read by no workgroup of this launch (they take the copy in `starts`), so one may write it
  if (KIND == KIND_MEMORY && part == 0 && tid < TIE_WAVE)
    for (int c = lane; c < copies; c += TIE_WAVE) nm[static_cast<size_t>(c) * (d + 1) + d] = static_cast<float>(m);
}

// Launch 3. A workgroup owns 64 NT value columns of one (chunk, head), its waves 2 x 2: 32 tokens x 32 NT columns each. It
// goes through the key dimensions 32 at a time - queries and keys [token][dimension], the starting state [dimension][column]
// in LDS, the next 32 on their way - and forms Q S and the 64 x 64 scores Q K^T together (nothing above the diagonal);
// then the scores times D meet the values, 32 tokens at a time. Rows read along their length are read four words a lane:
// lane l takes the words 8 u + 4 (l / 32) + t, and instruction t pairs the two halves' words t; the other operand follows.
#define CO_K 36            // words of a staged row of 32 query or key dimensions
#define CO_P 68            // words of a row of 64 scores
template <int KIND, int NT, bool WHOLE>
__global__ __launch_bounds__(256) void chunk_output_kernel(StateInputs in, StateFactors fa, ChunkPlan plan,
                                                           float* __restrict__ out) {
  constexpr int COLS = 64 * NT;
  constexpr int CO_S = COLS + 8;                        // words of a row of state or value columns
  constexpr int SV = 32 * COLS / 1024;                  // pieces of four values a thread stages of those
  constexpr int PIECES = COLS / 4;                      // ... of a row
  __shared__ __attribute__((aligned(16))) float qk_s[2 * CHUNK_ROWS * CO_K];    // queries | keys, later the scores
  __shared__ __attribute__((aligned(16))) float sv_s[32 * CO_S];
  __shared__ float n_s[32], left_s[CHUNK_ROWS], floor_s[CHUNK_ROWS], scale_s[CHUNK_ROWS];
  __shared__ double a_s[CHUNK_ROWS], top_s[CHUNK_ROWS];
  static_assert(CHUNK_ROWS * CO_P <= 2 * CHUNK_ROWS * CO_K, "the scores fit where queries and keys were");
  float* q_s = qk_s;
  float* k_s = qk_s + CHUNK_ROWS * CO_K;
  float* p_s = qk_s;
  const int tid = threadIdx.x, wave = tid / TIE_WAVE, lane = tid & (TIE_WAVE - 1);
  const int half = lane >> 5, l32 = lane & 31;
  const int hl = blockIdx.y, h = plan.h_first + hl, item = blockIdx.z;
  const int H = in.H, d = in.d, e = in.e;
  const int e_first = blockIdx.x * COLS;
  const int t0 = plan.items[item * 3 + 1], n = plan.items[item * 3 + 2] - t0;
  const float* S = plan.states + (static_cast<size_t>(item) * plan.heads + hl) * plan.per;
  const float* qp = in.proj + static_cast<size_t>(t0) * in.row + in.q_col + h * d;
  const float* kp = in.proj + static_cast<size_t>(t0) * in.row + in.k_col + h * d;
  const float* vp = in.proj + static_cast<size_t>(t0) * in.row + in.v_col + h * e;
  const float log2_lam = KIND == KIND_DECAY ? log2f(fa.decay[h]) : 0.f;

  float4 qr[2], kr[2], sr[SV];
  float nr = 0.f;
  const int qj = tid >> 3, qi = (tid & 7) * 4;          // of queries and keys a thread stages the tokens qj and qj + 32
  const int sj = tid / PIECES, sc = (tid % PIECES) * 4; // of state or values the rows sj + u 256 / PIECES
  auto fetch = [&](int k0) {
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int j = qj + 32 * u;
      const size_t at = static_cast<size_t>(min(j, n - 1)) * in.row;
      qr[u] = load_piece<WHOLE>(qp + at, k0 + qi, d, j < n);
      kr[u] = load_piece<WHOLE>(kp + at, k0 + qi, d, j < n);
    }
#pragma unroll
    for (int u = 0; u < SV; ++u) {
      const int i = k0 + sj + u * (256 / PIECES);
      sr[u] = load_piece<WHOLE>(S + static_cast<size_t>(min(i, d - 1)) * e, e_first + sc, e, i < d);
    }
    if (KIND == KIND_MEMORY && tid < 32) nr = k0 + tid < d ? S[static_cast<size_t>(d) * e + k0 + tid] : 0.f;
  };
  fetch(0);
  if (wave == 0) {
    if (KIND == KIND_MEMORY) {
      double b, a;
      chunk_gates(in, fa, h, t0, n, lane, b, a);
      const double start = plan.starts[static_cast<size_t>(item) * plan.heads + hl];
      const double top = fmax(start, wave_running_max(a, lane));
      a_s[lane] = a;
      top_s[lane] = top;
      left_s[lane] = expf(static_cast<float>(start - top));
      floor_s[lane] = expf(-static_cast<float>(b + top));
    } else {
      left_s[lane] = decay_power(log2_lam, lane + 1);
    }
  }
  const int mt = wave >> 1, ct = wave & 1;
  state_f16_t acc_p, acc[NT];
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    acc_p[r] = 0.f;
#pragma unroll
    for (int c = 0; c < NT; ++c) acc[c][r] = 0.f;
  }
  float nq = 0.f;                                       // of token tid / 4, the dimensions tid % 4 modulo 4
  for (int k0 = 0; k0 < d; k0 += 32) {                  // uniform for the workgroup
    if (k0 > 0) __syncthreads();
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      *reinterpret_cast<float4*>(&q_s[(qj + 32 * u) * CO_K + qi]) = f4_map(qr[u], in.activation, in.q_scale);
      *reinterpret_cast<float4*>(&k_s[(qj + 32 * u) * CO_K + qi]) = f4_map(kr[u], in.activation, 1.f);
    }
#pragma unroll
    for (int u = 0; u < SV; ++u) *reinterpret_cast<float4*>(&sv_s[(sj + u * (256 / PIECES)) * CO_S + sc]) = sr[u];
    if (KIND == KIND_MEMORY && tid < 32) n_s[tid] = nr;
    __syncthreads();
    if (k0 + 32 < d) fetch(k0 + 32);
    const float* qa = q_s + (mt * 32 + l32) * CO_K + 4 * half;
    const float* ka = k_s + (ct * 32 + l32) * CO_K + 4 * half;
    const float* sb = sv_s + 4 * half * CO_S + ct * 32 * NT + l32;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const float4 q4 = *reinterpret_cast<const float4*>(qa + 8 * u);
      const float q[4] = {q4.x, q4.y, q4.z, q4.w};
      if (ct <= mt) {
        const float4 k4 = *reinterpret_cast<const float4*>(ka + 8 * u);
        const float k[4] = {k4.x, k4.y, k4.z, k4.w};
#pragma unroll
        for (int t = 0; t < 4; ++t) acc_p = __builtin_amdgcn_mfma_f32_32x32x2f32(q[t], k[t], acc_p, 0, 0, 0);
      }
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int c = 0; c < NT; ++c)
          acc[c] = __builtin_amdgcn_mfma_f32_32x32x2f32(q[t], sb[(8 * u + t) * CO_S + c * 32], acc[c], 0, 0, 0);
    }
    if (KIND == KIND_MEMORY) {
      const float* row = q_s + (tid >> 2) * CO_K;
#pragma unroll
      for (int i = 0; i < 8; ++i) nq = fmaf(row[4 * i + (tid & 3)], n_s[4 * i + (tid & 3)], nq);
    }
  }
  // values of the first 32 tokens on their way while the scores are finished
  float4 vr[SV];
  auto fetch_values = [&](int from) {
#pragma unroll
    for (int u = 0; u < SV; ++u) {
      const int j = from + sj + u * (256 / PIECES);
      vr[u] = load_piece<WHOLE>(vp + static_cast<size_t>(min(j, n - 1)) * in.row, e_first + sc, e, j < n);
    }
  };
  auto publish_values = [&]() {
#pragma unroll
    for (int u = 0; u < SV; ++u)
      *reinterpret_cast<float4*>(&sv_s[(sj + u * (256 / PIECES)) * CO_S + sc]) = f4_map(vr[u], in.activation, 1.f);
  };
  fetch_values(0);
  __syncthreads();                                      // queries, keys and state have been read
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int i = mt * 32 + 8 * (r / 4) + 4 * half + (r % 4), j = ct * 32 + l32;
    float p = 0.f;
    if (j <= i && i < n)
      p = acc_p[r] * (KIND == KIND_MEMORY ? expf(static_cast<float>(a_s[j] - top_s[i])) : decay_power(log2_lam, i - j));
    p_s[i * CO_P + j] = p;
    const float left = left_s[i];
#pragma unroll
    for (int c = 0; c < NT; ++c) acc[c][r] *= left;
  }
  publish_values();
  __syncthreads();
  if (KIND == KIND_MEMORY) {                            // four lanes a token: what the outputs are divided by
    const int i = tid >> 2;
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < 16; ++j) sum += p_s[i * CO_P + 4 * j + (tid & 3)];
    sum = fmaf(left_s[i], nq, sum);
    sum += __shfl_xor(sum, 1, TIE_WAVE);
    sum += __shfl_xor(sum, 2, TIE_WAVE);
    if ((tid & 3) == 0) scale_s[i] = 1.0f / (fmaxf(fabsf(sum), floor_s[i]) + 1e-6f);
  }
  for (int from = 0; from < n; from += 32) {            // uniform for the workgroup
    if (from > 0) {
      __syncthreads();
      publish_values();
      __syncthreads();
    }
    if (from + 32 < n) fetch_values(from + 32);
    if (from <= mt * 32) {                              // later tokens' values weigh nothing in the earlier tokens' rows
      const float* pa = p_s + (mt * 32 + l32) * CO_P + from + 4 * half;
      const float* vb = sv_s + 4 * half * CO_S + ct * 32 * NT + l32;
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float4 p4 = *reinterpret_cast<const float4*>(pa + 8 * u);
        const float p[4] = {p4.x, p4.y, p4.z, p4.w};
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int c = 0; c < NT; ++c)
            acc[c] = __builtin_amdgcn_mfma_f32_32x32x2f32(p[t], vb[(8 * u + t) * CO_S + c * 32], acc[c], 0, 0, 0);
      }
    }
  }
  if (KIND == KIND_MEMORY && n <= 32) __syncthreads();  // the factors above, where no second half brought a barrier
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int i = mt * 32 + 8 * (r / 4) + 4 * half + (r % 4);
    if (i >= n) continue;
    const float scale = KIND == KIND_MEMORY ? scale_s[i] : 1.f;
#pragma unroll
    for (int c = 0; c < NT; ++c) {
      const int col = e_first + ct * 32 * NT + c * 32 + l32;
      if (col < e) out[(static_cast<size_t>(t0 + i) * H + h) * e + col] = acc[c][r] * scale;
    }
  }
}

// ------------------------------------------------------------------ launches
extern "C" int tie_matrix_state_walk_cols() { return WALK_COLS; }

static bool bad_inputs(const StateInputs& in, const StateFactors& fa, int kind) {
  if (in.proj == nullptr || in.H <= 0 || in.H > 65535 || in.d <= 0 || in.d > STATE_MAX_D || in.e <= 0 ||
      static_cast<long>(in.d) * in.e > (1L << 28) || kind < KIND_DECAY || kind > KIND_MEMORY)
    return true;
  const long row = in.row, hd = static_cast<long>(in.H) * in.d, he = static_cast<long>(in.H) * in.e;
  if (in.q_col < 0 || in.k_col < 0 || in.v_col < 0 || in.q_col + hd > row || in.k_col + hd > row || in.v_col + he > row)
    return true;
  if (kind == KIND_DECAY) return fa.decay == nullptr || (in.angles != nullptr && (in.rot <= 0 || in.rot % 2 || in.rot > in.d));
  return fa.i_bias == nullptr || fa.f_bias == nullptr || fa.i_col < 0 || fa.f_col < 0 || fa.i_col + in.H > row ||
         fa.f_col + in.H > row || !(fa.cap > 0.f) || in.angles != nullptr;
}

// kind 0: decay [H], angles [T][rot] or null; kind 1: biases [H], norm_state [slots][H][ceil(e / WALK_COLS)][d + 1].
// proj rows query_start[0] .. query_start[S] - 1; out [T][H][e]; state [slots][H][d][e]. single: every sequence brings one
// row.
extern "C" int tie_matrix_state_walk(int kind, const float* proj, int row, int q_col, int k_col, int v_col, int activation,
                                     float q_scale, const float* angles, int rot, const float* decay, const float* i_bias,
                                     const float* f_bias, int i_col, int f_col, float cap, float* out, float* state,
                                     float* norm_state, const int* query_start, const int* state_slots, int single, int S,
                                     int H, int d, int e, hipStream_t stream) {
  const StateInputs in{proj, row, q_col, k_col, v_col, activation, q_scale, angles, rot, H, d, e};
  const StateFactors fa{decay, i_bias, f_bias, i_col, f_col, cap};
  if (bad_inputs(in, fa, kind) || S <= 0 || S > 65535 || out == nullptr || state == nullptr ||
      (kind == KIND_MEMORY && norm_state == nullptr))
    return TIE_BAD_ARGUMENT;
  const dim3 grid((e + WALK_COLS - 1) / WALK_COLS, H, S);
#define WALK(KIND, RPT)                                                                                                    \
  {                                                                                                                       \
    if (single)                                                                                                           \
      state_step_kernel<KIND, RPT><<<grid, 256, 0, stream>>>(in, fa, out, state, norm_state, query_start, state_slots);   \
    else                                                                                                                  \
      state_walk_kernel<KIND, RPT><<<grid, 256, 0, stream>>>(in, fa, out, state, norm_state, query_start, state_slots);   \
  }
#define WALKS(RPT)                              \
  {                                             \
    if (kind == KIND_DECAY) WALK(KIND_DECAY, RPT) \
    else WALK(KIND_MEMORY, RPT)                 \
  }
  if (d <= 32) WALKS(1)
  else if (d <= 64) WALKS(2)
  else if (d <= 128) WALKS(4)
  else if (d <= 256) WALKS(8)
  else WALKS(16)
#undef WALKS
#undef WALK
  return tie_launch_status();
}

// The same over items [count][3] (chunks of at most CHUNK_ROWS rows) and first_item [S + 1], for the heads h_first ..
// h_first + heads - 1. Scratch: states [count][heads][d e (+ d for kind 1)], and for kind 1 sums [count][heads][2] doubles and
// starts [count][heads]. Queries and keys must have been rotated already.
extern "C" int tie_matrix_state_chunks(int kind, const float* proj, int row, int q_col, int k_col, int v_col, int activation,
                                       float q_scale, const float* decay, const float* i_bias, const float* f_bias, int i_col,
                                       int f_col, float cap, float* out, float* state, float* norm_state,
                                       const int* state_slots, const int* items, const int* first_item, int count,
                                       int longest, float* states, double* sums, float* starts, int h_first, int heads, int S,
                                       int H, int d, int e, hipStream_t stream) {
  const StateInputs in{proj, row, q_col, k_col, v_col, activation, q_scale, nullptr, 0, H, d, e};
  const StateFactors fa{decay, i_bias, f_bias, i_col, f_col, cap};
  if (bad_inputs(in, fa, kind) || S <= 0 || S > 65535 || out == nullptr || state == nullptr || items == nullptr ||
      first_item == nullptr || states == nullptr || count <= 0 || count > 65535 || longest <= 0 || longest > CHUNK_ROWS ||
      h_first < 0 || heads <= 0 || h_first + heads > H ||
      (kind == KIND_MEMORY && (norm_state == nullptr || sums == nullptr || starts == nullptr)))
    return TIE_BAD_ARGUMENT;
  const int per = d * e + (kind == KIND_MEMORY ? d : 0);
  const ChunkPlan plan{items, first_item, states, sums, starts, h_first, heads, per};
  const int copies = (e + WALK_COLS - 1) / WALK_COLS;
  const int blocks_e = (e + 127) / 128, blocks_d = (d + 127) / 128;
  const int per_head = (per + 255) / 256;
  const dim3 grid1(blocks_d * blocks_e, heads, count), grid2(per_head * heads, S);
  // rows of whole aligned pieces of four: keys, queries, values of every head, the chunks' states
  const bool whole = row % 4 == 0 && q_col % 4 == 0 && k_col % 4 == 0 && v_col % 4 == 0 && d % 4 == 0 && e % 4 == 0 &&
                     reinterpret_cast<uintptr_t>(proj) % 16 == 0 && reinterpret_cast<uintptr_t>(states) % 16 == 0;
#define PASSES_W(KIND, WHOLE)                                                                                         \
  {                                                                                                                   \
    chunk_state_kernel<KIND, WHOLE><<<grid1, 256, 0, stream>>>(in, fa, plan, norm_state, state_slots, blocks_e, copies); \
    combine_chunks_kernel<KIND><<<grid2, 256, 0, stream>>>(plan, fa, state, norm_state, state_slots, H, d, e,         \
                                                           per_head, copies);                                         \
    if (e <= 64)                                                                                                      \
      chunk_output_kernel<KIND, 1, WHOLE><<<dim3(1, heads, count), 256, 0, stream>>>(in, fa, plan, out);              \
    else                                                                                                              \
      chunk_output_kernel<KIND, 2, WHOLE><<<dim3(blocks_e, heads, count), 256, 0, stream>>>(in, fa, plan, out);       \
  }
#define PASSES(KIND)                   \
  {                                    \
    if (whole) PASSES_W(KIND, true)    \
    else PASSES_W(KIND, false)         \
  }
  if (kind == KIND_DECAY) PASSES(KIND_DECAY)
  else PASSES(KIND_MEMORY)
#undef PASSES
#undef PASSES_W
  return tie_launch_status();
}

// ------------------------------------------------------------------ rotation in place
// The first rot dimensions of `heads` heads of d columns each, from column q_col and again from column k_col, of float32
// rows: pairs (i, i + rot / 2) by the row's angles [T][rot] = cos | sin.
__global__ void rotate_heads_kernel(float* __restrict__ rows, int row, int q_col, int k_col, const float* __restrict__ angles,
                                    int rot, int heads, int d) {
  const int half = rot / 2, pairs = heads * half;
  const int p = blockIdx.x * blockDim.x + threadIdx.x;
  if (p >= 2 * pairs) return;
  const size_t t = blockIdx.y;
  const int j = p < pairs ? p : p - pairs;
  const int h = j / half, i = j - h * half;
  float* at = rows + t * row + (p < pairs ? q_col : k_col) + h * d + i;
  const float* a = angles + t * rot;
  const float u = at[0], v = at[half], cs = a[i], sn = a[half + i];
  at[0] = u * cs - v * sn;
  at[half] = v * cs + u * sn;
}

extern "C" int tie_rotate_heads(float* rows, int row, int q_col, int k_col, const float* angles, int rot, int T, int heads,
                                int d, hipStream_t stream) {
  if (rows == nullptr || angles == nullptr || T <= 0 || T > 65535 || heads <= 0 || d <= 0 || rot <= 0 || rot % 2 || rot > d ||
      q_col < 0 || k_col < 0 || static_cast<long>(q_col) + static_cast<long>(heads) * d > row ||
      static_cast<long>(k_col) + static_cast<long>(heads) * d > row)
    return TIE_BAD_ARGUMENT;
  const int pairs = heads * rot;
  rotate_heads_kernel<<<dim3((pairs + 255) / 256, T), 256, 0, stream>>>(rows, row, q_col, k_col, angles, rot, heads, d);
  return tie_launch_status();
}
