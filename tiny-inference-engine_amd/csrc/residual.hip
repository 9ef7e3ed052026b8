// What sub-layers that ran side by side on the same rows add to the residual stream, in one pass, with the norm that
// reads the stream next:
//
//   x <- x + scale * ( sum of a's planes + sum of b's planes + sum_k weights[k] parts[where[k]] ) ;   h = norm(x) * w
//
// a and b are results as rows (one plane) or as planes of partial sums of a product cut along K; parts / where /
// weights are a routed feed-forward's results not yet combined (where -1: the expert returned its input `self`).
// Everything is float32 but h and `self`, which have the activation type. One workgroup a row; sums run in the order
// above, planes and choices in their own order.
#include "common.h"

struct ResidualTerms {
  const float* a;          // null: absent
  size_t a_stride;         // elements between two planes
  int a_planes;
  const float* b;
  size_t b_stride;
  int b_planes;
  const float* parts;      // null: no routed result
  const int* where;        // [T][top]
  const float* weights;    // [T][top], or null: all 1
  const void* self;
  int self_bf16;
  int top;
};

struct ResidualNorm {
  const float* w;          // null: no norm in this launch
  float eps;
  int kind;                // 0: layer norm, 1: RMS norm
};

__device__ __forceinline__ float self_value(const ResidualTerms& s, size_t at) {
  return s.self_bf16 ? bf16_to_float(static_cast<const bf16_t*>(s.self)[at]) : static_cast<const float*>(s.self)[at];
}

// Any width up to 16384: the row lies in LDS between the passes.
template <typename TO>
__global__ void add_results_kernel(float* __restrict__ x, float scale, ResidualTerms s, ResidualNorm nm,
                                   TO* __restrict__ h, int n) {
  extern __shared__ float row_s[];
  __shared__ float scratch[16];
  const size_t t = blockIdx.x;
  float sum = 0.f;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    const size_t at = t * n + c;
    float y = 0.f;
    if (s.a)
      for (int p = 0; p < s.a_planes; ++p) y += s.a[p * s.a_stride + at];
    if (s.b)
      for (int p = 0; p < s.b_planes; ++p) y += s.b[p * s.b_stride + at];
    if (s.parts)
      for (int k = 0; k < s.top; ++k) {
        const int place = s.where[t * s.top + k];
        y = fmaf(s.weights ? s.weights[t * s.top + k] : 1.f, place >= 0 ? s.parts[static_cast<size_t>(place) * n + c] : self_value(s, at), y);
      }
    const float v = fmaf(scale, y, x[at]);
    x[at] = v;
    if (nm.w) row_s[c] = v;
    sum += v;
  }
  if (!nm.w) return;
  const float mean = nm.kind == 0 ? block_sum(sum, scratch) / static_cast<float>(n) : 0.f;
  float ss = 0.f;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    const float d = row_s[c] - mean;
    ss = fmaf(d, d, ss);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(n) + nm.eps);
  for (int c = threadIdx.x; c < n; c += blockDim.x) store_from_float(h + t * n + c, ((row_s[c] - mean) * inv) * nm.w[c]);
}

__device__ __forceinline__ float4 f4_add(float4 a, float4 b) {
  return make_float4(a.x + b.x, a.y + b.y, a.z + b.z, a.w + b.w);
}
__device__ __forceinline__ float4 f4_fma(float a, float4 b, float4 c) {
  return make_float4(fmaf(a, b.x, c.x), fmaf(a, b.y, c.y), fmaf(a, b.z, c.z), fmaf(a, b.w, c.w));
}
__device__ __forceinline__ float4 f4_load(const float* p) { return *reinterpret_cast<const float4*>(p); }

// Planes 0 .. planes - 1 added to y in order, four loads under way at a time.
__device__ __forceinline__ float4 add_planes(float4 y, const float* p, size_t stride, int planes) {
  int i = 0;
  for (; i + 4 <= planes; i += 4) {
    const float4 v0 = f4_load(p + i * stride), v1 = f4_load(p + (i + 1) * stride);
    const float4 v2 = f4_load(p + (i + 2) * stride), v3 = f4_load(p + (i + 3) * stride);
    y = f4_add(f4_add(f4_add(f4_add(y, v0), v1), v2), v3);
  }
  for (; i < planes; ++i) y = f4_add(y, f4_load(p + i * stride));
  return y;
}

// The same for rows in steps of four columns: a thread holds V x four columns in registers from the first load to the
// last store, and the stream's and the norm weight's values are asked for before anything is added.
template <typename TO, int V>
__global__ void add_results_row_kernel(float* __restrict__ x, float scale, ResidualTerms s, ResidualNorm nm,
                                       TO* __restrict__ h, int n) {
  __shared__ float scratch[16];
  const size_t t = blockIdx.x, row = t * n;
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 v[V], w[V];
#pragma unroll
  for (int j = 0; j < V; ++j) {
    const int c = (threadIdx.x + j * blockDim.x) * 4;
    v[j] = c < n ? f4_load(x + row + c) : zero;
    w[j] = (c < n && nm.w) ? f4_load(nm.w + c) : zero;
  }
  float sum = 0.f;
#pragma unroll
  for (int j = 0; j < V; ++j) {
    const int c = (threadIdx.x + j * blockDim.x) * 4;
    if (c >= n) continue;
    float4 y = zero;
    if (s.a) y = add_planes(y, s.a + row + c, s.a_stride, s.a_planes);
    if (s.b) y = add_planes(y, s.b + row + c, s.b_stride, s.b_planes);
    if (s.parts) {
      const int* places = s.where + t * s.top;
      const float* weights = s.weights ? s.weights + t * s.top : nullptr;
      for (int k0 = 0; k0 < s.top; k0 += 4) {
        float4 part[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          if (k0 + k >= s.top) break;
          const int place = places[k0 + k];
          part[k] = place >= 0 ? f4_load(s.parts + static_cast<size_t>(place) * n + c)
                               : make_float4(self_value(s, row + c), self_value(s, row + c + 1),
                                             self_value(s, row + c + 2), self_value(s, row + c + 3));
        }
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          if (k0 + k >= s.top) break;
          y = f4_fma(weights ? weights[k0 + k] : 1.f, part[k], y);
        }
      }
    }
    v[j] = f4_fma(scale, y, v[j]);
    *reinterpret_cast<float4*>(x + row + c) = v[j];
    sum += (v[j].x + v[j].y) + (v[j].z + v[j].w);
  }
  if (!nm.w) return;
  const float mean = nm.kind == 0 ? block_sum(sum, scratch) / static_cast<float>(n) : 0.f;
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < V; ++j) {
    if ((threadIdx.x + j * blockDim.x) * 4 >= n) continue;
    const float a = v[j].x - mean, b = v[j].y - mean, c = v[j].z - mean, d = v[j].w - mean;
    ss += (a * a + b * b) + (c * c + d * d);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(n) + nm.eps);
#pragma unroll
  for (int j = 0; j < V; ++j) {
    const int c = (threadIdx.x + j * blockDim.x) * 4;
    if (c >= n) continue;
    const float o0 = ((v[j].x - mean) * inv) * w[j].x, o1 = ((v[j].y - mean) * inv) * w[j].y;
    const float o2 = ((v[j].z - mean) * inv) * w[j].z, o3 = ((v[j].w - mean) * inv) * w[j].w;
    if constexpr (sizeof(TO) == 2)
      *reinterpret_cast<uint2*>(h + row + c) = make_uint2(pack_bf16x2(o0, o1), pack_bf16x2(o2, o3));
    else
      *reinterpret_cast<float4*>(h + row + c) = make_float4(o0, o1, o2, o3);
  }
}

template <typename TO>
static void launch_add_results(float* x, float scale, const ResidualTerms& s, const ResidualNorm& nm, TO* h, int T,
                               int n, hipStream_t stream) {
  const int quads = n / 4;
  if (n % 4 == 0 && s.a_stride % 4 == 0 && s.b_stride % 4 == 0) {
    if (quads <= 1024) {
      const int threads = (quads + TIE_WAVE - 1) / TIE_WAVE * TIE_WAVE;
      add_results_row_kernel<TO, 1><<<T, threads, 0, stream>>>(x, scale, s, nm, h, n);
    } else if (quads <= 2048) {
      add_results_row_kernel<TO, 2><<<T, 1024, 0, stream>>>(x, scale, s, nm, h, n);
    } else {
      add_results_row_kernel<TO, 4><<<T, 1024, 0, stream>>>(x, scale, s, nm, h, n);
    }
    return;
  }
  const int threads = n >= 4096 ? 512 : (n >= 1024 ? 256 : (n >= 256 ? 128 : 64));
  const size_t lds = nm.w ? static_cast<size_t>(n) * sizeof(float) : 0;
  add_results_kernel<TO><<<T, threads, lds, stream>>>(x, scale, s, nm, h, n);
}

// x [T][n]; a, b: `planes` planes of [T][n] `stride` elements apart (or null); parts [slots][n], where and weights
// [T][top], self [T][n] of self_dtype (or parts null). w (or null): the norm of the updated rows into h of h_dtype.
extern "C" int tie_add_results(float* x, float scale, const float* a, long a_stride, int a_planes, const float* b,
                               long b_stride, int b_planes, const float* parts, const int* where, const float* weights,
                               const void* self, int self_dtype, int top, const float* w, float eps, int kind, void* h,
                               int h_dtype, int T, int n, hipStream_t stream) {
  if (!x || T <= 0 || n <= 0 || n > 16384 || (a && a_planes < 1) || (b && b_planes < 1)) return TIE_BAD_ARGUMENT;
  if (parts && (!where || !self || top < 1 || (self_dtype != TIE_F32 && self_dtype != TIE_BF16)))
    return TIE_BAD_ARGUMENT;
  if (w && (!h || (kind != 0 && kind != 1))) return TIE_BAD_ARGUMENT;
  const ResidualTerms s{a, static_cast<size_t>(a_stride), a_planes, b, static_cast<size_t>(b_stride), b_planes,
                        parts, where, weights, self, self_dtype == TIE_BF16, top};
  const ResidualNorm nm{w, eps, kind};
  if (!w || h_dtype == TIE_F32) launch_add_results(x, scale, s, nm, static_cast<float*>(h), T, n, stream);
  else if (h_dtype == TIE_BF16) launch_add_results(x, scale, s, nm, static_cast<bf16_t*>(h), T, n, stream);
  else return TIE_BAD_ARGUMENT;
  return tie_launch_status();
}

// ------------------------------------------------------- results that are normed before they are added
//   x <- x + a / rms(a) * w_a + b / rms(b) * w_b ;   h = x / rms(x) * w
// for one or two results (rows or planes of partial sums). One workgroup a row, everything in float32, one pass.
struct NormedTerm {
  const float* y;          // null: absent
  size_t stride;
  int planes;
  const float* w;
  float eps;
};

__device__ __forceinline__ float2 block_sum2(float a, float b, float2* scratch) {
  const int lane = threadIdx.x & (TIE_WAVE - 1), wave = threadIdx.x / TIE_WAVE;
  const int waves = (blockDim.x + TIE_WAVE - 1) / TIE_WAVE;
  a = wave_sum(a);
  b = wave_sum(b);
  __syncthreads();
  if (lane == 0) scratch[wave] = make_float2(a, b);
  __syncthreads();
  float2 total = make_float2(0.f, 0.f);
  for (int w = 0; w < waves; ++w) total.x += scratch[w].x, total.y += scratch[w].y;
  return total;
}

__device__ __forceinline__ float term_value(const NormedTerm& s, size_t at) {
  float y = 0.f;
  for (int p = 0; p < s.planes; ++p) y += s.y[p * s.stride + at];
  return y;
}

// Any width: the results are read again for the second pass.
template <typename TO>
__global__ void add_normed_results_kernel(float* __restrict__ x, NormedTerm a, NormedTerm b, const float* __restrict__ w,
                                          float eps, TO* __restrict__ h, int n) {
  __shared__ float2 scratch2[16];
  __shared__ float scratch[16];
  const size_t row = static_cast<size_t>(blockIdx.x) * n;
  float sa = 0.f, sb = 0.f;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    const float va = term_value(a, row + c), vb = b.y ? term_value(b, row + c) : 0.f;
    sa = fmaf(va, va, sa);
    sb = fmaf(vb, vb, sb);
  }
  const float2 sums = block_sum2(sa, sb, scratch2);
  const float inv_a = 1.0f / sqrtf(sums.x / static_cast<float>(n) + a.eps);
  const float inv_b = b.y ? 1.0f / sqrtf(sums.y / static_cast<float>(n) + b.eps) : 0.f;
  float ss = 0.f;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    float v = x[row + c] + (term_value(a, row + c) * inv_a) * a.w[c];
    if (b.y) v += (term_value(b, row + c) * inv_b) * b.w[c];
    x[row + c] = v;
    ss = fmaf(v, v, ss);
  }
  if (!w) return;
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(n) + eps);
  for (int c = threadIdx.x; c < n; c += blockDim.x) store_from_float(h + row + c, (x[row + c] * inv) * w[c]);
}

__device__ __forceinline__ float4 f4_scaled(float4 y, float inv, float4 w) {
  return make_float4((y.x * inv) * w.x, (y.y * inv) * w.y, (y.z * inv) * w.z, (y.w * inv) * w.w);
}
__device__ __forceinline__ float f4_square(float4 v) { return (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w); }

// Rows in steps of four columns: V x four columns a thread, in registers from the first load to the last store.
template <typename TO, int V>
__global__ void add_normed_results_row_kernel(float* __restrict__ x, NormedTerm a, NormedTerm b,
                                              const float* __restrict__ w, float eps, TO* __restrict__ h, int n) {
  __shared__ float2 scratch2[16];
  __shared__ float scratch[16];
  const size_t row = static_cast<size_t>(blockIdx.x) * n;
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 v[V], ya[V], yb[V], wa[V], wb[V], wn[V];
  float sa = 0.f, sb = 0.f;
#pragma unroll
  for (int j = 0; j < V; ++j) {
    const int c = (threadIdx.x + j * blockDim.x) * 4;
    const bool in = c < n;
    v[j] = in ? f4_load(x + row + c) : zero;
    wa[j] = in ? f4_load(a.w + c) : zero;
    wb[j] = (in && b.y) ? f4_load(b.w + c) : zero;
    wn[j] = (in && w) ? f4_load(w + c) : zero;
    ya[j] = in ? add_planes(zero, a.y + row + c, a.stride, a.planes) : zero;
    yb[j] = (in && b.y) ? add_planes(zero, b.y + row + c, b.stride, b.planes) : zero;
    sa += f4_square(ya[j]);
    sb += f4_square(yb[j]);
  }
  const float2 sums = block_sum2(sa, sb, scratch2);
  const float inv_a = 1.0f / sqrtf(sums.x / static_cast<float>(n) + a.eps);
  const float inv_b = b.y ? 1.0f / sqrtf(sums.y / static_cast<float>(n) + b.eps) : 0.f;
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < V; ++j) {
    const int c = (threadIdx.x + j * blockDim.x) * 4;
    if (c >= n) continue;
    v[j] = f4_add(f4_add(v[j], f4_scaled(ya[j], inv_a, wa[j])), f4_scaled(yb[j], inv_b, wb[j]));
    *reinterpret_cast<float4*>(x + row + c) = v[j];
    ss += f4_square(v[j]);
  }
  if (!w) return;
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(n) + eps);
#pragma unroll
  for (int j = 0; j < V; ++j) {
    const int c = (threadIdx.x + j * blockDim.x) * 4;
    if (c >= n) continue;
    const float4 o = f4_scaled(v[j], inv, wn[j]);
    if constexpr (sizeof(TO) == 2)
      *reinterpret_cast<uint2*>(h + row + c) = make_uint2(pack_bf16x2(o.x, o.y), pack_bf16x2(o.z, o.w));
    else
      *reinterpret_cast<float4*>(h + row + c) = o;
  }
}

template <typename TO>
static void launch_add_normed(float* x, const NormedTerm& a, const NormedTerm& b, const float* w, float eps, TO* h, int T,
                              int n, hipStream_t stream) {
  const int quads = n / 4;
  if (n % 4 == 0 && a.stride % 4 == 0 && b.stride % 4 == 0) {
    if (quads <= 1024)
      add_normed_results_row_kernel<TO, 1><<<T, (quads + TIE_WAVE - 1) / TIE_WAVE * TIE_WAVE, 0, stream>>>(x, a, b, w, eps, h, n);
    else if (quads <= 2048)
      add_normed_results_row_kernel<TO, 2><<<T, 1024, 0, stream>>>(x, a, b, w, eps, h, n);
    else
      add_normed_results_row_kernel<TO, 4><<<T, 1024, 0, stream>>>(x, a, b, w, eps, h, n);
    return;
  }
  const int threads = n >= 4096 ? 512 : (n >= 1024 ? 256 : (n >= 256 ? 128 : 64));
  add_normed_results_kernel<TO><<<T, threads, 0, stream>>>(x, a, b, w, eps, h, n);
}

// x [T][n]; a and b (b.y null: one result): `planes` planes of [T][n] `stride` elements apart, a norm weight [n] and an eps
// each. w (or null): the RMS norm of the updated rows into h of h_dtype.
extern "C" int tie_add_normed_results(float* x, const float* a, long a_stride, int a_planes, const float* a_w, float a_eps,
                                      const float* b, long b_stride, int b_planes, const float* b_w, float b_eps,
                                      const float* w, float eps, void* h, int h_dtype, int T, int n, hipStream_t stream) {
  if (!x || !a || !a_w || a_planes < 1 || T <= 0 || n <= 0 || n > 16384 || (b && (!b_w || b_planes < 1)) || (w && !h))
    return TIE_BAD_ARGUMENT;
  const NormedTerm ta{a, static_cast<size_t>(a_stride), a_planes, a_w, a_eps};
  const NormedTerm tb{b, static_cast<size_t>(b_stride), b_planes, b_w, b_eps};
  if (!w || h_dtype == TIE_F32) launch_add_normed(x, ta, tb, w, eps, static_cast<float*>(h), T, n, stream);
  else if (h_dtype == TIE_BF16) launch_add_normed(x, ta, tb, w, eps, static_cast<bf16_t*>(h), T, n, stream);
  else return TIE_BAD_ARGUMENT;
  return tie_launch_status();
}
