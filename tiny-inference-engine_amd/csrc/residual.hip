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
  const float* weights;    // [T][top]
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
        y = fmaf(s.weights[t * s.top + k], place >= 0 ? s.parts[static_cast<size_t>(place) * n + c] : self_value(s, at), y);
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
      const float* weights = s.weights + t * s.top;
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
          y = f4_fma(weights[k0 + k], part[k], y);
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
  if (parts && (!where || !weights || !self || top < 1 || (self_dtype != TIE_F32 && self_dtype != TIE_BF16)))
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
