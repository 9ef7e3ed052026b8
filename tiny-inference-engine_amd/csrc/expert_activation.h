// What an expert makes of its first products' sums, by mode: 0 nothing (the down product), 1 silu(gate) * up,
// 2 relu(up)^2 (experts without a gate), 3 a gate and an up cut off at a limit, 4 as 1 with both sums times the weight of
// the (row, choice) slot: an expert whose input carries its weight.
#pragma once
#include "common.h"

struct GateParams {
  float limit, slope, shift;      // mode 3 only
  const float* slot_weights;      // mode 4 only: [slots]
};

__device__ __forceinline__ float silu_f(float g) { return g / (1.0f + expf(-g)); }
__device__ __forceinline__ float relu_squared_f(float a) { const float r = fmaxf(a, 0.f); return r * r; }
__device__ __forceinline__ float clipped_gate_f(float a, float b, GateParams p) {
  const float g = fminf(a, p.limit), u = fminf(fmaxf(b, -p.limit), p.limit);
  return g / (1.0f + expf(-p.slope * g)) * (u + p.shift);
}

// The same where the result is rounded to bfloat16: the hardware's exponential.
template <int MODE>
__device__ __forceinline__ float gated_fast(float a, float b, GateParams p) {
  static_assert(MODE == 1 || MODE == 3 || MODE == 4, "gated modes");
  if constexpr (MODE == 1 || MODE == 4) return a / (1.0f + __expf(-a)) * b;
  const float g = fminf(a, p.limit), u = fminf(fmaxf(b, -p.limit), p.limit);
  return g / (1.0f + __expf(-p.slope * g)) * (u + p.shift);
}
