// Activations: what a feed-forward makes of its gate and up columns, or (kinds from kGluKinds on) of its up columns alone.  The kind is
// the same for a whole launch.
#pragma once

#include "common.hpp"

namespace sgl_amd {

enum : int { kGluNone = 0, kGluSilu = 1, kGluGeluTanh = 2, kGluClampedSwish = 3, kGluKinds = 4, kActSquaredRelu = 4, kActKinds = 5 };

struct GluParams {
  int kind;
  float limit, alpha;          // of kGluClampedSwish
};

// gelu_tanh(g) * u: 0.5 (1 + tanh y) = 1 / (1 + exp(-2 y))
__device__ __forceinline__ float gelu_tanh_glu(float g, float u) {
  const float y = 0.7978845608028654f * (g + 0.044715f * g * g * g);
  return g / (1.0f + expf(-2.0f * y)) * u;
}
// g = min(g, limit), u in [-limit, limit]:  g sigmoid(alpha g) (u + 1)
__device__ __forceinline__ float clamped_swish_glu(const GluParams& p, float g, float u) {
  g = fminf(g, p.limit);
  u = fminf(fmaxf(u, -p.limit), p.limit);
  return g / (1.0f + expf(-p.alpha * g)) * (u + 1.0f);
}

__device__ __host__ __forceinline__ bool act_gated(int kind) { return kind > kGluNone && kind < kGluKinds; }
__device__ __host__ __forceinline__ bool act_pointwise(int kind) { return kind >= kGluKinds; }

// the one activation without a gate: relu(v)^2
__device__ __forceinline__ float squared_relu(float v) {
  v = fmaxf(v, 0.f);
  return v * v;
}

// kRound: silu keeps the rounding points of 16-bit activations (projection -> bf16, silu -> bf16); the other kinds stay in fp32
template <bool kRound>
__device__ __forceinline__ float glu(const GluParams& p, float g, float u) {
  if (p.kind == kGluGeluTanh) return gelu_tanh_glu(g, u);
  if (p.kind == kGluClampedSwish) return clamped_swish_glu(p, g, u);
  if (!kRound) return g / (1.0f + expf(-g)) * u;
  const float gb = rbf(g);
  return rbf(gb / (1.0f + expf(-gb))) * rbf(u);
}

}  // namespace sgl_amd
