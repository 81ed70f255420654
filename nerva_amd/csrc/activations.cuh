// Activations and recurrence steps shared by the projections' epilogues and the row kernels; all in f32.
#pragma once

#include "nv_common.cuh"

namespace nv {

__device__ __forceinline__ float sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }
__device__ __forceinline__ float softplus(float v) { return v > 20.0f ? v : log1pf(expf(v)); }

// xIELU: with two learned numbers (p, q), above zero softplus(p) z^2 + z / 2, at and below it
// (softplus(q) + 1/2) (e^z - 1 - z) + z / 2.
struct XieluParams {
  float above, below;
};
template <uint32_t DT>
__device__ __forceinline__ XieluParams xielu_params(const uint16_t *pq) {
  return XieluParams{softplus(dec16<DT>(pq[0])), 0.5f + softplus(dec16<DT>(pq[1]))};
}
__device__ __forceinline__ float xielu(float z, const XieluParams &a) {
  const float low = fminf(z, 0.0f);
  return (z > 0.0f ? a.above * z * z : a.below * (expm1f(low) - low)) + 0.5f * z;
}

// Gated linear unit with bounds: the gate from above, the linear part on both sides and moved up by one.
__device__ __forceinline__ float clamped_glu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid(1.702f * g) * (u + 1.0f);
}

// minGRU: gate and candidate from the current token alone (pre-activations with their biases added).
__device__ __forceinline__ float mingru_candidate(float u) { return u >= 0.0f ? u + 0.5f : sigmoid(u); }
__device__ __forceinline__ float mingru_step(float z_pre, float u, float state) {
  const float z = sigmoid(z_pre);
  return (1.0f - z) * state + z * mingru_candidate(u);
}

}  // namespace nv
