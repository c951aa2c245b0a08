// Gated activations of feed-forward products (gate g, up u), shared by the element-wise kernel, the grouped expert
// GEMMs' epilogues and gemm_pf's grouped form.
#pragma once

#include <hip/hip_runtime.h>

namespace xgk {

constexpr int kGluGeluTanh = 0, kGluClamped = 1, kGluSilu = 3;   // (2: an ungated activation of the expert products)

//   kGluGeluTanh   0.5 g (1 + tanh(sqrt(2 / pi) (g + 0.044715 g^3))) * u
//   kGluClamped    g' = min(g, limit), u' = clamp(u, -limit, limit):  g' sigmoid(alpha g') (u' + 1)
//   kGluSilu       g sigmoid(g) * u
__device__ __forceinline__ float glu(int kind, float g, float u, float limit, float alpha) {
  if (kind == kGluGeluTanh) {
    const float c = 0.7978845608028654f;  // sqrt(2 / pi)
    return 0.5f * g * (1.f + tanhf(c * (g + 0.044715f * g * g * g))) * u;
  }
  if (kind == kGluSilu) return g / (1.f + expf(-g)) * u;
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-alpha * g)) * (u + 1.f);
}

}  // namespace xgk
