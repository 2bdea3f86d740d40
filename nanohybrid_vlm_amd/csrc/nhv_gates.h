// What a gated feed-forward makes of a gate g and an up value u, for the kernels that have both (the few-rows product
// with two matrices, and the kernel that takes the packed rows of a product):
//   act 0: g sigmoid(g) u   (SiLU)
//   act 1: 0.5 g (1 + tanh(sqrt(2 / pi) (g + 0.044715 g^3))) u   (GELU in its tanh form)
//   act 2: with g' = min(g, limit) and u' = clamp(u, -limit, limit): g' sigmoid(alpha g') (u' + offset)
#pragma once
#include <hip/hip_runtime.h>

struct NhvGate {
  int act;
  float limit, alpha, offset;      // of act 2
};

template <int ACT>
__device__ __forceinline__ float nhv_gated(float g, float u, const NhvGate& p) {
  if (ACT == 2) {
    g = fminf(g, p.limit);
    u = fminf(fmaxf(u, -p.limit), p.limit);
    return g / (1.0f + expf(-p.alpha * g)) * (u + p.offset);
  }
  if (ACT == 1) return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g))) * u;
  return g / (1.0f + expf(-g)) * u;
}

__device__ __forceinline__ float nhv_gated(float g, float u, const NhvGate& p) {
  if (p.act == 2) return nhv_gated<2>(g, u, p);
  if (p.act == 1) return nhv_gated<1>(g, u, p);
  return nhv_gated<0>(g, u, p);
}
