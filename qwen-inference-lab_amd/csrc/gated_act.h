// The gate functions of gated feed-forwards, shared by the activation kernel and by product kernels that apply the
// activation in their epilogue.  Everything is float32.
#pragma once
#include "common.h"

enum { QIL_ACT_SILU = 0, QIL_ACT_CLAMPED = 1, QIL_ACT_RELU = 2, QIL_ACT_RELU_SQUARED = 16 };

//   QIL_ACT_SILU     g * sigmoid(g) * u
//   QIL_ACT_CLAMPED  g' = min(g, limit), u' = clamp(u, -limit, limit):  g' * sigmoid(alpha * g') * (u' + 1)
//   QIL_ACT_RELU     max(g, 0) * u
__device__ __forceinline__ float gated_act(float g, float u, int act, float limit, float alpha) {
  if (act == QIL_ACT_CLAMPED) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return (g / (1.f + expf(-alpha * g))) * (u + 1.f);
  }
  if (act == QIL_ACT_RELU) return fmaxf(g, 0.f) * u;
  return (g / (1.f + expf(-g))) * u;
}

// Activations of experts without a gate branch, by code from QIL_ACT_RELU_SQUARED on:
//   QIL_ACT_RELU_SQUARED  max(z, 0)^2
__device__ __forceinline__ float ungated_act(float z, int act) {
  const float r = fmaxf(z, 0.f);
  return r * r;
}
