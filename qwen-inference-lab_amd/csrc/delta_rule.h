// What the kernels of the gated delta rule share: where a step's inputs lie and the float32 arithmetic on them.
#pragma once
#include "common.h"
#include "operand.h"

struct DeltaInputs {
  const void* u;                                           // [n, u_row] of the model's type: queries, keys, values
  int u_row, q_off, k_off, v_off;
  Operand z;                                               // [n, z_row]: raw decays, column head * dim + channel
  int z_row;
  const float* bias;                                       // [heads * dim], joins the raw decays
  const float* rates;                                      // [heads]: -exp(A_log), natural logarithm's units
  Operand b;                                               // [n, b_row]: raw step size of head h at column h
  int b_row;
};

#define DELTA_UNIT_EPS 1e-6f                               // joins the sum of squares that makes unit vectors

__device__ __forceinline__ float delta_softplus(float v) { return v > 20.f ? v : log1pf(expf(v)); }
__device__ __forceinline__ float delta_log_decay(const DeltaInputs& in, int row, int h, int dim, int c) {
  return in.rates[h] * delta_softplus(operand_at(in.z, (size_t)row * in.z_row + h * dim + c) + in.bias[h * dim + c]);
}
__device__ __forceinline__ float delta_step_size(const DeltaInputs& in, int row, int h) {
  return 1.f / (1.f + expf(-operand_at(in.b, (size_t)row * in.b_row + h)));
}
