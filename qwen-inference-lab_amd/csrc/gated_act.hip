// Activations of gated feed-forwards over the gate and up halves of one product, by code:
//   0  silu(g) * u
//   1  g' = min(g, limit), u' = clamp(u, -limit, limit):  g' * sigmoid(alpha * g') * (u' + 1)
//   2  max(g, 0) * u
// The halves of a row of gate_up [n, 2 inner] are stacked (gate columns first) or interleaved in tiles of 16 columns.
#include "common.h"
#include "operand.h"
#include "partials.h"
#include "gated_act.h"

template <typename TD, typename T>
__global__ void gated_act_kernel(const TD* __restrict__ gate_up, int splits, size_t split_stride, size_t row, T* __restrict__ out,
                                 int inner, size_t total, int interleaved, int act, float limit, float alpha) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const size_t n = idx / inner;
  const int i = (int)(idx - n * inner);
  const size_t at = n * row + (interleaved ? (size_t)(i >> 4) * 32 + (i & 15) : (size_t)i);
  const float g = parts_sum(gate_up, at, splits, split_stride);
  const float u = parts_sum(gate_up, at + (interleaved ? 16 : inner), splits, split_stride);
  st(out + idx, gated_act(g, u, act, limit, alpha));
}

// Four results a thread, 16-byte (8-byte) loads and stores.
template <typename T>
__global__ void gated_act_vec_kernel(Operand gate_up, size_t row, T* __restrict__ out, int inner, size_t total4,
                                     int interleaved, int act, float limit, float alpha) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total4) return;
  const int per_row = inner / 4;
  const size_t n = idx / per_row;
  const int i = (int)(idx - n * per_row) * 4;
  const size_t at = n * row + (interleaved ? (size_t)(i >> 4) * 32 + (i & 15) : (size_t)i);
  const float4 g = operand_at4(gate_up, at), u = operand_at4(gate_up, at + (interleaved ? 16 : inner));
  st4(out + n * inner + i, make_float4(gated_act(g.x, u.x, act, limit, alpha), gated_act(g.y, u.y, act, limit, alpha),
                                       gated_act(g.z, u.z, act, limit, alpha), gated_act(g.w, u.w, act, limit, alpha)));
}

// bfloat16 in and out, eight results a thread.
__global__ void gated_act_bf16x8_kernel(const bf16_t* __restrict__ gate_up, size_t row, bf16_t* __restrict__ out, int inner,
                                        size_t total8, int interleaved, int act, float limit, float alpha) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total8) return;
  const int per_row = inner / 8;
  const size_t n = idx / per_row;
  const int i = (int)(idx - n * per_row) * 8;
  float g[8], u[8], y[8];
  const size_t at = n * row + (interleaved ? (size_t)(i >> 4) * 32 + (i & 15) : (size_t)i);
  ld8(gate_up + at, g);
  ld8(gate_up + at + (interleaved ? 16 : inner), u);
#pragma unroll
  for (int e = 0; e < 8; ++e) y[e] = gated_act(g[e], u[e], act, limit, alpha);
  *reinterpret_cast<uint4*>(out + n * (size_t)inner + i) =
      make_uint4(pack_bf16(y[0], y[1]), pack_bf16(y[2], y[3]), pack_bf16(y[4], y[5]), pack_bf16(y[6], y[7]));
}

extern "C" {

// gate_up: in_dtype QIL_BF16 [n, row] or QIL_F32 [splits][n][row] partial sums; a row holds 2 inner columns (and, row being
// larger, other columns that are skipped).
int qil_gated_act(const void* gate_up, int in_dtype, int splits, int row, void* out, int n, int inner, int out_dtype,
                  int interleaved, int act, float limit, float alpha, hipStream_t s) {
  const size_t total = (size_t)n * inner;
  if (total == 0) return 0;
  if (splits < 1 || (in_dtype == QIL_BF16 && splits != 1) || (interleaved && inner % 16) || act < 0 || act > QIL_ACT_RELU ||
      row < 2 * inner)
    return -1;
  const size_t stride = (size_t)n * row;
  const bool aligned = (((uintptr_t)gate_up | (uintptr_t)out) % 16) == 0;
  if (in_dtype == QIL_BF16 && out_dtype == QIL_BF16 && inner % 8 == 0 && row % 8 == 0 && aligned) {
    const size_t work = total / 8;
    hipLaunchKernelGGL(gated_act_bf16x8_kernel, dim3((unsigned)((work + 255) / 256)), dim3(256), 0, s, (const bf16_t*)gate_up,
                       (size_t)row, (bf16_t*)out, inner, work, interleaved, act, limit, alpha);
    QIL_RETURN_LAUNCH_STATUS();
  }
  if (in_dtype == QIL_F32 && inner % 4 == 0 && row % 4 == 0 && aligned) {
    const Operand in{gate_up, QIL_F32, splits, stride};
    const size_t work = total / 4;
    const unsigned blocks = (unsigned)((work + 255) / 256);
    if (out_dtype == QIL_F32)
      hipLaunchKernelGGL(gated_act_vec_kernel<float>, dim3(blocks), dim3(256), 0, s, in, (size_t)row, (float*)out, inner, work,
                         interleaved, act, limit, alpha);
    else
      hipLaunchKernelGGL(gated_act_vec_kernel<bf16_t>, dim3(blocks), dim3(256), 0, s, in, (size_t)row, (bf16_t*)out, inner,
                         work, interleaved, act, limit, alpha);
    QIL_RETURN_LAUNCH_STATUS();
  }
  const unsigned blocks = (unsigned)((total + 255) / 256);
#define QIL_ACT_CASE(TD, T)                                                                                            \
  hipLaunchKernelGGL((gated_act_kernel<TD, T>), dim3(blocks), dim3(256), 0, s, (const TD*)gate_up, splits, stride,      \
                     (size_t)row, (T*)out, inner, total, interleaved, act, limit, alpha)
  if (out_dtype == QIL_F32) {
    if (in_dtype != QIL_F32) return -1;
    QIL_ACT_CASE(float, float);
  } else if (in_dtype == QIL_F32) {
    QIL_ACT_CASE(float, bf16_t);
  } else {
    QIL_ACT_CASE(bf16_t, bf16_t);
  }
#undef QIL_ACT_CASE
  QIL_RETURN_LAUNCH_STATUS();
}

}  // extern "C"
