// What the sub-layers of a layer with gated branches leave joins the float32 residual stream, fused with the RMS norm
// that follows:
//     x = stream[r] + sigmoid(g1 + b1) * (a_scale * a + b_scale * b) + sigmoid(g2 + b2) * f + plus[r] + step
//     if (update) stream[r] = x
//     out[m] = x / sqrt(mean(x^2) + eps) * weight
// with r = rows ? rows[m] : m.  a, b: the mixer's output, or the outputs of two mixers side by side (b optional); f: the
// feed-forward's output (optional).  g1, g2: the gates' logits (columns [0, width) and [width, 2 width) of the operand
// `gates`) with stored biases b1, b2 behind one another; without gates the factors are 1.  plus float32 [.., width] and
// step float32 [width]: what a pass of a loop over layers adds before its first layer (optional).  Every operand is an
// array of the model's type or float32 partial sums (operand.h).  Everything is float32 until the one rounding of `out`.
// One block a row; the row waits in LDS between the sum and the norm.
#include "common.h"
#include "operand.h"

struct JoinInputs {
  Operand a, b, f, gates;                                  // data null: not there
  size_t a_row, b_row, f_row, g_row;                       // elements between two rows
  float a_scale, b_scale;
  const float* bias;                                       // [2 width] (or [width] without f)
  const float* plus;
  const float* step;
};

template <int V> __device__ __forceinline__ void join_load(const Operand& x, size_t at, float* v) {
  if constexpr (V == 4) {
    const float4 q = operand_at4(x, at);
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
  } else {
    v[0] = operand_at(x, at);
  }
}
template <int V> __device__ __forceinline__ void join_floats(const float* p, float* v) {
  if constexpr (V == 4) {
    const float4 q = ld4(p);
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
  } else {
    v[0] = p[0];
  }
}

template <typename T, int V>
__global__ void residual_join_kernel(float* __restrict__ stream, JoinInputs in, const int* __restrict__ rows,
                                     const float* __restrict__ weight, T* __restrict__ out, int width, float eps, int update) {
  extern __shared__ __align__(16) float held[];            // [width]
  __shared__ float scratch[16];
  const int m = blockIdx.x;
  const size_t r = rows ? (size_t)rows[m] : (size_t)m;
  float* x = stream + r * width;
  float squares = 0.f;
  for (int i = threadIdx.x * V; i < width; i += blockDim.x * V) {
    float v[V], t[V], u[V];
    join_floats<V>(x + i, v);
    if (in.a.data) {
      join_load<V>(in.a, r * in.a_row + i, t);
#pragma unroll
      for (int e = 0; e < V; ++e) t[e] *= in.a_scale;
      if (in.b.data) {
        join_load<V>(in.b, r * in.b_row + i, u);
#pragma unroll
        for (int e = 0; e < V; ++e) t[e] += in.b_scale * u[e];
      }
      if (in.gates.data) {
        float b[V];
        join_load<V>(in.gates, r * in.g_row + i, u);
        join_floats<V>(in.bias + i, b);
#pragma unroll
        for (int e = 0; e < V; ++e) t[e] = t[e] / (1.f + expf(-(u[e] + b[e])));
      }
      if (in.f.data) {
        float f[V];
        join_load<V>(in.f, r * in.f_row + i, f);
        if (in.gates.data) {
          float b[V];
          join_load<V>(in.gates, r * in.g_row + width + i, u);
          join_floats<V>(in.bias + width + i, b);
#pragma unroll
          for (int e = 0; e < V; ++e) f[e] = f[e] / (1.f + expf(-(u[e] + b[e])));
        }
#pragma unroll
        for (int e = 0; e < V; ++e) t[e] += f[e];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] += t[e];
    }
    if (in.plus) {
      join_floats<V>(in.plus + r * width + i, u);
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] += u[e];
    }
    if (in.step) {
      join_floats<V>(in.step + i, u);
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] += u[e];
    }
#pragma unroll
    for (int e = 0; e < V; ++e) {
      held[i + e] = v[e];
      squares += v[e] * v[e];
    }
    if (update) {
      if constexpr (V == 4) st4(x + i, make_float4(v[0], v[1], v[2], v[3]));
      else x[i] = v[0];
    }
  }
  squares = block_sum(squares, scratch);
  const float unit = 1.f / sqrtf(squares / (float)width + eps);
  T* y = out + (size_t)m * width;
  for (int i = threadIdx.x * V; i < width; i += blockDim.x * V) {      // (a thread meets its own elements again)
    if constexpr (V == 4) {
      const float4 w = ld4(weight + i);
      st4(y + i, make_float4(held[i] * unit * w.x, held[i + 1] * unit * w.y, held[i + 2] * unit * w.z, held[i + 3] * unit * w.w));
    } else {
      st(y + i, held[i] * unit * weight[i]);
    }
  }
}

extern "C" {

// a, b, f, gates: (pointer or null, code, splits, elements of a row); the split stride is total_rows times the row.
// out [n_out, width] of out_dtype.
int qil_residual_join(float* stream, const void* a, int a_code, int a_splits, int a_row, float a_scale, const void* b,
                      int b_code, int b_splits, int b_row, float b_scale, const void* f, int f_code, int f_splits, int f_row,
                      const void* gates, int g_code, int g_splits, int g_row, const float* bias, const float* plus,
                      const float* step, const int* rows, const float* weight, void* out, int n_out, int total_rows,
                      int width, float eps, int update, int out_dtype, hipStream_t s) {
  if (n_out == 0) return 0;
  if (width < 1 || !weight || !out || (b && !a) || (f && !a) || (gates && !bias) || (gates && !a)) return -1;
  const void* data[4] = {a, b, f, gates};
  const int codes[4] = {a_code, b_code, f_code, g_code}, splits[4] = {a_splits, b_splits, f_splits, g_splits};
  const int row[4] = {a_row, b_row, f_row, g_row};
  JoinInputs in;
  Operand* ops[4] = {&in.a, &in.b, &in.f, &in.gates};
  bool vec = width % 4 == 0;
  for (int k = 0; k < 4; ++k) {
    if (data[k] && (splits[k] < 1 || (codes[k] == QIL_BF16 && splits[k] != 1) || row[k] < (k == 3 && f ? 2 * width : width)))
      return -1;
    *ops[k] = Operand{data[k], codes[k], splits[k], (size_t)total_rows * row[k]};
    vec = vec && (!data[k] || (row[k] % 4 == 0 && (uintptr_t)data[k] % 16 == 0));
  }
  in.a_row = a_row; in.b_row = b_row; in.f_row = f_row; in.g_row = g_row;
  in.a_scale = a_scale; in.b_scale = b_scale;
  in.bias = bias; in.plus = plus; in.step = step;
  vec = vec && (((uintptr_t)stream | (uintptr_t)bias | (uintptr_t)plus | (uintptr_t)step | (uintptr_t)weight | (uintptr_t)out) % 16) == 0;
  const size_t lds = (size_t)width * sizeof(float);
  if (lds > 128 * 1024) return -1;
  const int lanes = vec ? width / 4 : width;
  const int threads = lanes >= 1024 ? 1024 : (lanes + 63) / 64 * 64;
#define QIL_JOIN(T, V)                                                                                               \
  do {                                                                                                               \
    if (lds > 60 * 1024) {                                                                                           \
      hipError_t e = hipFuncSetAttribute((const void*)residual_join_kernel<T, V>,                                    \
                                         hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                      \
      if (e != hipSuccess) return (int)e;                                                                            \
    }                                                                                                                \
    hipLaunchKernelGGL((residual_join_kernel<T, V>), dim3(n_out), dim3(threads), lds, s, stream, in, rows, weight,    \
                       (T*)out, width, eps, update);                                                                 \
  } while (0)
  if (out_dtype == QIL_F32) { if (vec) QIL_JOIN(float, 4); else QIL_JOIN(float, 1); }
  else { if (vec) QIL_JOIN(bf16_t, 4); else QIL_JOIN(bf16_t, 1); }
#undef QIL_JOIN
  QIL_RETURN_LAUNCH_STATUS();
}

}  // extern "C"
