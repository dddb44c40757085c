// Several residual streams side by side (hyper-connections): what a sub-layer leaves joins all streams, the next
// sub-layer's input is made from them, and the norm by a hyperbolic tangent is applied, in one kernel:
//     x_t <- sum_s mix[s, t] x_s + out[t] y          for all t at once from the old x   (if there is a y)
//     u = sum_s read[s] x_s
//     result = tanh(alpha u) w + b                    (without an alpha: u)
// The streams of a row lie one behind another, float32 [rows][streams][width].  y is an array of the model's type, float32
// partial sums (operand.h), or the experts' rows of a routed feed-forward with their weights (the weighted sum is made
// here).  A single stream without a mix is the ordinary residual sum x + y with that norm.  Everything is float32 until
// the one rounding of the result; no element depends on another of its row, so a thread takes V neighbouring channels of
// one row and nothing is shared.
#include "common.h"
#include "operand.h"

struct StreamValue {
  Operand y;                                               // data null: nothing joins
  size_t row;                                              // elements between two rows of y
  const float* pairs;                                      // routed: [rows * top][width] float32, or null
  const float* weights;                                    // [rows * top]
  const int* chosen;                                       // [rows * top]; an index from `experts` on passes the input x
  const void* x;                                           // [rows][width] of x_code
  int x_code, top, experts;
};

template <int V> __device__ __forceinline__ void stream_load(const float* p, float (&v)[V]) {
  if constexpr (V == 4) {
    const float4 q = ld4(p);
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
  } else {
    v[0] = p[0];
  }
}
template <int V> __device__ __forceinline__ void stream_store(float* p, const float (&v)[V]) {
  if constexpr (V == 4) st4(p, make_float4(v[0], v[1], v[2], v[3]));
  else p[0] = v[0];
}
template <int V> __device__ __forceinline__ void stream_operand(const Operand& x, size_t at, float (&v)[V]) {
  if constexpr (V == 4) {
    const float4 q = operand_at4(x, at);
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
  } else {
    v[0] = operand_at(x, at);
  }
}

// S: most streams (registers); the actual number is `streams`.
template <typename T, int V, int S, bool ROUTED>
__global__ void __launch_bounds__(256)
stream_join_kernel(float* __restrict__ x, int streams, StreamValue in, const float* __restrict__ mix,
                   const float* __restrict__ out_weights, const float* __restrict__ read, const int* __restrict__ rows,
                   const float* __restrict__ alpha, const float* __restrict__ w, const float* __restrict__ b,
                   T* __restrict__ result, size_t items, int per_row, int update) {
  const size_t item = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (item >= items) return;
  const size_t m = item / per_row;
  const int c = (int)(item - m * per_row) * V, width = per_row * V;
  const size_t r = rows ? (size_t)rows[m] : m;
  float* mine = x + r * streams * width + c;
  float v[S][V];
#pragma unroll
  for (int s = 0; s < S; ++s)
    if (s < streams) stream_load<V>(mine + (size_t)s * width, v[s]);
  if (ROUTED || in.y.data) {
    float y[V];
    if constexpr (ROUTED) {
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] = 0.f;
      for (int slot = 0; slot < in.top; ++slot) {          // in slot order
        const size_t pair = r * in.top + slot;
        float t[V];
        if (in.chosen[pair] >= in.experts) {
          const Operand plain{in.x, in.x_code, 1, 0};
          stream_operand<V>(plain, r * width + c, t);
        } else {
          stream_load<V>(in.pairs + pair * width + c, t);
        }
        const float f = in.weights[pair];
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] += f * t[e];
      }
    } else {
      stream_operand<V>(in.y, r * in.row + c, y);
    }
    float fresh[S][V];
#pragma unroll
    for (int t = 0; t < S; ++t) {
      if (t < streams) {
        const float o = out_weights ? out_weights[t] : 1.f;
#pragma unroll
        for (int e = 0; e < V; ++e) fresh[t][e] = o * y[e];
        if (mix) {
#pragma unroll
          for (int s = 0; s < S; ++s)
            if (s < streams) {
              const float f = mix[s * streams + t];
#pragma unroll
              for (int e = 0; e < V; ++e) fresh[t][e] += f * v[s][e];
            }
        } else {
#pragma unroll
          for (int e = 0; e < V; ++e) fresh[t][e] += v[t][e];
        }
        if (update) stream_store<V>(mine + (size_t)t * width, fresh[t]);
      }
    }
#pragma unroll
    for (int s = 0; s < S; ++s)
      if (s < streams)
#pragma unroll
        for (int e = 0; e < V; ++e) v[s][e] = fresh[s][e];
  }
  float u[V];
#pragma unroll
  for (int e = 0; e < V; ++e) u[e] = 0.f;
#pragma unroll
  for (int s = 0; s < S; ++s)
    if (s < streams) {
      const float f = read ? read[s] : 1.f;
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] += f * v[s][e];
    }
  if (alpha) {
    const float a = alpha[0];
    float wv[V], bv[V];
    stream_load<V>(w + c, wv);
    stream_load<V>(b + c, bv);
#pragma unroll
    for (int e = 0; e < V; ++e) u[e] = tanhf(a * u[e]) * wv[e] + bv[e];
  }
  T* to = result + m * width + c;
  if constexpr (V == 4) st4(to, make_float4(u[0], u[1], u[2], u[3]));
  else st(to, u[0]);
}

// stream[n][k][:] = float(table[token[n], :]) * scale for every k < copies
template <typename T, int V>
__global__ void embed_streams_kernel(const int* __restrict__ tokens, const T* __restrict__ table, float* __restrict__ out,
                                     size_t items, int per_row, int copies, float scale) {
  const size_t item = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (item >= items) return;
  const size_t n = item / per_row;
  const int c = (int)(item - n * per_row) * V, width = per_row * V;
  const T* row = table + (size_t)tokens[n] * width + c;
  float v[V];
  if constexpr (V == 4) {
    const float4 q = ld4(row);
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
  } else {
    v[0] = ld(row);
  }
#pragma unroll
  for (int e = 0; e < V; ++e) v[e] *= scale;
  for (int k = 0; k < copies; ++k) stream_store<V>(out + (n * copies + k) * width + c, v);
}

#define QIL_MOST_STREAMS 16

extern "C" {

int qil_stream_join_takes(int streams) { return streams >= 1 && streams <= QIL_MOST_STREAMS; }

// x float32 [total_rows, streams, width]; y (null: nothing joins): an operand of rows of y_row elements (split stride
// total_rows * y_row); pairs (or null): float32 [total_rows * top, width] with weights and chosen, x_in [total_rows, width]
// of result_dtype.  mix [streams, streams] (from, to) and out_weights, read [streams], float32, each null for the
// identity or ones.  alpha float32 [1] or null.  rows int32 [count] or null (count == total_rows).  result [count, width].
int qil_stream_join(float* x, int streams, const void* y, int y_code, int y_splits, int y_row, const float* pairs,
                    const float* weights, const int* chosen, const void* x_in, int top, int experts, const float* mix,
                    const float* out_weights, const float* read, const int* rows, const float* alpha, const float* w,
                    const float* b, void* result, int count, int total_rows, int width, int update, int result_dtype,
                    hipStream_t s) {
  if (count == 0) return 0;
  if (!qil_stream_join_takes(streams) || width < 1 || !x || !result || (y && pairs) || (alpha && (!w || !b)) ||
      (rows && update) || (y && (y_splits < 1 || (y_code == QIL_BF16 && y_splits != 1) || y_row < width)) ||
      (pairs && (!weights || !chosen || top < 1 || !x_in)))
    return -1;
  StreamValue in;
  in.y = Operand{y, y_code, y_splits, (size_t)total_rows * y_row};
  in.row = y_row;
  in.pairs = pairs; in.weights = weights; in.chosen = chosen; in.x = x_in;
  in.x_code = result_dtype; in.top = top; in.experts = experts;
  const bool vec = width % 4 == 0 && (!y || y_row % 4 == 0) &&
                   (((uintptr_t)x | (uintptr_t)y | (uintptr_t)pairs | (uintptr_t)x_in | (uintptr_t)w | (uintptr_t)b | (uintptr_t)result) % 16) == 0;
  const int per_row = vec ? width / 4 : width;
  const size_t items = (size_t)count * per_row;
  const int threads = items >= 65536 ? 256 : 64;           // few rows: more blocks, so more CUs ask for memory at a time
  const dim3 grid((unsigned)((items + threads - 1) / threads));
#define QIL_SJ(T, V, S, R)                                                                                            \
  hipLaunchKernelGGL((stream_join_kernel<T, V, S, R>), grid, dim3(threads), 0, s, x, streams, in, mix, out_weights,     \
                     read, rows, alpha, w, b, (T*)result, items, per_row, update)
#define QIL_SJ_R(T, V, S) do { if (pairs) QIL_SJ(T, V, S, true); else QIL_SJ(T, V, S, false); } while (0)
#define QIL_SJ_S(T, V)                                                                                                \
  do {                                                                                                                \
    if (streams == 1) QIL_SJ_R(T, V, 1);                                                                              \
    else if (streams == 2) QIL_SJ_R(T, V, 2);                                                                         \
    else if (streams <= 4) QIL_SJ_R(T, V, 4);                                                                         \
    else QIL_SJ_R(T, V, QIL_MOST_STREAMS);                                                                            \
  } while (0)
  if (result_dtype == QIL_F32) { if (vec) QIL_SJ_S(float, 4); else QIL_SJ_S(float, 1); }
  else { if (vec) QIL_SJ_S(bf16_t, 4); else QIL_SJ_S(bf16_t, 1); }
#undef QIL_SJ_S
#undef QIL_SJ_R
#undef QIL_SJ
  QIL_RETURN_LAUNCH_STATUS();
}

// The embedding into every stream: out float32 [n, copies, width].
int qil_embed_streams(const int* tokens, const void* table, float* out, int n, int width, int copies, float scale, int dtype,
                      hipStream_t s) {
  if (n == 0) return 0;
  if (width < 1 || copies < 1) return -1;
  const bool vec = width % 4 == 0 && (((uintptr_t)table | (uintptr_t)out) % 16) == 0;
  const int per_row = vec ? width / 4 : width;
  const size_t items = (size_t)n * per_row;
  const dim3 grid((unsigned)((items + 255) / 256));
#define QIL_ES(T, V)                                                                                                  \
  hipLaunchKernelGGL((embed_streams_kernel<T, V>), grid, dim3(256), 0, s, tokens, (const T*)table, out, items, per_row, \
                     copies, scale)
  if (dtype == QIL_F32) { if (vec) QIL_ES(float, 4); else QIL_ES(float, 1); }
  else { if (vec) QIL_ES(bf16_t, 4); else QIL_ES(bf16_t, 1); }
#undef QIL_ES
  QIL_RETURN_LAUNCH_STATUS();
}

}  // extern "C"
