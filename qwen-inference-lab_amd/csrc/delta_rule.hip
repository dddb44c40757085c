// The gated delta rule with a decay per key channel.  Per head a state S [dim, vdim] in float32; with k and q unit vectors
// (q also times dim^(-1/2)), a step size beta in (0, 1) and decays g [dim] of the token:
//     S <- diag(g) S;   w = beta (v - S^T k);   S <- S + k w^T;   o = S^T q
// g_c = exp(rate_h softplus(raw_c + bias_c)), beta = sigmoid(raw).  Everything from the raw numbers on is float32.
//
// This file: token by token, the state in registers from the first token of the step to its last (decoding, short
// portions, sizes the matrix-core form does not take), and the norm and gate that follow.  A state's columns do not
// depend on one another: a block takes one (sequence, head) and up to 256 columns, its threads C lanes along the columns (VW
// neighbours each) and R row groups; the two sums over rows a token needs go through LDS.
#include "delta_rule.h"

#define DELTA_THREADS 512

struct DeltaEnd {                                          // the output's norm and gate, when a block holds whole heads
  const float* weight;                                     // [vdim]
  Operand gate;                                            // [n, gate_row]: logits, column head * vdim + j
  int gate_row;
  float eps;
};

template <typename T, int VW, int U, bool ENDED>
__global__ void __launch_bounds__(DELTA_THREADS)
delta_tokens_kernel(DeltaInputs in, DeltaEnd end, float* __restrict__ slots, const int* __restrict__ cu_seqlens,
                    const int* __restrict__ seq_starts, const int* __restrict__ seq_slots, float* __restrict__ raw_out,
                    T* __restrict__ out, int heads, int kv_heads, int dim, int vdim) {
  __shared__ float ks[256], qs[256], gs[256], wv[256], sums[DELTA_THREADS * VW];
  __shared__ float squares[2][4], norm_squares[4];
  const int seq = blockIdx.x, h = blockIdx.y, j0 = blockIdx.z * 256, cols = min(256, vdim - j0), tid = threadIdx.x;
  const int row0 = cu_seqlens[seq], len = cu_seqlens[seq + 1] - row0;
  if (len <= 0) return;
  const int C = (cols + VW - 1) / VW, R = DELTA_THREADS / C, c = tid % C, g = tid / C;
  const int lane = tid & (QIL_WAVE - 1), wave = tid / QIL_WAVE;
  const bool member = g < R;
  const bool fresh = seq_starts[seq] == 0;
  float* mine = slots + ((size_t)seq_slots[seq] * heads + h) * dim * vdim + j0 + c * VW;
  float s[U][VW];
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int i = g + u * R;
    const bool there = member && i < dim && !fresh;
    if constexpr (VW == 4) {
      const float4 v = there ? ld4(mine + (size_t)i * vdim) : make_float4(0.f, 0.f, 0.f, 0.f);
      s[u][0] = v.x; s[u][1] = v.y; s[u][2] = v.z; s[u][3] = v.w;
    } else {
      s[u][0] = there ? mine[(size_t)i * vdim] : 0.f;
    }
  }
  const int shared_head = h / (heads / kv_heads);
  for (int t = 0; t < len; ++t) {
    const int row = row0 + t;
    const T* x = reinterpret_cast<const T*>(in.u) + (size_t)row * in.u_row;
    if (wave < 4) {
      float k = 0.f, q = 0.f;
      if (tid < dim) {
        k = ld(x + in.k_off + shared_head * dim + tid);
        q = ld(x + in.q_off + shared_head * dim + tid);
        ks[tid] = k;
        qs[tid] = q;
        gs[tid] = expf(delta_log_decay(in, row, h, dim, tid));
      }
      const float kk = wave_sum(k * k), qq = wave_sum(q * q);
      if (lane == 0) { squares[0][wave] = kk; squares[1][wave] = qq; }
    }
    const float beta = delta_step_size(in, row, h);
    const float v = tid < cols ? ld(x + in.v_off + h * vdim + j0 + tid) : 0.f;
    float gate = 0.f;
    if constexpr (ENDED) gate = tid < cols ? operand_at(end.gate, (size_t)row * end.gate_row + h * vdim + tid) : 0.f;
    __syncthreads();
    const float k_unit = 1.f / sqrtf(squares[0][0] + squares[0][1] + squares[0][2] + squares[0][3] + DELTA_UNIT_EPS);
    const float q_unit = 1.f / sqrtf(squares[1][0] + squares[1][1] + squares[1][2] + squares[1][3] + DELTA_UNIT_EPS) / sqrtf((float)dim);
    float acc[VW];
#pragma unroll
    for (int e = 0; e < VW; ++e) acc[e] = 0.f;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int i = g + u * R;
      if (i < dim) {
        const float keep = gs[i], k = ks[i];
#pragma unroll
        for (int e = 0; e < VW; ++e) {
          s[u][e] *= keep;
          acc[e] += s[u][e] * k;
        }
      }
    }
    if (member) {
#pragma unroll
      for (int e = 0; e < VW; ++e) sums[(g * C + c) * VW + e] = acc[e];
    }
    __syncthreads();
    if (tid < cols) {
      float total = 0.f;
      for (int p = 0; p < R; ++p) total += sums[p * C * VW + tid];
      wv[tid] = beta * (v - total * k_unit) * k_unit;
    }
    __syncthreads();
    float w[VW];
#pragma unroll
    for (int e = 0; e < VW; ++e) {
      w[e] = c * VW + e < cols ? wv[c * VW + e] : 0.f;
      acc[e] = 0.f;
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int i = g + u * R;
      if (i < dim) {
        const float k = ks[i], q = qs[i];
#pragma unroll
        for (int e = 0; e < VW; ++e) {
          s[u][e] += k * w[e];
          acc[e] += s[u][e] * q;
        }
      }
    }
    if (member) {
#pragma unroll
      for (int e = 0; e < VW; ++e) sums[(g * C + c) * VW + e] = acc[e];
    }
    __syncthreads();
    float o = 0.f;
    if (tid < cols) {
      for (int p = 0; p < R; ++p) o += sums[p * C * VW + tid];
      o *= q_unit;
    }
    if constexpr (ENDED) {
      if (wave < 4) {
        const float oo = wave_sum(o * o);
        if (lane == 0) norm_squares[wave] = oo;
      }
      __syncthreads();
      if (tid < cols) {
        const float mean = (norm_squares[0] + norm_squares[1] + norm_squares[2] + norm_squares[3]) / (float)vdim;
        st(out + ((size_t)row * heads + h) * vdim + tid, o / sqrtf(mean + end.eps) * end.weight[tid] / (1.f + expf(-gate)));
      }
    } else {
      if (tid < cols) raw_out[((size_t)row * heads + h) * vdim + j0 + tid] = o;
    }
  }
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int i = g + u * R;
    if (member && i < dim) {
      if constexpr (VW == 4) st4(mine + (size_t)i * vdim, make_float4(s[u][0], s[u][1], s[u][2], s[u][3]));
      else mine[(size_t)i * vdim] = s[u][0];
    }
  }
}

// out = o / sqrt(mean(o^2) + eps) * weight * sigmoid(gate), per row and head over vdim; a wave a (row, head).
template <typename T, int V>
__global__ void __launch_bounds__(256)
delta_end_kernel(const float* __restrict__ o, DeltaEnd end, T* __restrict__ out, int items, int heads, int vdim) {
  const int item = blockIdx.x * (256 / QIL_WAVE) + threadIdx.x / QIL_WAVE, lane = threadIdx.x & (QIL_WAVE - 1);
  if (item >= items) return;
  const int row = item / heads, h = item - row * heads;
  const float* mine = o + (size_t)item * vdim;
  const size_t gate_at = (size_t)row * end.gate_row + (size_t)h * vdim;
  float squares = 0.f;
  float held[V], gates[V];                                 // the first round's elements, used again below
#pragma unroll
  for (int e = 0; e < V; ++e) { held[e] = 0.f; gates[e] = 0.f; }
  for (int i = lane * V; i < vdim; i += QIL_WAVE * V) {
    float v[V], g[V];
    if constexpr (V == 4) {
      const float4 a = ld4(mine + i), b = operand_at4(end.gate, gate_at + i);
      v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
      g[0] = b.x; g[1] = b.y; g[2] = b.z; g[3] = b.w;
    } else {
      v[0] = mine[i];
      g[0] = operand_at(end.gate, gate_at + i);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) squares += v[e] * v[e];
    if (i == lane * V) {
#pragma unroll
      for (int e = 0; e < V; ++e) { held[e] = v[e]; gates[e] = g[e]; }
    }
  }
  const float unit = 1.f / sqrtf(wave_sum(squares) / (float)vdim + end.eps);
  T* to = out + (size_t)item * vdim;
  for (int i = lane * V; i < vdim; i += QIL_WAVE * V) {
    float v[V], g[V], y[V];
#pragma unroll
    for (int e = 0; e < V; ++e) { v[e] = held[e]; g[e] = gates[e]; }
    if (i != lane * V) {
      if constexpr (V == 4) {
        const float4 a = ld4(mine + i), b = operand_at4(end.gate, gate_at + i);
        v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
        g[0] = b.x; g[1] = b.y; g[2] = b.z; g[3] = b.w;
      } else {
        v[0] = mine[i];
        g[0] = operand_at(end.gate, gate_at + i);
      }
    }
#pragma unroll
    for (int e = 0; e < V; ++e) y[e] = v[e] * unit * end.weight[i + e] / (1.f + expf(-g[e]));
    if constexpr (V == 4) st4(to + i, make_float4(y[0], y[1], y[2], y[3]));
    else st(to + i, y[0]);
  }
}

static bool bad_operand(const void* p, int code, int splits, int row, int columns) {
  return !p || splits < 1 || (code == QIL_BF16 && splits != 1) || row < columns;
}

extern "C" {

int qil_delta_takes(int dim, int vdim) { return dim >= 1 && dim <= 256 && vdim >= 1 && (vdim + 255) / 256 <= 65535; }
// Whether one block holds a head's whole output, so that the norm and the gate can end the token kernel.
int qil_delta_ends(int vdim) { return vdim <= 256; }

// u [n, u_row] of dtype (queries from column q_off, keys from k_off: kv_heads * dim each; values from v_off: heads * vdim); z, b,
// gate: operands of rows of z_row, b_row, gate_row elements (split strides n * row).  state float32 [slots, heads, dim,
// vdim].  Sequences 0 .. n_seqs - 1 of the tables given.  out (with weight and gate): [n, heads * vdim] of dtype, normed and
// gated; or raw_out float32 [n, heads * vdim], neither.
int qil_delta_tokens(const void* u, int dtype, int u_row, int q_off, int k_off, int v_off, const void* z, int z_code, int z_splits,
                     int z_row, const float* bias, const float* rates, const void* b, int b_code, int b_splits, int b_row,
                     float* state, const int* cu_seqlens, const int* seq_starts, const int* seq_slots, float* raw_out, void* out,
                     const float* weight, const void* gate, int gate_code, int gate_splits, int gate_row, float eps, int n,
                     int n_seqs, int heads, int kv_heads, int dim, int vdim, hipStream_t s) {
  if (n == 0 || n_seqs == 0) return 0;
  if (!qil_delta_takes(dim, vdim) || heads < 1 || heads > 65535 || kv_heads < 1 || heads % kv_heads || !u || !bias || !rates || !state ||
      bad_operand(z, z_code, z_splits, z_row, heads * dim) || bad_operand(b, b_code, b_splits, b_row, heads) ||
      (!out) == (!raw_out) || (out && (!qil_delta_ends(vdim) || !weight || bad_operand(gate, gate_code, gate_splits, gate_row, heads * vdim))) ||
      q_off < 0 || k_off < 0 || v_off < 0 || q_off + kv_heads * dim > u_row || k_off + kv_heads * dim > u_row || v_off + heads * vdim > u_row)
    return -1;
  const DeltaInputs in{u, u_row, q_off, k_off, v_off, Operand{z, z_code, z_splits, (size_t)n * z_row}, z_row, bias, rates,
                       Operand{b, b_code, b_splits, (size_t)n * b_row}, b_row};
  const DeltaEnd end{weight, Operand{gate, gate_code, gate_splits, (size_t)n * gate_row}, gate_row, eps};
  const int cols = vdim < 256 ? vdim : 256;
  const int vw = vdim % 4 == 0 && (uintptr_t)state % 16 == 0 ? 4 : 1;
  const int C = (cols + vw - 1) / vw, R = DELTA_THREADS / C, rows = (dim + R - 1) / R;
  const dim3 grid(n_seqs, heads, (vdim + 255) / 256);
#define QIL_DT(T, VW, U)                                                                                              \
  do {                                                                                                                \
    if (out)                                                                                                          \
      hipLaunchKernelGGL((delta_tokens_kernel<T, VW, U, true>), grid, dim3(DELTA_THREADS), 0, s, in, end, state,       \
                         cu_seqlens, seq_starts, seq_slots, (float*)nullptr, (T*)out, heads, kv_heads, dim, vdim);     \
    else                                                                                                              \
      hipLaunchKernelGGL((delta_tokens_kernel<T, VW, U, false>), grid, dim3(DELTA_THREADS), 0, s, in, end, state,      \
                         cu_seqlens, seq_starts, seq_slots, raw_out, (T*)nullptr, heads, kv_heads, dim, vdim);         \
  } while (0)
#define QIL_DT_U(T)                                                                                                   \
  do {                                                                                                                \
    if (vw == 4) {                                                                                                    \
      if (rows <= 4) QIL_DT(T, 4, 4);                                                                                 \
      else if (rows <= 8) QIL_DT(T, 4, 8);                                                                            \
      else if (rows <= 16) QIL_DT(T, 4, 16);                                                                          \
      else QIL_DT(T, 4, 32);                                                                                          \
    } else {                                                                                                          \
      if (rows <= 32) QIL_DT(T, 1, 32);                                                                               \
      else QIL_DT(T, 1, 128);                                                                                         \
    }                                                                                                                 \
  } while (0)
  if (dtype == QIL_F32) QIL_DT_U(float); else QIL_DT_U(bf16_t);
#undef QIL_DT_U
#undef QIL_DT
  QIL_RETURN_LAUNCH_STATUS();
}

// The norm and gate alone: o float32 [n, heads * vdim] -> out of dtype.
int qil_delta_end(const float* o, const float* weight, const void* gate, int gate_code, int gate_splits, int gate_row, float eps,
                  void* out, int n, int heads, int vdim, int dtype, hipStream_t s) {
  if (n == 0) return 0;
  if (!o || !weight || !out || heads < 1 || vdim < 1 || bad_operand(gate, gate_code, gate_splits, gate_row, heads * vdim)) return -1;
  const DeltaEnd end{weight, Operand{gate, gate_code, gate_splits, (size_t)n * gate_row}, gate_row, eps};
  const bool vec = vdim % 4 == 0 && gate_row % 4 == 0 && (((uintptr_t)o | (uintptr_t)gate | (uintptr_t)out) % 16) == 0;
  const int items = n * heads;
  const dim3 grid((items + 3) / 4);
#define QIL_DE(T, V) hipLaunchKernelGGL((delta_end_kernel<T, V>), grid, dim3(256), 0, s, o, end, (T*)out, items, heads, vdim)
  if (dtype == QIL_F32) { if (vec) QIL_DE(float, 4); else QIL_DE(float, 1); }
  else { if (vec) QIL_DE(bf16_t, 4); else QIL_DE(bf16_t, 1); }
#undef QIL_DE
  QIL_RETURN_LAUNCH_STATUS();
}

}  // extern "C"
