// The recurrence with a step size per head and token (QIL_SCAN_STEP of recurrence.hip: S_t = a_t S_(t-1) + d_t k_t v_t^T,
// o_t = S_t^T q_t, a_t = exp(rate_h d_t), d_t = softplus(raw_t[h] + bias[h]), queries and keys shared by groups of heads),
// two forms of its own:
//
// 1. Long runs of tokens of a bfloat16 model, on the matrix cores, in blocks of STEP_L tokens worked on side by side.  With
// F_t the block's running sum of log2 a (float64) and S_in the state it starts from:
//     O^T[j, t] = 2^F_t sum_i S_in[i, j] q_t[i] + sum_(s <= t) x_s[j] (k_s . q_t) 2^(F_t - F_s) d_s
//     U^T[j, i] = sum_s (2^(F_end - F_s) d_s x_s[j]) k_s[i]        what the block adds to the state at its end
//   sums     every block's U and its decay 2^F_end;
//   carry    block after block, S_out = 2^F_end S_in + U; S_in replaces U, the last S_out goes to the state slot;
//   outputs  every block's O.
// q, k and x are bfloat16 numbers; what meets them in a product (the state, the weighted scores, the weighted x) is
// float32 and is taken apart into three bfloat16 numbers whose sum it is (8 + 8 + 8 bits), one matrix product each with
// float32 sums: nothing of the recurrence is rounded to less than 32 bits.  v_mfma_f32_16x16x32_bf16; the states lie
// transposed, [j][i], between the kernels, so that a lane's eight elements along i are 32 bytes in a row; x (and k for
// the sums) are transposed on their way into LDS; the scores are made as S^T = K Q^T with the rows of a score tile
// assigned to keys so that a lane ends up with eight consecutive keys of one query: the operand of the product with x.
//
// 2. One token a sequence (decoding): a block takes one (sequence, head), its lanes four columns each and every R-th row of
// the state, all loads in whole lines and ahead of their use.
#include "common.h"
#include "operand.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

#define STEP_L 128                                         // tokens a block
#define STEP_ROW (STEP_L + 8)                              // elements of a transposed row in LDS

struct StepGates {
  Operand raw;                                             // [n, row]: the raw step size of head h at column h
  int row;
  const float* bias;                                       // [heads]
  const float* rates;                                      // [heads], natural logarithm's units
};

__device__ __forceinline__ float step_size(const StepGates& g, int row, int h) {
  const float v = operand_at(g.raw, (size_t)row * g.row + h) + g.bias[h];
  return v > 20.f ? v : log1pf(expf(v));
}

// The first wave: F_t (log2 units) and d_t of the block's tokens into LDS; tokens past the end have d = 0 and F unchanged.
__device__ __forceinline__ void step_prefix(const StepGates& g, int r0, int lc, int h, int lane, double* F, float* d) {
  const double rate = (double)g.rates[h] * 1.4426950408889634;
  float mine[STEP_L / QIL_WAVE];
#pragma unroll
  for (int u = 0; u < STEP_L / QIL_WAVE; ++u) {
    const int t = lane + u * QIL_WAVE;
    mine[u] = t < lc ? step_size(g, r0 + t, h) : 0.f;
  }
  double before = 0.0;
#pragma unroll
  for (int u = 0; u < STEP_L / QIL_WAVE; ++u) {
    double sum = rate * (double)mine[u];
#pragma unroll
    for (int o = 1; o < QIL_WAVE; o <<= 1) {
      const double up = __shfl_up(sum, o, QIL_WAVE);
      if (lane >= o) sum += up;
    }
    sum += before;
    before = __shfl(sum, QIL_WAVE - 1, QIL_WAVE);
    F[lane + u * QIL_WAVE] = sum;
    d[lane + u * QIL_WAVE] = mine[u];
  }
}

// Eight float32 numbers as three bfloat16 each.
struct Split3 { bf16x8 part[3]; };
__device__ __forceinline__ Split3 split3(const float (&v)[8]) {
  uint32_t w[3][4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    float a = v[2 * e], b = v[2 * e + 1];
#pragma unroll
    for (int k = 0; k < 3; ++k) {
      w[k][e] = pack_bf16(a, b);
      a -= __uint_as_float(w[k][e] << 16);
      b -= __uint_as_float(w[k][e] & 0xffff0000u);
    }
  }
  Split3 s;
#pragma unroll
  for (int k = 0; k < 3; ++k) s.part[k] = __builtin_bit_cast(bf16x8, make_uint4(w[k][0], w[k][1], w[k][2], w[k][3]));
  return s;
}
__device__ __forceinline__ bf16x8 lds_fragment(const bf16_t* p) { return __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(p)); }

// Columns [first, first + 8 chunks) of the block's rows, transposed into LDS: to[column][token].  Two tokens at a time: a
// dword holds the same column of both.  Columns from `columns` on and tokens from lc on are zeros.
__device__ __forceinline__ void stage_transposed(const bf16_t* __restrict__ src, int src_row, int r0, int lc, int columns,
                                                 int chunks, bf16_t* __restrict__ to) {
  for (int item = threadIdx.x; item < chunks * (STEP_L / 2); item += blockDim.x) {
    const int chunk = (item & 7) + ((item >> 3) / (STEP_L / 2)) * 8, s = ((item >> 3) % (STEP_L / 2)) * 2;
    if (chunk >= chunks) continue;
    uint4 a = make_uint4(0, 0, 0, 0), b = make_uint4(0, 0, 0, 0);
    if (chunk * 8 < columns) {
      const bf16_t* p = src + (size_t)(r0 + s) * src_row + chunk * 8;
      if (s < lc) a = *reinterpret_cast<const uint4*>(p);
      if (s + 1 < lc) b = *reinterpret_cast<const uint4*>(p + src_row);
    }
    const uint32_t x[4] = {a.x, a.y, a.z, a.w}, y[4] = {b.x, b.y, b.z, b.w};
    uint32_t* out = reinterpret_cast<uint32_t*>(to + (size_t)chunk * 8 * STEP_ROW + s);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const uint32_t lo = (e & 1) ? x[e >> 1] >> 16 : x[e >> 1] & 0xffffu;
      const uint32_t hi = (e & 1) ? y[e >> 1] & 0xffff0000u : y[e >> 1] << 16;
      out[e * (STEP_ROW / 2)] = lo | hi;
    }
  }
}

// Where block c of sequence seq keeps its state: sequences before it took at most row0 / STEP_L + seq places.
__device__ __forceinline__ size_t step_place(int row0, int seq, int c) { return (size_t)(row0 / STEP_L + seq + c); }

// grid (blocks of the longest sequence, sequences x heads, value tiles of 64); NT: 16-row tiles of i a wave (dim <= 64 NT)
template <int NT>
__global__ void __launch_bounds__(256)
step_sums_kernel(const bf16_t* __restrict__ proj, int proj_row, int k_off, int v_off, StepGates gates,
                 const int* __restrict__ cu_seqlens, float* __restrict__ states, float* __restrict__ keeps, int heads,
                 int groups, int dim, int vdim) {
  extern __shared__ __align__(16) unsigned char lds_raw[];
  bf16_t* kT = reinterpret_cast<bf16_t*>(lds_raw);         // [NT * 64][STEP_ROW]
  bf16_t* xT = kT + NT * 64 * STEP_ROW;                    // [64][STEP_ROW]
  double* F = reinterpret_cast<double*>(xT + 64 * STEP_ROW);
  float* w = reinterpret_cast<float*>(F + STEP_L);
  const int c = blockIdx.x, seq = blockIdx.y / heads, h = blockIdx.y % heads, j0 = blockIdx.z * 64;
  const int row0 = cu_seqlens[seq], len = cu_seqlens[seq + 1] - row0;
  if (c * STEP_L >= len) return;
  const int r0 = row0 + c * STEP_L, lc = min(STEP_L, len - c * STEP_L);
  const int lane = threadIdx.x & (QIL_WAVE - 1), wave = threadIdx.x / QIL_WAVE, r = lane & 15, kb = lane >> 4;
  const int group = h / (heads / groups);
  const size_t at = step_place(row0, seq, c) * heads + h;
  if (wave == 0) {
    step_prefix(gates, r0, lc, h, lane, F, w);
    const double end = F[lc - 1];                          // (a wave's LDS operations are in order)
#pragma unroll
    for (int u = 0; u < STEP_L / QIL_WAVE; ++u) {
      const int t = lane + u * QIL_WAVE;
      w[t] *= exp2f((float)(end - F[t]));
    }
    if (lane == 0 && blockIdx.z == 0) keeps[at] = exp2f((float)end);
  }
  stage_transposed(proj + k_off + group * dim, proj_row, r0, lc, dim, NT * 8, kT);
  stage_transposed(proj + v_off + h * vdim + j0, proj_row, r0, lc, vdim - j0, 8, xT);
  __syncthreads();
  f32x4 acc[NT][4];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) acc[n][jt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int s0 = 0; s0 < lc; s0 += 32) {
    float ws[8];
    ld8(w + s0 + 8 * kb, ws);
    bf16x8 k[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) k[n] = lds_fragment(kT + ((wave * NT + n) * 16 + r) * STEP_ROW + s0 + 8 * kb);
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      float x[8];
      ld8(xT + (jt * 16 + r) * STEP_ROW + s0 + 8 * kb, x);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] *= ws[e];
      const Split3 xs = split3(x);
#pragma unroll
      for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int p = 0; p < 3; ++p) acc[n][jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[n], xs.part[p], acc[n][jt], 0, 0, 0);
    }
  }
  // lane: U[i = tile + 4 kb ..][j = jt * 16 + r]: four neighbours of a row [j][i]
  float* u = states + at * dim * vdim;
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int i = (wave * NT + n) * 16 + 4 * kb;
    if (i >= dim) continue;
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      const int j = j0 + jt * 16 + r;
      if (j < vdim) *reinterpret_cast<f32x4*>(u + (size_t)j * dim + i) = acc[n][jt];
    }
  }
}

// grid (sequences, heads, tiles of 32 i x 8 j): a thread an element, block after block.  The state slot is [i][j].
__global__ void __launch_bounds__(256)
step_carry_kernel(float* __restrict__ states, const float* __restrict__ keeps, float* __restrict__ slots, size_t slot_stride,
                  const int* __restrict__ cu_seqlens, const int* __restrict__ seq_starts, const int* __restrict__ seq_slots,
                  int heads, int dim, int vdim, int i_tiles) {
  __shared__ float tile[8][33];
  const int seq = blockIdx.x, h = blockIdx.y, i0 = (blockIdx.z % i_tiles) * 32, j0 = (blockIdx.z / i_tiles) * 8;
  const int row0 = cu_seqlens[seq], len = cu_seqlens[seq + 1] - row0;
  if (len <= 0) return;
  float* mine = slots + (size_t)seq_slots[seq] * slot_stride + (size_t)h * dim * vdim;
  const int si = i0 + (int)threadIdx.x / 8, sj = j0 + (int)threadIdx.x % 8;      // as the slot lies
  const int i = i0 + (int)threadIdx.x % 32, j = j0 + (int)threadIdx.x / 32;      // as the states between blocks lie
  const bool there = si < dim && sj < vdim, live = i < dim && j < vdim;
  tile[threadIdx.x % 8][threadIdx.x / 8] = (there && seq_starts[seq] > 0) ? mine[(size_t)si * vdim + sj] : 0.f;
  __syncthreads();
  float value = tile[threadIdx.x / 32][threadIdx.x % 32];
  const int blocks = (len + STEP_L - 1) / STEP_L;
  const size_t first = step_place(row0, seq, 0) * heads + h, stride = (size_t)heads * dim * vdim;
  float* u = states + first * dim * vdim + (size_t)j * dim + i;
  for (int c0 = 0; c0 < blocks; c0 += 4) {                 // four blocks' loads first
    float add[4], keep[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int c = min(c0 + k, blocks - 1);
      add[k] = live ? u[c * stride] : 0.f;
      keep[k] = keeps[first + (size_t)c * heads];
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (c0 + k < blocks) {
        if (live) u[(c0 + k) * stride] = value;
        value = keep[k] * value + add[k];
      }
    }
  }
  __syncthreads();
  tile[threadIdx.x / 32][threadIdx.x % 32] = value;
  __syncthreads();
  if (there) mine[(size_t)si * vdim + sj] = tile[threadIdx.x % 8][threadIdx.x / 8];
}

// grid (blocks of the longest sequence, sequences x heads, value tiles of 64); dim <= 32 NF.  A wave owns the 16-token
// tiles `wave` and 7 - wave: the early one has few keys, the late one many.
template <int NF>
__global__ void __launch_bounds__(256)
step_outputs_kernel(const bf16_t* __restrict__ proj, int proj_row, int q_off, int k_off, int v_off, StepGates gates,
                    const int* __restrict__ cu_seqlens, const float* __restrict__ states, float* __restrict__ out, int heads,
                    int groups, int dim, int vdim) {
  constexpr int K_ROW = NF * 32 + 8;
  extern __shared__ __align__(16) unsigned char lds_raw[];
  bf16_t* Ks = reinterpret_cast<bf16_t*>(lds_raw);         // [STEP_L][K_ROW]
  bf16_t* xT = Ks + STEP_L * K_ROW;                        // [64][STEP_ROW]
  double* F = reinterpret_cast<double*>(xT + 64 * STEP_ROW);
  float* d = reinterpret_cast<float*>(F + STEP_L);
  const int c = blockIdx.x, seq = blockIdx.y / heads, h = blockIdx.y % heads, j0 = blockIdx.z * 64;
  const int row0 = cu_seqlens[seq], len = cu_seqlens[seq + 1] - row0;
  if (c * STEP_L >= len) return;
  const int r0 = row0 + c * STEP_L, lc = min(STEP_L, len - c * STEP_L);
  const int lane = threadIdx.x & (QIL_WAVE - 1), wave = threadIdx.x / QIL_WAVE, r = lane & 15, kb = lane >> 4;
  const int group = h / (heads / groups);
  const bf16_t* keys = proj + k_off + group * dim;
  const bf16_t* queries = proj + q_off + group * dim;
  const int tiles[2] = {wave, 7 - wave};
  bf16x8 q[2][NF];
#pragma unroll
  for (int b = 0; b < 2; ++b)
#pragma unroll
    for (int ks = 0; ks < NF; ++ks) {
      const int t = tiles[b] * 16 + r, i = ks * 32 + 8 * kb;
      uint4 raw = make_uint4(0, 0, 0, 0);
      if (t < lc && i < dim) raw = *reinterpret_cast<const uint4*>(queries + (size_t)(r0 + t) * proj_row + i);
      q[b][ks] = __builtin_bit_cast(bf16x8, raw);
    }
  for (int item = threadIdx.x; item < STEP_L * NF * 4; item += 256) {
    const int s = item / (NF * 4), i = item % (NF * 4) * 8;
    uint4 raw = make_uint4(0, 0, 0, 0);
    if (s < lc && i < dim) raw = *reinterpret_cast<const uint4*>(keys + (size_t)(r0 + s) * proj_row + i);
    *reinterpret_cast<uint4*>(Ks + s * K_ROW + i) = raw;
  }
  stage_transposed(proj + v_off + h * vdim + j0, proj_row, r0, lc, vdim - j0, 8, xT);
  if (wave == 0) step_prefix(gates, r0, lc, h, lane, F, d);
  f32x4 o[2][4];
#pragma unroll
  for (int b = 0; b < 2; ++b)
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) o[b][jt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // what came in: rows j of S_in^T (float32, taken apart) with the queries
  const float* s_in = states + (step_place(row0, seq, c) * heads + h) * dim * vdim;
#pragma unroll
  for (int ks = 0; ks < NF; ++ks) {
    const int i = ks * 32 + 8 * kb;
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      const int j = j0 + jt * 16 + r;
      float v[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = 0.f;
      if (i < dim && j < vdim) ld8(s_in + (size_t)j * dim + i, v);
      const Split3 s = split3(v);
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int p = 0; p < 3; ++p) o[b][jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(s.part[p], q[b][ks], o[b][jt], 0, 0, 0);
    }
  }
  __syncthreads();
#pragma unroll
  for (int b = 0; b < 2; ++b) {
    const int t = tiles[b] * 16 + r;
    const double mine = F[t];
    const float brought = exp2f((float)mine);
#pragma unroll
    for (int jt = 0; jt < 4; ++jt)
#pragma unroll
      for (int e = 0; e < 4; ++e) o[b][jt][e] *= brought;
    if (tiles[b] * 16 >= lc) continue;
    for (int s0 = 0; s0 <= tiles[b] * 16 + 15; s0 += 32) {
      f32x4 score[2];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        score[half] = (f32x4){0.f, 0.f, 0.f, 0.f};
        const bf16_t* row = Ks + (s0 + 8 * (r >> 2) + 4 * half + (r & 3)) * K_ROW + 8 * kb;
#pragma unroll
        for (int ks = 0; ks < NF; ++ks)
          score[half] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds_fragment(row + ks * 32), q[b][ks], score[half], 0, 0, 0);
      }
      float p[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int s = s0 + 8 * kb + e;
        p[e] = s <= t ? score[e >> 2][e & 3] * exp2f((float)(mine - F[s])) * d[s] : 0.f;
      }
      const Split3 ps = split3(p);
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        const bf16x8 x = lds_fragment(xT + (jt * 16 + r) * STEP_ROW + s0 + 8 * kb);
#pragma unroll
        for (int k = 0; k < 3; ++k) o[b][jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, ps.part[k], o[b][jt], 0, 0, 0);
      }
    }
    if (t < lc) {
      float* row = out + (size_t)(r0 + t) * heads * vdim + (size_t)h * vdim;
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        const int j = j0 + jt * 16 + 4 * kb;
        if (j < vdim) *reinterpret_cast<f32x4*>(row + j) = o[b][jt];
      }
    }
  }
}

// One token a sequence.  grid (sequences, heads), 256 threads: thread (c, g) takes the columns 4 c .. 4 c + 3 and the rows
// g, g + R, ... of the head's state, C = vdim / 4 lanes across, R = 256 / C rows at a time.
#define STEP_AHEAD 8
template <typename T>
__global__ void __launch_bounds__(256)
step_token_kernel(const T* __restrict__ proj, int proj_row, int q_off, int k_off, int v_off, StepGates gates,
                  float* __restrict__ slots, size_t slot_stride, const int* __restrict__ cu_seqlens,
                  const int* __restrict__ seq_starts, const int* __restrict__ seq_slots, float* __restrict__ out, int heads,
                  int groups, int dim, int vdim, int c_log2) {
  __shared__ float ks[256], qs[256];
  __shared__ __align__(16) float sums[4][256];             // a wave's sums by column
  const int seq = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int row = cu_seqlens[seq], C = 1 << c_log2, R = 256 >> c_log2;
  const int c = tid & (C - 1), g = tid >> c_log2, lane = tid & (QIL_WAVE - 1), wave = tid / QIL_WAVE;
  const bool fresh = seq_starts[seq] == 0;
  float* s_mat = slots + (size_t)seq_slots[seq] * slot_stride + (size_t)h * dim * vdim + 4 * c;
  float4 s[STEP_AHEAD];
  auto request = [&](int i0) {
#pragma unroll
    for (int u = 0; u < STEP_AHEAD; ++u) {
      const int i = i0 + g + u * R;
      s[u] = (!fresh && i < dim) ? ld4(s_mat + (size_t)i * vdim) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
  };
  request(0);
  const int group = h / (heads / groups);
  const T* mine = proj + (size_t)row * proj_row;
  if (tid < dim) {
    ks[tid] = ld(mine + k_off + group * dim + tid);
    qs[tid] = ld(mine + q_off + group * dim + tid);
  }
  const float step = step_size(gates, row, h), keep = expf(gates.rates[h] * step);
  const T* x = mine + v_off + h * vdim + 4 * c;
  const float v[4] = {step * ld(x), step * ld(x + 1), step * ld(x + 2), step * ld(x + 3)};
  __syncthreads();
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  for (int i0 = 0; i0 < dim; i0 += STEP_AHEAD * R) {
    if (i0 > 0) request(i0);
#pragma unroll
    for (int u = 0; u < STEP_AHEAD; ++u) {
      const int i = i0 + g + u * R;
      if (i < dim) {
        const float k = ks[i], q = qs[i];
        const float4 n = make_float4(keep * s[u].x + k * v[0], keep * s[u].y + k * v[1], keep * s[u].z + k * v[2],
                                     keep * s[u].w + k * v[3]);
        st4(s_mat + (size_t)i * vdim, n);
        o.x += n.x * q; o.y += n.y * q; o.z += n.z * q; o.w += n.w * q;
      }
    }
  }
  for (int m = C; m < QIL_WAVE; m <<= 1) {                 // the row groups of a wave, then the waves
    o.x += __shfl_xor(o.x, m, QIL_WAVE); o.y += __shfl_xor(o.y, m, QIL_WAVE);
    o.z += __shfl_xor(o.z, m, QIL_WAVE); o.w += __shfl_xor(o.w, m, QIL_WAVE);
  }
  if (lane < C) st4(&sums[wave][4 * c], o);
  __syncthreads();
  if (tid < vdim) out[(size_t)row * heads * vdim + (size_t)h * vdim + tid] = sums[0][tid] + sums[1][tid] + sums[2][tid] + sums[3][tid];
}

extern "C" {

// 1 if form 1 (bfloat16 rows, many tokens) takes the sizes: offsets and sizes in whole pieces of 8 elements.
int qil_step_scan_takes(int proj_row, int q_off, int k_off, int v_off, int dim, int vdim) {
  return dim >= 8 && dim <= 256 && dim % 8 == 0 && vdim >= 8 && vdim % 8 == 0 && proj_row % 8 == 0 && q_off % 8 == 0 &&
         k_off % 8 == 0 && v_off % 8 == 0;
}
// 1 if form 2 (one token a sequence) does: a power of two of columns' quadruples, up to 64.
int qil_step_token_takes(int dim, int vdim) {
  return dim >= 1 && dim <= 256 && vdim >= 4 && vdim <= 256 && (vdim & (vdim - 1)) == 0;
}

// Floats of form 1's scratch memory.
size_t qil_step_scan_workspace(int n, int n_seqs, int heads, int dim, int vdim) {
  const size_t places = (size_t)n / STEP_L + n_seqs;
  return places * heads * dim * vdim + places * heads;
}

// proj [n, proj_row] bfloat16 (values at v_off + h * vdim, keys at k_off + group * dim, queries at q_off + group * dim); raw: an
// operand of rows of raw_row elements (split stride n * raw_row); bias, rates float32 [heads]; state float32
// [slots][heads * dim * vdim]; out float32 [n, heads * vdim].
int qil_step_scan(const void* proj, int proj_row, int q_off, int k_off, int v_off, const void* raw, int raw_code,
                  int raw_splits, int raw_row, const float* bias, const float* rates, float* state, const int* cu_seqlens,
                  const int* seq_starts, const int* seq_slots, float* out, float* workspace, int n, int n_seqs, int max_query,
                  int heads, int groups, int dim, int vdim, hipStream_t s) {
  if (n == 0 || n_seqs == 0) return 0;
  if (!qil_step_scan_takes(proj_row, q_off, k_off, v_off, dim, vdim) || !raw || !bias || !rates || !state || !workspace ||
      groups < 1 || heads % groups || raw_splits < 1 || (raw_code == QIL_BF16 && raw_splits != 1) || raw_row < heads ||
      max_query < 1 || (size_t)n_seqs * heads > 65535 || (((uintptr_t)proj | (uintptr_t)workspace | (uintptr_t)out) % 16))
    return -1;
  const size_t places = (size_t)n / STEP_L + n_seqs;
  float* states = workspace;
  float* keeps = workspace + places * heads * dim * vdim;
  const StepGates gates{{raw, raw_code, raw_splits, (size_t)n * raw_row}, raw_row, bias, rates};
  const int blocks = (max_query + STEP_L - 1) / STEP_L, v_tiles = (vdim + 63) / 64;
  const dim3 grid(blocks, n_seqs * heads, v_tiles);
  const size_t tail = STEP_L * (sizeof(double) + sizeof(float));
#define QIL_STEP_SUMS(NT)                                                                                             \
  do {                                                                                                                \
    const size_t lds = (size_t)(NT + 1) * 64 * STEP_ROW * sizeof(bf16_t) + tail;                                      \
    if (lds > 64 * 1024) {                                                                                            \
      hipError_t e = hipFuncSetAttribute((const void*)step_sums_kernel<NT>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                         (int)lds);                                                                   \
      if (e != hipSuccess) return (int)e;                                                                             \
    }                                                                                                                 \
    hipLaunchKernelGGL(step_sums_kernel<NT>, grid, dim3(256), lds, s, (const bf16_t*)proj, proj_row, k_off, v_off,     \
                       gates, cu_seqlens, states, keeps, heads, groups, dim, vdim);                                   \
  } while (0)
  if (dim <= 64) QIL_STEP_SUMS(1);
  else if (dim <= 128) QIL_STEP_SUMS(2);
  else QIL_STEP_SUMS(4);
#undef QIL_STEP_SUMS
  const int i_tiles = (dim + 31) / 32, j_tiles = (vdim + 7) / 8;
  hipLaunchKernelGGL(step_carry_kernel, dim3(n_seqs, heads, i_tiles * j_tiles), dim3(256), 0, s, states, keeps, state,
                     (size_t)heads * dim * vdim, cu_seqlens, seq_starts, seq_slots, heads, dim, vdim, i_tiles);
#define QIL_STEP_OUT(NF)                                                                                              \
  do {                                                                                                                \
    const size_t lds = ((size_t)STEP_L * (NF * 32 + 8) + 64 * STEP_ROW) * sizeof(bf16_t) + tail;                      \
    if (lds > 64 * 1024) {                                                                                            \
      hipError_t e = hipFuncSetAttribute((const void*)step_outputs_kernel<NF>,                                        \
                                         hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                       \
      if (e != hipSuccess) return (int)e;                                                                             \
    }                                                                                                                 \
    hipLaunchKernelGGL(step_outputs_kernel<NF>, grid, dim3(256), lds, s, (const bf16_t*)proj, proj_row, q_off, k_off,  \
                       v_off, gates, cu_seqlens, states, out, heads, groups, dim, vdim);                              \
  } while (0)
  if (dim <= 32) QIL_STEP_OUT(1);
  else if (dim <= 64) QIL_STEP_OUT(2);
  else if (dim <= 128) QIL_STEP_OUT(4);
  else QIL_STEP_OUT(8);
#undef QIL_STEP_OUT
  QIL_RETURN_LAUNCH_STATUS();
}

// One token a sequence (row cu_seqlens[i] of the step is sequence i's).  proj of dtype; the rest as above.
int qil_step_token(const void* proj, int dtype, int proj_row, int q_off, int k_off, int v_off, const void* raw, int raw_code,
                   int raw_splits, int raw_row, const float* bias, const float* rates, float* state, const int* cu_seqlens,
                   const int* seq_starts, const int* seq_slots, float* out, int n, int n_seqs, int heads, int groups, int dim,
                   int vdim, hipStream_t s) {
  if (n == 0 || n_seqs == 0) return 0;
  if (!qil_step_token_takes(dim, vdim) || n != n_seqs || !raw || !bias || !rates || !state || groups < 1 || heads % groups ||
      heads > 65535 || raw_splits < 1 || (raw_code == QIL_BF16 && raw_splits != 1) || raw_row < heads ||
      ((uintptr_t)state % 16))
    return -1;
  int c_log2 = 0;
  while ((4 << c_log2) < vdim) ++c_log2;
  const StepGates gates{{raw, raw_code, raw_splits, (size_t)n * raw_row}, raw_row, bias, rates};
  const size_t slot_stride = (size_t)heads * dim * vdim;
  if (dtype == QIL_F32)
    hipLaunchKernelGGL(step_token_kernel<float>, dim3(n_seqs, heads), dim3(256), 0, s, (const float*)proj, proj_row, q_off,
                       k_off, v_off, gates, state, slot_stride, cu_seqlens, seq_starts, seq_slots, out, heads, groups, dim,
                       vdim, c_log2);
  else
    hipLaunchKernelGGL(step_token_kernel<bf16_t>, dim3(n_seqs, heads), dim3(256), 0, s, (const bf16_t*)proj, proj_row, q_off,
                       k_off, v_off, gates, state, slot_stride, cu_seqlens, seq_starts, seq_slots, out, heads, groups, dim,
                       vdim, c_log2);
  QIL_RETURN_LAUNCH_STATUS();
}

}  // extern "C"
