// The gated delta rule with a decay per key channel (delta_rule.hip) over long runs of tokens: chunks of 64 tokens on the
// matrix cores, v_mfma_f32_16x16x4_f32, whose operands, products and sums are float32.
//
// With the log decays summed from the chunk's start, G_t, and the state S the chunk starts from, the tokens' writes w solve
// a triangular system (beta_t, unit vectors k_t, q_t; products of vectors channel by channel):
//     w_t + sum_(s < t) A_ts w_s = beta_t (v_t - S^T (k_t e^(G_t))),     A_ts = beta_t sum_c k_tc k_sc e^(G_tc - G_sc)
//     o_t = S^T (q_t e^(G_t)) + sum_(s <= t) B_ts w_s,                   B_ts = sum_c q_tc k_sc e^(G_tc - G_sc)
//     S  <- e^(G_end) S + sum_t (k_t e^(G_end - G_t)) w_t^T
// The system is linear in what the state does not touch, so w = U - W S with (I + A) U = beta v and (I + A) W = beta k e^G.
//   prepare  all chunks side by side: A, B, the solution of both systems, and the other operands, into scratch memory;
//   walk     chunk after chunk, a block 16 columns of the state (they do not depend on one another).
// Every exponent is of a sum of log decays over later minus earlier tokens, at most zero: nothing overflows, whatever the decays.
// A chunk is four blocks of 16 tokens.  Between blocks an exponent is split at the later block's start (both parts are at
// most zero) and A and B are matrix products; inside a block every pair's exponential is taken by itself.  The triangular
// system goes block by block: the 16 x 16 diagonal blocks of I + A are inverted, a column a lane.
//
// The operands lie in the scratch memory tile by tile as the lanes of the walk hold them (64 lanes x 4 floats, a kilobyte in a
// row): a load of 16 rows by 16 bytes would occupy the address path for 64 cycles, four times what the tile's product takes.
// The layout trick throughout: a result tile holds rows 4 kb + e and column r in lane 16 kb + r; as the next product's
// right operand, whose k-step e then stands for the rows 4 kb + e, it needs no move, and the left operand's 4 neighbouring
// elements a lane are one 16-byte load.
#include "delta_rule.h"

typedef float f32x4 __attribute__((ext_vector_type(4)));

#define DC_L 64                                            // tokens a chunk
#define DC_THREADS 512
#define DC_BLOCK 256                                       // floats of a 16 x 16 block in LDS

// Where row i, column j of such a block lies: rows of 16 floats, their pieces of four turned so that the 16 rows a fragment
// read touches fall on all banks.
__device__ __forceinline__ int dc_in_block(int i, int j) { return i * 16 + ((((j >> 2) ^ (i >> 2)) & 3) << 2) + (j & 3); }

__device__ __forceinline__ f32x4 dc_ld(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 dc_ld(const bf16_t* p) { const float4 v = ld4(p); return (f32x4){v.x, v.y, v.z, v.w}; }
__device__ __forceinline__ f32x4 dc_mma(const f32x4& a, const f32x4& b, f32x4 acc) {
#pragma unroll
  for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], acc, 0, 0, 0);
  return acc;
}
__device__ __forceinline__ float dc_exp2(float v) { return __builtin_amdgcn_exp2f(v); }

// ln(1 + e^v) = max(v, 0) + ln(1 + t), t = e^(-|v|), with the hardware's exponential and logarithm; a small t by its series (the
// logarithm of 1 + t would lose it).
__device__ __forceinline__ float dc_softplus(float v) {
  const float t = dc_exp2(-fabsf(v) * 1.44269504088896f);
  const float series = t * (1.f - t * (0.5f - t * (0.33333333f - t * 0.25f)));
  return fmaxf(v, 0.f) + (t < 0.015f ? series : __builtin_amdgcn_logf(1.f + t) * 0.69314718055995f);
}

// A barrier for what went through LDS: the waves' loads from memory stay on their way (the compiler's barrier would wait
// for them as well).
__device__ __forceinline__ void dc_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// Element (row i, column j) of a left operand's tile.
__device__ __forceinline__ int dc_in_operand(int i, int j) { return (i + 16 * (j >> 2)) * 4 + (j & 3); }

// Where chunk c of sequence seq keeps its operands: sequences before it took at most row0 / DC_L + seq places.
__device__ __forceinline__ size_t dc_place(int row0, int seq, int c) { return (size_t)(row0 / DC_L + seq + c); }

// Floats of one (place, head), in tiles: W (negated) and Q [4 token blocks][DP / 16], K^T [DP / 16][4], U [VP / 16][4] (result
// tiles), B [4][4], and the decay e^(G_end) [DP].
__host__ __device__ __forceinline__ size_t dc_cell(int dp, int vp) { return (size_t)3 * DC_L * dp + DC_L * vp + DC_L * DC_L + dp; }

// grid (chunks of the longest sequence, sequences x heads), 8 waves.
template <typename T, int DP>
__global__ void __launch_bounds__(DC_THREADS, DP <= 128 ? 4 : 2)
delta_prepare_kernel(DeltaInputs in, const int* __restrict__ cu_seqlens, float* __restrict__ scratch, int heads, int kv_heads,
                     int dim, int vdim, int vp) {
  constexpr int KROW = DP + 16 / (int)sizeof(T), LROW = DP + 4;
  extern __shared__ __align__(16) unsigned char lds_raw[];
  float* L = reinterpret_cast<float*>(lds_raw);            // [64][LROW] log2 decays summed from the token's block's start
  T* ks = reinterpret_cast<T*>(L + DC_L * LROW);           // [64][KROW]
  T* qs = ks + DC_L * KROW;
  float* A = reinterpret_cast<float*>(qs + DC_L * KROW);   // [10] blocks of -A (b >= j: b (b + 1) / 2 + j), the diagonal ones then inverted
  float* units = A + 10 * DC_BLOCK;                   // [3][64]: 1 / |k|, dim^(-1/2) / |q|, beta
  const int c = blockIdx.x, seq = blockIdx.y / heads, h = blockIdx.y % heads;
  const int row0 = cu_seqlens[seq], len = cu_seqlens[seq + 1] - row0;
  if (c * DC_L >= len) return;
  const int r0 = row0 + c * DC_L, lc = min(DC_L, len - c * DC_L);
  const int tid = threadIdx.x, lane = tid & (QIL_WAVE - 1), wave = tid / QIL_WAVE, r = lane & 15, kb = lane >> 4;
  const int shared_head = h / (heads / kv_heads);
  float* cell = scratch + (dc_place(row0, seq, c) * heads + h) * dc_cell(DP, vp);
  float* W = cell;
  float* Q = W + DC_L * DP;
  float* KT = Q + DC_L * DP;
  float* Uo = KT + DC_L * DP;
  float* B = Uo + DC_L * vp;
  float* end = B + DC_L * DC_L;
  const T* u = reinterpret_cast<const T*>(in.u);
  {                                                        // queries and keys into LDS, and their lengths: 8 threads a token
    const int t = tid >> 3, part = tid & 7;
    const T* x = u + (size_t)(r0 + min(t, lc - 1)) * in.u_row;
    const T* k = x + in.k_off + shared_head * dim;
    const T* q = x + in.q_off + shared_head * dim;
    float kk = 0.f, qq = 0.f;
    constexpr int PIECES = DP / 32;
    float4 kv[PIECES], qv[PIECES];
    if (dim % 4 == 0) {                                    // (the host checked that rows and offsets are multiples of 4)
#pragma unroll
      for (int n = 0; n < PIECES; ++n) {
        const int e0 = min(part * 4 + n * 32, dim - 4);
        kv[n] = ld4(k + e0);
        qv[n] = ld4(q + e0);
      }
    } else {
#pragma unroll
      for (int n = 0; n < PIECES; ++n) {
        float v[2][4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int at = part * 4 + n * 32 + e;
          v[0][e] = at < dim ? ld(k + at) : 0.f;
          v[1][e] = at < dim ? ld(q + at) : 0.f;
        }
        kv[n] = make_float4(v[0][0], v[0][1], v[0][2], v[0][3]);
        qv[n] = make_float4(v[1][0], v[1][1], v[1][2], v[1][3]);
      }
    }
#pragma unroll
    for (int n = 0; n < PIECES; ++n) {
      const int e0 = part * 4 + n * 32;
      if (t >= lc || e0 >= dim) kv[n] = qv[n] = make_float4(0.f, 0.f, 0.f, 0.f);
      st4(ks + t * KROW + e0, kv[n]);
      st4(qs + t * KROW + e0, qv[n]);
      kk += kv[n].x * kv[n].x + kv[n].y * kv[n].y + kv[n].z * kv[n].z + kv[n].w * kv[n].w;
      qq += qv[n].x * qv[n].x + qv[n].y * qv[n].y + qv[n].z * qv[n].z + qv[n].w * qv[n].w;
    }
#pragma unroll
    for (int o = 1; o < 8; o <<= 1) { kk += __shfl_xor(kk, o, QIL_WAVE); qq += __shfl_xor(qq, o, QIL_WAVE); }
    if (part == 0) {
      units[t] = 1.f / sqrtf(kk + DELTA_UNIT_EPS);
      units[DC_L + t] = 1.f / sqrtf(qq + DELTA_UNIT_EPS) / sqrtf((float)dim);
      units[2 * DC_L + t] = t < lc ? delta_step_size(in, r0 + t, h) : 0.f;
    }
  }
  for (int item = tid; item < DP * 4; item += DC_THREADS) {    // a thread a channel and block of 16 tokens, all loads first
    const int ch = item % DP, b = item / DP, own = min(ch, dim - 1);
    float raw[16], sum = 0.f;
    const size_t first = (size_t)r0 * in.z_row + h * dim + own;
    int at[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) at[t] = min(b * 16 + t, lc - 1) * in.z_row;
    if (in.z.code == QIL_BF16) {
      const bf16_t* base = reinterpret_cast<const bf16_t*>(in.z.data) + first;
#pragma unroll
      for (int t = 0; t < 16; ++t) raw[t] = ld(base + at[t]);
    } else {
      const float* base = reinterpret_cast<const float*>(in.z.data) + first;
#pragma unroll
      for (int t = 0; t < 16; ++t) raw[t] = base[at[t]];
      for (int split = 1; split < in.z.splits; ++split) {
        base += in.z.stride;
#pragma unroll
        for (int t = 0; t < 16; ++t) raw[t] += base[at[t]];
      }
    }
    const float bias = in.bias[h * dim + own], rate = in.rates[h] * 1.44269504088896f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      if (ch < dim && b * 16 + t < lc) sum += rate * dc_softplus(raw[t] + bias);
      L[(b * 16 + t) * LROW + ch] = sum;
    }
  }
  __syncthreads();
  // inside the blocks of 16: wave (block, half of its columns); a lane two pairs (row i, columns j, j + 1)
  {
    const int b = wave >> 1, i = b * 16 + r, j = b * 16 + 8 * (wave & 1) + 2 * kb;
    float kk[2] = {0.f, 0.f}, qk[2] = {0.f, 0.f};
    if (i >= j) {
      for (int ch = 0; ch < DP; ch += 4) {
        const f32x4 li = dc_ld(L + i * LROW + ch), ki = dc_ld(ks + i * KROW + ch), qi = dc_ld(qs + i * KROW + ch);
#pragma unroll
        for (int p = 0; p < 2; ++p) {
          const f32x4 lj = dc_ld(L + (j + p) * LROW + ch), kj = dc_ld(ks + (j + p) * KROW + ch);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float t = kj[e] * dc_exp2(fminf(li[e] - lj[e], 0.f));
            kk[p] += ki[e] * t;
            qk[p] += qi[e] * t;
          }
        }
      }
    }
    float* a = A + (b * (b + 1) / 2 + b) * DC_BLOCK;
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const float uk = units[j + p];
      a[dc_in_block(r, j + p - b * 16)] = i > j + p ? -kk[p] * units[i] * uk * units[2 * DC_L + i] : 0.f;
      B[(b * 4 + b) * DC_BLOCK + dc_in_operand(r, j + p - b * 16)] = i >= j + p ? qk[p] * units[DC_L + i] * uk : 0.f;
    }
  }
  // between blocks: waves 0 .. 5 a pair (later block bi, earlier block bj) each
  if (wave < 6) {
    const int bi = wave < 1 ? 1 : wave < 3 ? 2 : 3, bj = wave - bi * (bi - 1) / 2;
    f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
    for (int ch = 4 * kb; ch < DP; ch += 16) {
      const int i = bi * 16 + r, j = bj * 16 + r;
      const f32x4 li = dc_ld(L + i * LROW + ch), lj = dc_ld(L + j * LROW + ch);
      f32x4 upto = dc_ld(L + (bj * 16 + 15) * LROW + ch) - lj;
      for (int m = bj + 1; m < bi; ++m) upto += dc_ld(L + (m * 16 + 15) * LROW + ch);
      f32x4 ki = dc_ld(ks + i * KROW + ch), qi = dc_ld(qs + i * KROW + ch), kj = dc_ld(ks + j * KROW + ch);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float d = dc_exp2(li[e]);
        ki[e] *= d;
        qi[e] *= d;
        kj[e] *= dc_exp2(fminf(upto[e], 0.f));
      }
      kk = dc_mma(ki, kj, kk);
      qk = dc_mma(qi, kj, qk);
    }
    float* a = A + (bi * (bi + 1) / 2 + bj) * DC_BLOCK;
    const float uk = units[bj * 16 + r];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = bi * 16 + 4 * kb + e;
      a[dc_in_block(4 * kb + e, r)] = -kk[e] * units[i] * uk * units[2 * DC_L + i];
      B[(bi * 4 + bj) * DC_BLOCK + dc_in_operand(4 * kb + e, r)] = qk[e] * units[DC_L + i] * uk;
    }
  }
  __syncthreads();
  if (wave < 4) {                                          // (I + A_bb)^(-1), a column a lane: x_i = delta_ij - sum_(m < i) A_im x_m
    float* a = A + (wave * (wave + 1) / 2 + wave) * DC_BLOCK;
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == r ? 1.f : 0.f;
#pragma unroll
      for (int m0 = 0; m0 < i; m0 += 4) {
        const f32x4 row = dc_ld(a + dc_in_block(i, m0));
#pragma unroll
        for (int m = m0; m < i && m < m0 + 4; ++m) v += row[m - m0] * x[m];
      }
      x[i] = v;
    }
    // (a wave's LDS operations are in order: every lane has read the block before any lane writes it)
    if (lane < 16) {
#pragma unroll
      for (int i = 0; i < 16; ++i) a[dc_in_block(i, r)] = x[i];
    }
  }
  __syncthreads();
  // both systems, 16 columns a wave at a time: W's, then U's
  for (int tile = wave; tile < DP / 16 + vp / 16; tile += DC_THREADS / QIL_WAVE) {
    const bool is_w = tile < DP / 16;
    const int col = is_w ? tile * 16 + r : (tile - DP / 16) * 16 + r;
    f32x4 x[4];
    float before = 0.f;
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      f32x4 acc;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = b * 16 + 4 * kb + e;
        float v;
        if (is_w) v = ld(ks + t * KROW + col) * units[t] * dc_exp2(before + L[t * LROW + col]);
        else v = t < lc && col < vdim ? ld(u + (size_t)(r0 + t) * in.u_row + in.v_off + h * vdim + col) : 0.f;
        acc[e] = v * units[2 * DC_L + t];
      }
      if (is_w) before += L[(b * 16 + 15) * LROW + col];
#pragma unroll
      for (int j = 0; j < b; ++j) acc = dc_mma(dc_ld(A + (b * (b + 1) / 2 + j) * DC_BLOCK + dc_in_block(r, 4 * kb)), x[j], acc);
      x[b] = dc_mma(dc_ld(A + (b * (b + 1) / 2 + b) * DC_BLOCK + dc_in_block(r, 4 * kb)), acc, (f32x4){0.f, 0.f, 0.f, 0.f});
      if (is_w) {
#pragma unroll
        for (int e = 0; e < 4; ++e) W[(b * (DP / 16) + tile) * DC_BLOCK + dc_in_operand(4 * kb + e, r)] = -x[b][e];
      } else {
        *reinterpret_cast<f32x4*>(Uo + (((tile - DP / 16) * 4 + b) * 64 + lane) * 4) = x[b];
      }
    }
  }
  // the queries with their decays from the chunk's start, the keys with theirs to its end (transposed): a wave a channel tile
  for (int n = wave; n < DP / 16; n += DC_THREADS / QIL_WAVE) {
    f32x4 before = {0.f, 0.f, 0.f, 0.f};
    const int ch = n * 16 + 4 * kb;
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const int t = b * 16 + r;
      const f32x4 from = before + dc_ld(L + t * LROW + ch);
      f32x4 q = dc_ld(qs + t * KROW + ch);
#pragma unroll
      for (int e = 0; e < 4; ++e) q[e] *= units[DC_L + t] * dc_exp2(from[e]);
      *reinterpret_cast<f32x4*>(Q + ((b * (DP / 16) + n) * 64 + lane) * 4) = q;
      before += dc_ld(L + (b * 16 + 15) * LROW + ch);
    }
    float after = 0.f;
#pragma unroll
    for (int b = 3; b >= 0; --b) {
      const float whole = L[(b * 16 + 15) * LROW + n * 16 + r];
      f32x4 k;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = b * 16 + 4 * kb + e;
        k[e] = ld(ks + t * KROW + n * 16 + r) * units[t] * dc_exp2(fminf(after + whole - L[t * LROW + n * 16 + r], 0.f));
      }
      *reinterpret_cast<f32x4*>(KT + ((n * 4 + b) * 64 + lane) * 4) = k;
      after += whole;
    }
  }
  for (int ch = tid; ch < DP; ch += DC_THREADS)
    end[ch] = dc_exp2(L[15 * LROW + ch] + L[31 * LROW + ch] + L[47 * LROW + ch] + L[63 * LROW + ch]);
}

// grid (sequences x heads, column tiles of 16), 4 waves.  Wave w makes the writes and outputs of token block w and the
// state's channel tiles w, w + 4, ..; the state is held in registers by its owners and in LDS for everyone.
template <int DT>
__global__ void __launch_bounds__(256)
delta_walk_kernel(const float* __restrict__ scratch, float* __restrict__ slots, const int* __restrict__ cu_seqlens,
                  const int* __restrict__ seq_starts, const int* __restrict__ seq_slots, float* __restrict__ out, int heads,
                  int dim, int vdim, int vp) {
  constexpr int DP = DT * 16, OWN = DT / 4;
  __shared__ __align__(16) float S[DT * 256];              // [tile][lane][4]: a result tile as its lanes hold it
  __shared__ __align__(16) float V[4 * 256];
  const int seq = blockIdx.x / heads, h = blockIdx.x % heads, j0 = blockIdx.y * 16;
  const int row0 = cu_seqlens[seq], len = cu_seqlens[seq + 1] - row0;
  if (len <= 0) return;
  const int lane = threadIdx.x & (QIL_WAVE - 1), wave = __builtin_amdgcn_readfirstlane(threadIdx.x / QIL_WAVE);
  const int r = lane & 15, kb = lane >> 4;
  const bool column = j0 + r < vdim;
  float* mine = slots + ((size_t)seq_slots[seq] * heads + h) * dim * vdim + j0 + r;
  const bool fresh = seq_starts[seq] == 0;
  f32x4 s[OWN];
#pragma unroll
  for (int n = 0; n < OWN; ++n) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int ch = (wave + 4 * n) * 16 + 4 * kb + e;
      s[n][e] = column && ch < dim && !fresh ? mine[(size_t)ch * vdim] : 0.f;
    }
    *reinterpret_cast<f32x4*>(S + ((wave + 4 * n) * 64 + lane) * 4) = s[n];
  }
  const size_t cell = dc_cell(DP, vp), stride = cell * heads;
  const float* at = scratch + (dc_place(row0, seq, 0) * heads + h) * cell;
  const int chunks = (len + DC_L - 1) / DC_L;
  // this chunk's operands; each is asked for again, for the next chunk, as soon as it has been used
  f32x4 w[DT], q[DT], b[4], k[OWN][4], keep[OWN], write;
  auto load_w = [&](const float* p) {
#pragma unroll
    for (int n = 0; n < DT; ++n) w[n] = dc_ld(p + ((wave * DT + n) * 64 + lane) * 4);
    write = dc_ld(p + 3 * DC_L * DP + (((j0 >> 4) * 4 + wave) * 64 + lane) * 4);
  };
  auto load_q = [&](const float* p) {
#pragma unroll
    for (int n = 0; n < DT; ++n) q[n] = dc_ld(p + DC_L * DP + ((wave * DT + n) * 64 + lane) * 4);
    const float* bo = p + 3 * DC_L * DP + DC_L * vp;
#pragma unroll
    for (int j = 0; j < 4; ++j) b[j] = dc_ld(bo + ((wave * 4 + j) * 64 + lane) * 4);   // (nobody wrote or uses those of j > wave)
  };
  auto load_k = [&](const float* p) {
    const float* eo = p + 3 * DC_L * DP + DC_L * vp + DC_L * DC_L;
#pragma unroll
    for (int n = 0; n < OWN; ++n) {
#pragma unroll
      for (int j = 0; j < 4; ++j) k[n][j] = dc_ld(p + 2 * DC_L * DP + (((wave + 4 * n) * 4 + j) * 64 + lane) * 4);
      keep[n] = dc_ld(eo + (wave + 4 * n) * 16 + 4 * kb);
    }
  };
  load_w(at);
  load_q(at);
  load_k(at);
  dc_barrier();
  for (int c = 0; c < chunks; ++c) {
    const float* next = at + (c + 1 < chunks ? stride : 0);
    f32x4 acc = write, acc2 = {0.f, 0.f, 0.f, 0.f};        // w = U - W S (two sums: the products of one wait for each other)
#pragma unroll
    for (int n = 0; n < DT; n += 2) {
      acc = dc_mma(w[n], dc_ld(S + (n * 64 + lane) * 4), acc);
      acc2 = dc_mma(w[n + 1], dc_ld(S + ((n + 1) * 64 + lane) * 4), acc2);
    }
    acc += acc2;
    *reinterpret_cast<f32x4*>(V + (wave * 64 + lane) * 4) = acc;
    load_w(next);
    f32x4 o = {0.f, 0.f, 0.f, 0.f}, o2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int n = 0; n < DT; n += 2) {                      // what the state brings: before the other waves' writes are needed
      o = dc_mma(q[n], dc_ld(S + (n * 64 + lane) * 4), o);
      o2 = dc_mma(q[n + 1], dc_ld(S + ((n + 1) * 64 + lane) * 4), o2);
    }
    dc_barrier();
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wave) o = dc_mma(b[j], dc_ld(V + (j * 64 + lane) * 4), o);
    o += o2;
    load_q(next);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = c * DC_L + wave * 16 + 4 * kb + e;
      if (column && t < len) out[((size_t)(row0 + t) * heads + h) * vdim + j0 + r] = o[e];
    }
#pragma unroll
    for (int n = 0; n < OWN; ++n) s[n] *= keep[n];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const f32x4 v = dc_ld(V + (j * 64 + lane) * 4);
#pragma unroll
      for (int n = 0; n < OWN; ++n) s[n] = dc_mma(k[n][j], v, s[n]);
    }
    load_k(next);
#pragma unroll
    for (int n = 0; n < OWN; ++n) *reinterpret_cast<f32x4*>(S + ((wave + 4 * n) * 64 + lane) * 4) = s[n];   // (read before the barrier)
    dc_barrier();
    at = next;
  }
#pragma unroll
  for (int n = 0; n < OWN; ++n)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int ch = (wave + 4 * n) * 16 + 4 * kb + e;
      if (column && ch < dim) mine[(size_t)ch * vdim] = s[n][e];
    }
}

static int dc_padded(int dim) { return dim <= 64 ? 64 : dim <= 128 ? 128 : 256; }
static size_t dc_lds(int dp, int dtype) {
  const size_t element = dtype == QIL_F32 ? 4 : 2;
  return (size_t)DC_L * (dp + 4) * 4 + 2 * (size_t)DC_L * (dp + 16 / element) * element + 10 * DC_BLOCK * 4 + 3 * DC_L * 4;
}

extern "C" {

// 1 if the chunked form takes the sizes (an LDS block holds a chunk's keys, queries and decays).
int qil_delta_chunked_takes(int dim, int vdim, int u_row, int q_off, int k_off, int dtype) {
  return dim >= 1 && dim <= 256 && vdim >= 1 && vdim <= 65536 && dc_lds(dc_padded(dim), dtype) <= 160 * 1024 &&
         (dim % 4 != 0 || (u_row % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0));
}
// Floats of scratch memory.
size_t qil_delta_chunked_workspace(int n, int n_seqs, int heads, int dim, int vdim) {
  return ((size_t)n / DC_L + n_seqs) * heads * dc_cell(dc_padded(dim), (vdim + 15) / 16 * 16);
}

// As qil_delta_tokens, for sequences 0 .. n_seqs - 1 of at most max_query rows each; raw_out float32 [n, heads * vdim].
int qil_delta_chunked(const void* u, int dtype, int u_row, int q_off, int k_off, int v_off, const void* z, int z_code, int z_splits,
                      int z_row, const float* bias, const float* rates, const void* b, int b_code, int b_splits, int b_row,
                      float* state, const int* cu_seqlens, const int* seq_starts, const int* seq_slots, float* raw_out,
                      float* scratch, int n, int n_seqs, int max_query, int heads, int kv_heads, int dim, int vdim, hipStream_t s) {
  if (n == 0 || n_seqs == 0) return 0;
  if (!qil_delta_chunked_takes(dim, vdim, u_row, q_off, k_off, dtype) || heads < 1 || kv_heads < 1 || heads % kv_heads || !u || !z ||
      !b || !bias || !rates || !state || !raw_out || !scratch || z_splits < 1 || b_splits < 1 ||
      (z_code == QIL_BF16 && z_splits != 1) || (b_code == QIL_BF16 && b_splits != 1) || z_row < heads * dim || b_row < heads ||
      max_query < 1 || (size_t)n_seqs * heads > 65535 || ((uintptr_t)u % 16) || ((uintptr_t)scratch % 16) || q_off < 0 || k_off < 0 ||
      v_off < 0 || q_off + kv_heads * dim > u_row || k_off + kv_heads * dim > u_row || v_off + heads * vdim > u_row)
    return -1;
  const DeltaInputs in{u, u_row, q_off, k_off, v_off, Operand{z, z_code, z_splits, (size_t)n * z_row}, z_row, bias, rates,
                       Operand{b, b_code, b_splits, (size_t)n * b_row}, b_row};
  const int dp = dc_padded(dim), vp = (vdim + 15) / 16 * 16;
  const size_t lds = dc_lds(dp, dtype);
  const dim3 grid((max_query + DC_L - 1) / DC_L, n_seqs * heads), walk(n_seqs * heads, vp / 16);
#define QIL_DCP(T, DP)                                                                                                \
  do {                                                                                                                \
    static bool granted = false;                                                                                      \
    if (!granted && lds > 64 * 1024) {                                                                                \
      hipError_t e = hipFuncSetAttribute((const void*)delta_prepare_kernel<T, DP>,                                    \
                                         hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                       \
      if (e != hipSuccess) return (int)e;                                                                             \
      granted = true;                                                                                                 \
    }                                                                                                                 \
    hipLaunchKernelGGL((delta_prepare_kernel<T, DP>), grid, dim3(DC_THREADS), lds, s, in, cu_seqlens, scratch, heads,  \
                       kv_heads, dim, vdim, vp);                                                                      \
  } while (0)
  if (dtype == QIL_F32) {
    if (dp == 64) QIL_DCP(float, 64);
    else QIL_DCP(float, 128);
  } else {
    if (dp == 64) QIL_DCP(bf16_t, 64);
    else if (dp == 128) QIL_DCP(bf16_t, 128);
    else QIL_DCP(bf16_t, 256);
  }
#undef QIL_DCP
#define QIL_DCW(DT)                                                                                                   \
  hipLaunchKernelGGL((delta_walk_kernel<DT>), walk, dim3(256), 0, s, scratch, state, cu_seqlens, seq_starts, seq_slots, raw_out, \
                     heads, dim, vdim, vp)
  if (dp == 64) QIL_DCW(4);
  else if (dp == 128) QIL_DCW(8);
  else QIL_DCW(16);
#undef QIL_DCW
  QIL_RETURN_LAUNCH_STATUS();
}

}  // extern "C"
