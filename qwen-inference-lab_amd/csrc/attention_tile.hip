// Attention of prompt portions (sequences with two or more rows in the step) over the paged cache,
// flash style on the matrix cores: no score matrix in memory, float32 online softmax.
//
// Block = 4 waves sharing one kv head and one range of keys; each wave owns a 16-row tile of one
// query head.  With g = heads / kv_heads query heads per kv head, a block covers GH = min(g, 4)
// heads (4 if g >= 3) and 4 / GH row tiles, so K and V tiles are staged in LDS once for the whole
// group (qil/model.py:59-61 expands them per query head instead).  Grid: (row tiles of the
// longest sequence, sequences, kv_heads * head chunks); blocks past a sequence's rows and
// sequences with a single row (the row kernel's) return at once.
//
// A row at absolute position p sees key j iff j <= p, and j > p - window with a window
// (qil/model.py:62-64).  Keys at or beyond the block's last position + 1 are never loaded: they
// are not written yet or belong to nobody; their LDS slots are zero so that 0 * garbage cannot
// make a NaN.  A wave skips key sub-tiles that lie wholly in the future of all its rows.
// keep > 0 (with a window, keys in one part): the first `keep` keys stay visible; a block walks the tiles that hold
// them, then goes on at its window's first tile.  slopes: slopes[h] * (position - key) is taken off head h's scaled
// score.
//
// Matrix-core formulation (wave64, 16x16 tiles).  Scores are computed transposed,
//   S^T[key, row] = sum_dim K[key, dim] Q[row, dim]        A = K tile (LDS), B = Q (registers)
// so that a lane ends up with the scores of ONE row (row = lane % 16) for keys 4 (lane / 16) + i:
// maxima, sums and rescaling are per-lane scalars, reduced over the 4 lane groups by two
// shuffles.  The same registers are then the B operand of
//   O^T[dim, row] = sum_key V^T[dim, key] P^T[key, row]    A = V tile transposed in LDS
// bfloat16 uses v_mfma_f32_16x16x32_bf16 (P rounded to bfloat16, float32 accumulation); float32
// uses v_mfma_f32_16x16x4_f32: float32 inputs and products, no reduced-precision mode.
#include <algorithm>

#include "common.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

#define TILE_THREADS 256

template <typename T> struct TileTraits;
template <> struct TileTraits<bf16_t> {
  static constexpr int BK = 64;        // keys per LDS tile
  static constexpr int KSTEP = 32;     // dims per score MFMA
  static constexpr int PAD = 8;        // LDS row padding in elements
};
template <> struct TileTraits<float> {
  static constexpr int BK = 32;
  static constexpr int KSTEP = 4;
  static constexpr int PAD = 4;
};

// exp(scale * (x - base)): one fused multiply-add and the hardware's exp2 for bfloat16; the library's
// exp on an exactly rounded argument for float32.
__device__ __forceinline__ float scaled_exp(float x, float base, float scale, bf16_t) {
  const float c = scale * 1.44269504088896f;
  return __builtin_amdgcn_exp2f(fmaf(x, c, -base * c));
}
__device__ __forceinline__ float scaled_exp(float x, float base, float scale, float) { return expf((x - base) * scale); }

// RB: 16-row tiles per wave.  A K or V^T fragment read from LDS serves RB products, which is what
// keeps the kernel from being bound by LDS reads.
// (float32 with head sizes above 64 needs more than 256 registers unless the head size is known at compile time
// and at most 128: one block a CU there, so that what does not fit goes to the other half of the register file and
// not to memory)
// WHOLE: d == DMAX, known when the kernel is compiled: no condition on the head size remains in the loops over
// dim tiles (with such conditions the float32 kernel spent most of its time copying accumulators between registers).
template <typename T, int DMAX, int RB, bool WHOLE>
__global__ void __launch_bounds__(TILE_THREADS, (sizeof(T) == 4 && DMAX > 64 && (!WHOLE || DMAX > 128)) ? 1 : 2)
attn_tile_kernel(const T* __restrict__ q, int q_stride, const T* __restrict__ k_cache, const T* __restrict__ v_cache,
                 const int* __restrict__ block_tables, int table_stride, const int* __restrict__ cu_seqlens,
                 const int* __restrict__ seq_starts, T* __restrict__ out, int heads, int kv_heads, int d,
                 int page_size, int window, float scale, int GH, int chunks, int ps_shift,
                 float* __restrict__ part_acc, float* __restrict__ part_m, float* __restrict__ part_l, int P, int parts,
                 float softcap, const float* __restrict__ sinks, const float* __restrict__ slopes, int keep) {
  // with a soft cap or a bias by distance the scores are scaled as they are made, and nothing is left for the exponent
  const float raw_scale = scale;
  if (softcap > 0.f || slopes) scale = 1.f;
  using TT = TileTraits<T>;
  constexpr int BK = TT::BK, KSTEP = TT::KSTEP, PAD = TT::PAD;
  constexpr bool BF16 = sizeof(T) == 2;
  constexpr int QFRAGS = DMAX / KSTEP;          // score MFMA steps over the head dim
  constexpr int DTILES = DMAX / 16;             // output dim tiles
  constexpr int SUB = BK / 16;                  // 16-key sub-tiles per LDS tile
  extern __shared__ __align__(16) unsigned char lds_raw[];

  const int seq = blockIdx.y;
  const int q0 = cu_seqlens[seq], n = cu_seqlens[seq + 1] - q0;
  if (n < 2) return;
  const int RT = 4 / GH;                        // waves along rows
  const int block_rows = 16 * RB * RT;
  // Later rows see more keys.  Blocks are handed to the 256 CUs in launch order, so consecutive groups
  // of 256 blocks walk the row tiles in opposite directions: a CU that got a long block gets a short one.
  // (The direction is fixed per (sequence, head group), so every row tile is still served exactly once.)
  const int linear = gridDim.x * (blockIdx.y + gridDim.y * blockIdx.z);
  const int across = ((linear >> 8) & 1) ? (int)blockIdx.x : (int)gridDim.x - 1 - (int)blockIdx.x;
  const int tile_row0 = across * block_rows;
  if (tile_row0 >= n) return;
  // parts > 1 (a few row tiles against a long context): grid.z also counts the parts of P keys, and a block
  // leaves float32 partial results (the layout of the split-context row kernels) for the merge kernel
  int pair = blockIdx.z;
  const int part = pair / (kv_heads * chunks);
  pair -= part * (kv_heads * chunks);
  const int kvh = pair / chunks, chunk = pair % chunks;
  const int g = heads / kv_heads;
  const int lane = threadIdx.x & (QIL_WAVE - 1), wave = threadIdx.x / QIL_WAVE;
  const int r = lane & 15, kb = lane >> 4;
  const int head_local = chunk * GH + wave % GH, row_group = wave / GH;
  const int wave_row0 = tile_row0 + row_group * 16 * RB;
  const bool wave_active = head_local < g && wave_row0 < n;
  const int head = kvh * g + head_local;
  const int start = seq_starts[seq];

  const int rows_in_block = min(block_rows, n - tile_row0);
  const int pos_first = start + tile_row0;
  int key_end = pos_first + rows_in_block;                             // last position + 1
  int key_begin = window > 0 ? max(0, pos_first - window + 1) : 0;
  if (parts > 1) {                                                     // P is a multiple of the tile's keys
    key_begin = max(key_begin, part * P);
    key_end = min(key_end, (part + 1) * P);
    if (key_begin >= key_end) return;                                  // no row of the block sees a key of this part
  }

  const int dt = WHOLE ? DMAX / 16 : (d + 15) / 16;    // dim tiles in use
  const int k_row = (BF16 ? (d + 31) / 32 * 32 : dt * 16) + PAD;       // elements per K row in LDS (staging
                                                                       // writes whole dim tiles)
  const int v_row = BK + PAD;                                          // elements per V^T row in LDS
  T* Ks = reinterpret_cast<T*>(lds_raw);                               // [BK][k_row]
  T* Vt = Ks + BK * k_row;                                             // [dt * 16][v_row]
  const int* table = block_tables + (size_t)seq * table_stride;

  int my_row[RB], my_pos[RB];
  bool row_valid[RB];
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    my_row[b] = wave_row0 + b * 16 + r;
    row_valid[b] = wave_active && my_row[b] < n;
    my_pos[b] = start + my_row[b];
  }
  const int wave_last_pos = start + min(n, wave_row0 + 16 * RB) - 1;   // nothing beyond it is visible to this wave

  // ---- Q fragments: B operands, Q[row r of tile b][dims of this lane's k slots]
  bf16x8 qb[RB][BF16 ? QFRAGS : 1];
  float qf[RB][BF16 ? 1 : QFRAGS];
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    const T* qrow = q + (size_t)(q0 + (row_valid[b] ? my_row[b] : 0)) * q_stride + (size_t)(wave_active ? head : 0) * d;
    if constexpr (BF16) {
#pragma unroll
      for (int ks = 0; ks < QFRAGS; ++ks) {
        const int dim = ks * 32 + kb * 8;
        uint4 raw = make_uint4(0, 0, 0, 0);
        if (row_valid[b] && dim < d) raw = *reinterpret_cast<const uint4*>(qrow + dim);
        qb[b][ks] = __builtin_bit_cast(bf16x8, raw);
      }
    } else {
      // step 4 j + i of a row's product takes dim 16 j + 4 kb + i from this lane: four steps' K values are one
      // 16-byte LDS read (any assignment of dims to steps will do, as long as K and Q share it)
#pragma unroll
      for (int ks = 0; ks < QFRAGS; ++ks) {
        const int dim = (ks >> 2) * 16 + 4 * kb + (ks & 3);
        qf[b][ks] = (row_valid[b] && (WHOLE || dim < d)) ? qrow[dim] : 0.f;
      }
    }
  }

  float m[RB], l[RB];
  f32x4 o[RB][DTILES];
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    m[b] = -INFINITY;
    l[b] = 0.f;
#pragma unroll
    for (int t = 0; t < DTILES; ++t) o[b][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }

  // ---- what this thread stages of every tile (the same places each time; only the keys move on)
  const int vec_per_key = (dt * 16) / 8;               // 8-element vectors per key covering the dim tiles
  const bool fast_v = page_size % 8 == 0;              // 8 keys of a dim are 16 (32) contiguous bytes of a V page
  constexpr int K_ITERS = (BK * (DMAX / 8) + TILE_THREADS - 1) / TILE_THREADS;
  constexpr int V_ITERS = (DMAX * (BK / 8) + TILE_THREADS - 1) / TILE_THREADS;
  int k_kl[K_ITERS], k_dv[K_ITERS], v_grp[V_ITERS], v_dim[V_ITERS];
#pragma unroll
  for (int it = 0; it < K_ITERS; ++it) {
    const int idx = threadIdx.x + it * TILE_THREADS;
    k_kl[it] = idx < BK * vec_per_key ? idx / vec_per_key : -1;
    k_dv[it] = (idx - max(k_kl[it], 0) * vec_per_key) * 8;
  }
#pragma unroll
  for (int it = 0; it < V_ITERS; ++it) {
    const int idx = threadIdx.x + it * TILE_THREADS;
    v_grp[it] = idx < dt * 16 * (BK / 8) ? idx / (dt * 16) : -1;         // consecutive threads: consecutive dims
    v_dim[it] = idx - max(v_grp[it], 0) * (dt * 16);
  }
  auto page_of = [&](int key, int& offset) -> size_t {
    int block;
    if (ps_shift >= 0) { block = key >> ps_shift; offset = key & (page_size - 1); }
    else { block = key / page_size; offset = key - block * page_size; }
    return (size_t)table[block];
  };

  // Fast staging (bfloat16, page_size % 8 == 0): no branch around a load, so that all table lookups of
  // a tile go out together, then all K and V^T vectors, and the zeroing of invisible keys is a select.
  // Addresses of places that are not needed are clamped onto needed ones.
  const bool fast = BF16 && fast_v;
  const int first_tile = key_begin / BK * BK;
  // the tiles that hold kept keys come first (those that lie below the window's first tile)
  const int kept_end = keep > 0 ? min((keep + BK - 1) / BK * BK, first_tile) : 0;
  const int low_key = keep > 0 ? 0 : key_begin;            // the first key whose page the block's table is asked for
  const float slope = (slopes && wave_active) ? slopes[head] : 0.f;
  auto needed = [&](int key) { return key < key_end && (key >= key_begin || key < keep); };

  for (int k0 = kept_end > 0 ? 0 : first_tile; k0 < key_end; k0 = k0 + BK == kept_end ? first_tile : k0 + BK) {
    __syncthreads();                                   // the previous tile is consumed
    if (fast) {
      if constexpr (BF16) {
        const bool inside = (k0 >= key_begin || k0 + BK <= keep) && k0 + BK <= key_end;     // no key of the tile needs zeroing
        size_t k_page[K_ITERS], v_page[V_ITERS];
        int k_off[K_ITERS], v_off[V_ITERS];
#pragma unroll
        for (int it = 0; it < K_ITERS; ++it) {
          const int key = min(max(k0 + max(k_kl[it], 0), low_key), key_end - 1);
          k_page[it] = page_of(key, k_off[it]);
        }
#pragma unroll
        for (int it = 0; it < V_ITERS; ++it) {
          const int key = min(max(k0 + max(v_grp[it], 0) * 8, low_key & ~7), (key_end - 1) & ~7);
          v_page[it] = page_of(key, v_off[it]);
        }
        uint4 k_reg[K_ITERS], v_reg[V_ITERS];
#pragma unroll
        for (int it = 0; it < K_ITERS; ++it)
          k_reg[it] = *reinterpret_cast<const uint4*>(
              k_cache + ((k_page[it] * kv_heads + kvh) * page_size + k_off[it]) * (size_t)d + min(k_dv[it], d - 8));
#pragma unroll
        for (int it = 0; it < V_ITERS; ++it)
          v_reg[it] = *reinterpret_cast<const uint4*>(
              v_cache + ((v_page[it] * kv_heads + kvh) * (size_t)d + min(v_dim[it], d - 1)) * page_size + v_off[it]);
#pragma unroll
        for (int it = 0; it < K_ITERS; ++it) {
          if (k_kl[it] < 0) continue;
          const int key = k0 + k_kl[it];
          const bool valid = needed(key) && k_dv[it] < d;
          *reinterpret_cast<uint4*>(Ks + k_kl[it] * k_row + k_dv[it]) = valid ? k_reg[it] : make_uint4(0, 0, 0, 0);
        }
#pragma unroll
        for (int it = 0; it < V_ITERS; ++it) {
          if (v_grp[it] < 0) continue;
          uint4 raw = v_dim[it] < d ? v_reg[it] : make_uint4(0, 0, 0, 0);
          if (!inside) {   // zero what lies outside [key_begin, key_end): never written, or someone else's
            const int key = k0 + v_grp[it] * 8;
            uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
            for (int e = 0; e < 8; ++e)
              if (!needed(key + e)) w[e >> 1] &= (e & 1) ? 0x0000ffffu : 0xffff0000u;
            raw = make_uint4(w[0], w[1], w[2], w[3]);
          }
          *reinterpret_cast<uint4*>(Vt + v_dim[it] * v_row + v_grp[it] * 8) = raw;
        }
      }
    } else {
    // ---- stage K (row major) of keys [k0, k0 + BK); V too on the generic path
#pragma unroll
    for (int it = 0; it < K_ITERS; ++it) {
      if (k_kl[it] < 0) continue;
      const int kl = k_kl[it], dv = k_dv[it], key = k0 + kl;
      const bool valid = needed(key) && dv < d;
      T* kdst = Ks + kl * k_row + dv;
      size_t page = 0;
      int offset = 0;
      if (valid) page = page_of(key, offset);
      const size_t kbase = ((page * kv_heads + kvh) * page_size + offset) * (size_t)d + dv;
      const T* column = v_cache + ((page * kv_heads + kvh) * (size_t)d + dv) * page_size + offset;
      if constexpr (BF16) {
        uint4 kraw = make_uint4(0, 0, 0, 0);
        if (valid) kraw = *reinterpret_cast<const uint4*>(k_cache + kbase);
        *reinterpret_cast<uint4*>(kdst) = kraw;
        if (!fast_v) {
#pragma unroll
          for (int e = 0; e < 8; ++e) Vt[(dv + e) * v_row + kl] = valid ? column[(size_t)e * page_size] : (bf16_t)0;
        }
      } else {
        float kv8[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) kv8[e] = 0.f;
        if (valid) ld8(k_cache + kbase, kv8);
#pragma unroll
        for (int e = 0; e < 8; ++e) kdst[e] = kv8[e];
        if (!fast_v) {
#pragma unroll
          for (int e = 0; e < 8; ++e) Vt[(dv + e) * v_row + kl] = valid ? column[(size_t)e * page_size] : 0.f;
        }
      }
    }
    if (fast_v) {
      // ---- stage V^T: a thread copies 8 consecutive keys of one dim (one vector of the page's row)
#pragma unroll
      for (int it = 0; it < V_ITERS; ++it) {
        if (v_grp[it] < 0) continue;
        const int grp = v_grp[it], dim = v_dim[it], key = k0 + grp * 8;
        T* dst = Vt + dim * v_row + grp * 8;
        const bool any = (key + 7 >= key_begin || key < keep) && key < key_end && dim < d;
        float vals[8];
        if (any) {
          int offset;
          const size_t page = page_of(key, offset);
          ld8(v_cache + ((page * kv_heads + kvh) * (size_t)d + dim) * page_size + offset, vals);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) dst[e] = (any && needed(key + e)) ? vals[e] : 0.f;
      }
    }
    }
    if constexpr (BF16) {
      // K rows are read in steps of 32 dims: zero the tail between the dim tiles and the padded width
      const int tail0 = dt * 16, tail = (d + 31) / 32 * 32 - tail0;
      if (tail > 0)
        for (int idx = threadIdx.x; idx < BK * tail; idx += TILE_THREADS)
          Ks[(idx / tail) * k_row + tail0 + idx % tail] = 0;
    }
    __syncthreads();
    if (!wave_active || k0 > wave_last_pos) continue;

    // ---- S^T = K Q^T for the tile's 16-key sub-tiles, each K fragment serving the RB row tiles
    f32x4 s[RB][SUB];
#pragma unroll
    for (int jt = 0; jt < SUB; ++jt) {
#pragma unroll
      for (int b = 0; b < RB; ++b) s[b][jt] = (f32x4){0.f, 0.f, 0.f, 0.f};
      if (k0 + jt * 16 > wave_last_pos) continue;                     // wholly in the future of every row
      const T* krow = Ks + (jt * 16 + r) * k_row;
      if constexpr (BF16) {
#pragma unroll
        for (int ks = 0; ks < QFRAGS; ++ks) {
          if (WHOLE || ks * 32 < d) {
            const bf16x8 a = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(krow + ks * 32 + kb * 8));
#pragma unroll
            for (int b = 0; b < RB; ++b) s[b][jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qb[b][ks], s[b][jt], 0, 0, 0);
          }
        }
      } else {
#pragma unroll
        for (int j = 0; j < QFRAGS / 4; ++j)
          if (WHOLE || j * 16 < d) {
            // dims 16 j + 4 kb + i; past d (a head size that is no multiple of 16) the row's padding or the next
            // row is read, finite values that meet zeros of Q
            const f32x4 a = *reinterpret_cast<const f32x4*>(krow + j * 16 + 4 * kb);
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
              for (int b = 0; b < RB; ++b)
                s[b][jt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], qf[b][4 * j + i], s[b][jt], 0, 0, 0);
            __builtin_amdgcn_sched_barrier(0);              // reads of all 32 steps at once would spill
          }
      }
    }
    if (softcap > 0.f) {
      const float fast = 2.88539008177793f / softcap;
#pragma unroll
      for (int b = 0; b < RB; ++b)
#pragma unroll
        for (int jt = 0; jt < SUB; ++jt)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            s[b][jt][i] = BF16 ? soft_cap_fast(s[b][jt][i] * raw_scale, softcap, fast) : soft_cap(s[b][jt][i] * raw_scale, softcap);
    }
    if (slopes) {
      const float rest = softcap > 0.f ? 1.f : raw_scale;
#pragma unroll
      for (int b = 0; b < RB; ++b)
#pragma unroll
        for (int jt = 0; jt < SUB; ++jt)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            s[b][jt][i] = fmaf(slope, (float)(k0 + jt * 16 + 4 * kb + i - my_pos[b]), s[b][jt][i] * rest);
    }
    // ---- mask and online softmax (per-lane row statistics).  m holds the running maximum of the RAW
    // scores; the scale (> 0) enters once, in the exponent: p = exp(scale * (s - m)).
    // every key of the tile is visible to every row of the wave unless the tile touches the wave's
    // first row's future, the window's edge or the rows beyond the sequence
    const bool all_visible = k0 + BK - 1 <= start + wave_row0 && wave_row0 + 16 * RB <= n &&
                             (window <= 0 || k0 > wave_last_pos - window || k0 + BK <= keep);
#pragma unroll
    for (int b = 0; b < RB; ++b) {
      float mx = -INFINITY;
      if (all_visible) {
#pragma unroll
        for (int jt = 0; jt < SUB; ++jt)
#pragma unroll
          for (int i = 0; i < 4; ++i) mx = fmaxf(mx, s[b][jt][i]);
      } else {
#pragma unroll
        for (int jt = 0; jt < SUB; ++jt)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int key = k0 + jt * 16 + 4 * kb + i;
            const bool visible = row_valid[b] && key <= my_pos[b] &&
                                 (window <= 0 || key > my_pos[b] - window || key < keep);
            const float v = visible ? s[b][jt][i] : -INFINITY;
            s[b][jt][i] = v;
            mx = fmaxf(mx, v);
          }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, QIL_WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, QIL_WAVE));
      const float m_new = fmaxf(m[b], mx);
      const float base = (m_new == -INFINITY) ? 0.f : m_new;                              // exp(-inf - 0) = 0
      const float alpha = (m_new == -INFINITY) ? 1.f : scaled_exp(m[b], base, scale, T());  // m = -inf gives 0
      float psum = 0.f;
#pragma unroll
      for (int jt = 0; jt < SUB; ++jt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float p = scaled_exp(s[b][jt][i], base, scale, T());
          s[b][jt][i] = p;
          psum += p;
        }
      l[b] = l[b] * alpha + psum;
      if (m_new != m[b]) {                       // nothing to rescale while the maximum stands
#pragma unroll
        for (int t = 0; t < DTILES; ++t)
#pragma unroll
          for (int i = 0; i < 4; ++i) o[b][t][i] *= alpha;
      }
      m[b] = m_new;
    }

    // ---- O^T += V^T P^T, each V^T fragment serving the RB row tiles
    if constexpr (BF16) {
#pragma unroll
      for (int st = 0; st < SUB / 2; ++st) {
        if (k0 + st * 32 > wave_last_pos) continue;
        bf16x8 pb[RB];
#pragma unroll
        for (int b = 0; b < RB; ++b) {
          uint32_t packed[4];
#pragma unroll
          for (int i = 0; i < 2; ++i) {
            packed[i] = pack_bf16(s[b][2 * st][2 * i], s[b][2 * st][2 * i + 1]);
            packed[2 + i] = pack_bf16(s[b][2 * st + 1][2 * i], s[b][2 * st + 1][2 * i + 1]);
          }
          pb[b] = __builtin_bit_cast(bf16x8, make_uint4(packed[0], packed[1], packed[2], packed[3]));
        }
#pragma unroll
        for (int t = 0; t < DTILES; ++t) {
          if (WHOLE || t < dt) {
            const T* vrow = Vt + (t * 16 + r) * v_row + st * 32 + 4 * kb;
            const uint2 lo = *reinterpret_cast<const uint2*>(vrow);
            const uint2 hi = *reinterpret_cast<const uint2*>(vrow + 16);
            const bf16x8 a = __builtin_bit_cast(bf16x8, make_uint4(lo.x, lo.y, hi.x, hi.y));
#pragma unroll
            for (int b = 0; b < RB; ++b) o[b][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pb[b], o[b][t], 0, 0, 0);
          }
        }
      }
    } else {
#pragma unroll
      for (int jt = 0; jt < SUB; ++jt) {
        if (k0 + jt * 16 > wave_last_pos) continue;
#pragma unroll
        for (int t = 0; t < DTILES; ++t)
          if (WHOLE || t < dt) {
            const f32x4 a = *reinterpret_cast<const f32x4*>(Vt + (t * 16 + r) * v_row + jt * 16 + 4 * kb);
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
              for (int b = 0; b < RB; ++b)
                o[b][t] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], s[b][jt][i], o[b][t], 0, 0, 0);
            if (t & 1) __builtin_amdgcn_sched_barrier(0);   // reads of all dim tiles at once would spill
          }
      }
    }
  }

  if (!wave_active) return;
#pragma unroll
  for (int b = 0; b < RB; ++b) {
    float total = l[b];
    total += __shfl_xor(total, 16, QIL_WAVE);
    total += __shfl_xor(total, 32, QIL_WAVE);
    if (!row_valid[b]) continue;
    if (parts > 1) {
      // acc [row, head, part, d] unnormalised, m (the maximum in the exponent's units) and l [row, head, part]; a row
      // that sees no key of this part leaves m = -inf, l = 0 in a cell the merge does not read
      const size_t cell = ((size_t)(q0 + my_row[b]) * heads + head) * parts + part;
#pragma unroll
      for (int t = 0; t < DTILES; ++t)
        if (WHOLE || t * 16 + 4 * kb < d)                   // d % 4 == 0: the four dims are inside together
          *reinterpret_cast<float4*>(part_acc + cell * d + t * 16 + 4 * kb) =
              make_float4(o[b][t][0], o[b][t][1], o[b][t][2], o[b][t][3]);
      if (kb == 0) {
        part_m[cell] = m[b] == -INFINITY ? -INFINITY : m[b] * scale;
        part_l[cell] = total;
      }
      continue;
    }
    // a division, as in the merge of parts: keys that all lie in one part then give the same bits either way
    T* orow = out + ((size_t)(q0 + my_row[b]) * heads + head) * d;
    if (sinks) {                                            // one more term in the divisor: exp(sink), no key, no value
      const float r = sink_reciprocal(total, m[b] * scale, sinks[head]);
#pragma unroll
      for (int t = 0; t < DTILES; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int dim = t * 16 + 4 * kb + i;
          if (WHOLE || dim < d) st(orow + dim, o[b][t][i] * r);
        }
      continue;
    }
#pragma unroll
    for (int t = 0; t < DTILES; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int dim = t * 16 + 4 * kb + i;
        if (WHOLE || dim < d) st(orow + dim, o[b][t][i] / total);
      }
  }
}

template <typename T, int DMAX, int RB>
static int launch_tile(const void* q, int q_stride, const void* k_cache, const void* v_cache, const int* block_tables,
                       int table_stride, const int* cu_seqlens, const int* seq_starts, void* out, int n_seqs,
                       int max_query, int heads, int kv_heads, int d, int page_size, int window, float scale,
                       hipStream_t s, float* workspace = nullptr, int total_rows = 0, int P = 0, int parts = 1,
                       float softcap = 0.f, const float* sinks = nullptr, const float* slopes = nullptr, int keep = 0) {
  using TT = TileTraits<T>;
  const int g = heads / kv_heads;
  const int GH = g >= 3 ? 4 : g, chunks = (g + GH - 1) / GH, RT = 4 / GH;
  const bool bf16 = sizeof(T) == 2;
  const int k_row = (bf16 ? (d + 31) / 32 * 32 : (d + 15) / 16 * 16) + TT::PAD, v_row = TT::BK + TT::PAD;
  const size_t lds = ((size_t)TT::BK * k_row + (size_t)((d + 15) / 16 * 16) * v_row) * sizeof(T);
  const bool whole = !bf16 && d == DMAX;                 // (the common bfloat16 sizes have a kernel of their own)
  auto kernel = whole ? attn_tile_kernel<T, DMAX, RB, sizeof(T) == 4> : attn_tile_kernel<T, DMAX, RB, false>;
  static size_t granted[2] = {0, 0};                     // per instantiation
  if (lds > 64 * 1024 && lds > granted[whole]) {
    hipError_t e = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
    granted[whole] = lds;
  }
  if ((long)kv_heads * chunks * parts > 65535) return -1;
  dim3 grid((max_query + 16 * RB * RT - 1) / (16 * RB * RT), n_seqs, kv_heads * chunks * parts);
  float* part_m = workspace ? workspace + (size_t)total_rows * heads * parts * d : nullptr;
  float* part_l = part_m ? part_m + (size_t)total_rows * heads * parts : nullptr;
  int ps_shift = -1;                                      // log2 of a power-of-two page size
  for (int b = 0; b < 30; ++b)
    if (page_size == (1 << b)) ps_shift = b;
  hipLaunchKernelGGL(kernel, grid, dim3(TILE_THREADS), lds, s, (const T*)q, q_stride, (const T*)k_cache,
                     (const T*)v_cache, block_tables, table_stride, cu_seqlens, seq_starts, (T*)out, heads, kv_heads, d,
                     page_size, window, scale, GH, chunks, ps_shift, workspace, part_m, part_l, P, parts, softcap, sinks, slopes,
                     keep);
  return (int)hipGetLastError();
}

// The branch-free kernel for the common bfloat16 case (attention_tile_bf16.hip).
extern "C" int qil_attn_tile_bf16_takes(int d, int page_size, int table_stride);
extern "C" int qil_attn_tile_bf16(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                                  const int* block_tables, int table_stride, const int* cu_seqlens,
                                  const int* seq_starts, void* out, int n_seqs, int max_query, int heads, int kv_heads,
                                  int d, int page_size, int window, float scale, hipStream_t s);

extern "C" int qil_attn_prompt_takes(int d, int page_size, int table_stride);
extern "C" int qil_attn_prompt_capped(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                                      const int* block_tables, int table_stride, const int* cu_seqlens,
                                      const int* seq_starts, void* out, int n_seqs, int max_query, int heads, int kv_heads,
                                      int page_size, int window, float scale, float softcap, void* workspace,
                                      int total_rows, int P, int parts, hipStream_t s);

// Keys in parts for this file's kernel (the float32 path, and bfloat16 sizes that the branch-free kernel does not
// take): a portion of a prompt deep in a long context is a few row tiles, each with all its keys ahead of it one
// after the other, on fewer blocks than the chip has CUs.  Returns the number of parts to cut the keys into (1: do
// not) and their size in *P: about four blocks a CU, parts of at least 128 keys, at most 32 of them (measured with
// float32 portions of 128 rows at 1,000 to 2,700 keys, 32 blocks of row tiles: parts of 128 keys 4.60 ms a step of
// 28 layers, 192 4.76, 256 4.92, 64 4.87).
extern "C" int qil_attn_tile_key_parts(int n_seqs, int max_query, int heads, int kv_heads, int d, int max_context,
                                       int dtype, int* P) {
  *P = 0;
  if (heads % kv_heads || max_query < 2 || max_context < 512) return 1;
  const int g = heads / kv_heads, GH = g >= 3 ? 4 : g, chunks = (g + GH - 1) / GH, RT = 4 / GH;
  const int RB = (dtype == QIL_BF16 && d <= 128) ? 2 : 1;
  const long blocks = (long)((max_query + 16 * RB * RT - 1) / (16 * RB * RT)) * n_seqs * kv_heads * chunks;
  if (blocks >= QIL_CUS) return 1;
  const int want = (int)std::min(32L, (4 * QIL_CUS + blocks - 1) / blocks);
  int part = ((max_context + want - 1) / want + 63) / 64 * 64;         // whole tiles of 32 (float32) or 64 keys
  part = std::max(part, 128);
  const int parts = (max_context + part - 1) / part;
  if (parts < 2 || (long)kv_heads * chunks * parts > 65535) return 1;
  *P = part;
  return parts;
}

// Sequences with >= 2 rows.  q: rows of stride q_stride, head h at h * d; out [rows, heads * d].
// Requires d % 8 == 0, 8 <= d <= 256.  Returns -1 on a size it does not take.
extern "C" int qil_attn_prompt_sinks(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                                     const int* block_tables, int table_stride, const int* cu_seqlens,
                                     const int* seq_starts, void* out, int n_seqs, int max_query, int heads, int kv_heads,
                                     int page_size, int window, float scale, const float* sinks, hipStream_t s);
extern "C" int qil_attn_prompt_extended(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                                        const int* block_tables, int table_stride, const int* cu_seqlens,
                                        const int* seq_starts, void* out, int n_seqs, int max_query, int heads, int kv_heads,
                                        int page_size, int window, float scale, const float* sinks, const float* slopes,
                                        int keep, hipStream_t s);
// parts > 1: the keys in `parts` parts of P keys (P a multiple of 64) on this file's kernel; every row of a sequence
// of two or more rows gets float32 partial results in `workspace` (qil_attn_rows_workspace bytes for all `total_rows`
// rows of the step, indexed by the step's row) for qil_attn_merge, and `out` is not written.
static int tile_dispatch(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                         const int* block_tables, int table_stride, const int* cu_seqlens, const int* seq_starts,
                         void* out, int n_seqs, int max_query, int heads, int kv_heads, int d, int page_size,
                         int window, float scale, int dtype, hipStream_t s, float* workspace, int total_rows, int P,
                         int parts, float softcap, const float* sinks = nullptr, const float* slopes = nullptr, int keep = 0) {
  if (n_seqs == 0 || max_query < 2) return 0;
  if (keep < 0 || (keep > 0 && (window <= 0 || parts > 1))) return -1;
  const bool extended = slopes || keep > 0;
  // a bias by distance or kept first keys on bfloat16 heads of 128, keys in one part: the prompt kernel's extended form
  if (extended && parts == 1 && softcap <= 0.f && dtype == QIL_BF16 && qil_attn_prompt_takes(d, page_size, table_stride))
    return qil_attn_prompt_extended(q, q_stride, k_cache, v_cache, block_tables, table_stride, cu_seqlens, seq_starts, out,
                                    n_seqs, max_query, heads, kv_heads, page_size, window, scale, sinks, slopes, keep, s);
  if (d % 8 || d < 8 || d > 256 || heads % kv_heads || n_seqs > 65535 || kv_heads * 2 > 65535) return -1;
  // capped scores of bfloat16 heads of 128: the prompt kernel's capped form (keys in one part or in parts of whole tiles)
  if (softcap > 0.f && !sinks && !extended && dtype == QIL_BF16 && qil_attn_prompt_takes(d, page_size, table_stride) && (parts == 1 || P % 64 == 0))
    return qil_attn_prompt_capped(q, q_stride, k_cache, v_cache, block_tables, table_stride, cu_seqlens, seq_starts, out,
                                  n_seqs, max_query, heads, kv_heads, page_size, window, scale, softcap, workspace,
                                  total_rows, P, parts, s);
  // sinks on bfloat16 heads of 128, keys in one part: the prompt kernel's form with sinks
  if (sinks && !extended && parts == 1 && softcap <= 0.f && dtype == QIL_BF16 && qil_attn_prompt_takes(d, page_size, table_stride))
    return qil_attn_prompt_sinks(q, q_stride, k_cache, v_cache, block_tables, table_stride, cu_seqlens, seq_starts, out,
                                 n_seqs, max_query, heads, kv_heads, page_size, window, scale, sinks, s);
  if (parts == 1 && softcap <= 0.f && !sinks && !extended && dtype == QIL_BF16 && qil_attn_tile_bf16_takes(d, page_size, table_stride))
    return qil_attn_tile_bf16(q, q_stride, k_cache, v_cache, block_tables, table_stride, cu_seqlens, seq_starts, out,
                              n_seqs, max_query, heads, kv_heads, d, page_size, window, scale, s);
#define QIL_TILE_CASE(T, DMAX)                                                                                      \
  return launch_tile<T, DMAX, (sizeof(T) == 2 && DMAX <= 128) ? 2 : 1>(q, q_stride, k_cache, v_cache, block_tables, table_stride, cu_seqlens, seq_starts, out, \
                              n_seqs, max_query, heads, kv_heads, d, page_size, window, scale, s, workspace, total_rows, P, parts, softcap, sinks, slopes, keep)
  if (dtype == QIL_F32) {
    if (d <= 64) QIL_TILE_CASE(float, 64);
    if (d <= 128) QIL_TILE_CASE(float, 128);
    QIL_TILE_CASE(float, 256);
  }
  if (d <= 64) QIL_TILE_CASE(bf16_t, 64);
  if (d <= 128) QIL_TILE_CASE(bf16_t, 128);
  QIL_TILE_CASE(bf16_t, 256);
#undef QIL_TILE_CASE
}

extern "C" int qil_attn_tile(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                             const int* block_tables, int table_stride, const int* cu_seqlens, const int* seq_starts,
                             void* out, int n_seqs, int max_query, int heads, int kv_heads, int d, int page_size,
                             int window, float scale, float softcap, int dtype, const float* sinks, const float* slopes,
                             int keep, hipStream_t s) {
  return tile_dispatch(q, q_stride, k_cache, v_cache, block_tables, table_stride, cu_seqlens, seq_starts, out, n_seqs,
                       max_query, heads, kv_heads, d, page_size, window, scale, dtype, s, nullptr, 0, 0, 1, softcap, sinks, slopes, keep);
}

extern "C" int qil_attn_tile_in_parts(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                                      const int* block_tables, int table_stride, const int* cu_seqlens,
                                      const int* seq_starts, void* workspace, int total_rows, int n_seqs, int max_query,
                                      int heads, int kv_heads, int d, int page_size, int window, float scale,
                                      float softcap, int P, int parts, int dtype, const float* slopes, hipStream_t s) {
  if (n_seqs == 0 || max_query < 2) return 0;
  if (parts < 2 || P < 64 || P % 64 || !workspace || total_rows < 1) return -1;
  return tile_dispatch(q, q_stride, k_cache, v_cache, block_tables, table_stride, cu_seqlens, seq_starts, nullptr, n_seqs,
                       max_query, heads, kv_heads, d, page_size, window, scale, dtype, s, (float*)workspace, total_rows,
                       P, parts, softcap, nullptr, slopes);
}
