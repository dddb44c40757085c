// Split-context attention of single rows (decoded tokens) on the matrix cores, bfloat16.
//
// Same task and the same partial results as the row kernel in attention_rows.hip (a block owns
// the keys [part * P, (part + 1) * P) of one row and one kv head and serves the whole group of
// query heads reading that kv head; the merge kernel there combines the parts), but the operands
// go from global memory straight into v_mfma_f32_16x16x32_bf16, with no staging in LDS:
//
//   S^T[key, head] = sum_dim K[key, dim] Q[head, dim]     A = K rows      (K is [.., page_size, d])
//   O^T[dim, head] = sum_key V^T[dim, key] P^T[key, head] A = V^T rows    (V is [.., d, page_size])
//
// The 16 columns of a tile are the g query heads of the kv head (columns from g on are zero), so
// a lane holds the scores of ONE head for eight keys (8 (lane / 16) + j of a 32-key step: the rows
// of the two 16-key score tiles are assigned to keys accordingly), and softmax statistics are
// per-lane scalars reduced over the 4 lane groups by two shuffles (qil/paged_attention.py:27-41
// computes the same maxima, sums and weighted values in float32).  Each of the block's waves
// takes every waves-th 32-key step and keeps its own running (m, l, O); they meet in LDS once.
//
// Invisible keys (j > position, or outside the window) may lie in pages that were never
// written or belong to someone else: their scores are replaced, not multiplied, and their V
// elements are zeroed before the product, so garbage (even NaN) cannot enter a sum.
//
// keep > 0: the first `keep` keys stay visible behind a window; steps and parts then count places (key_span.h).
// slopes: slopes[h] * (position - key) is taken off head h's scaled score.
//
// Takes page_size % 8 == 0, d % 16 == 0, d <= 256, g <= 16; other sizes go to the row kernel.
#include "common.h"
#include "key_span.h"
#include "qk_math.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

#define DEC_MAX_WAVES 8                                    // waves of a block; each takes every waves-th 32-key step

// FUSED: the queries do not come from memory but from the partial sums of the q/k/v product, with the
// head norm and the rotation made here (the arithmetic of qk_rope.hip, shared through qk_math.h); and the
// wave that meets the row's own position makes the new key and value the same way, writes them into the
// pages and uses them from its registers.  One kernel less per layer in a decode step.
struct FusedQKV {
  const float* qkv;                                        // [splits][rows][(heads + 2 kv_heads) d] partial sums
  size_t split_stride;
  int splits;
  const float* q_weight;                                   // null: no head norm
  const float* k_weight;
  float eps;
  const float* cos_table;                                  // null: no rotation
  const float* sin_table;                                  // null with a cos_table: that holds rot / 2 frequencies
  int rot;
  int rotate_first;                                        // the rotation comes before the head norm
  int writes;                                              // 0: the cache belongs to another layer, which wrote it
  int row_elems;                                           // elements of a row of qkv (more than q, k and v where another
                                                           // branch's columns follow; q alone for a reader without k and v)
  int v_head;                                              // the head-sized piece of a row at which the values begin
                                                           // (heads + kv_heads; heads: the values are the keys before norm
                                                           // and rotation)
  const float* bias;                                       // null, or the projection's bias by column, added to the sums
  float temp_coef;                                         // temp_every > 0: the query at position p is multiplied by
  int temp_every;                                          // 1 + temp_coef * ln(floor((p + 1) / temp_every) + 1) last
};

// Keys and values are read once a step by one block (the whole group of query heads is served by it).
__device__ __forceinline__ uint4 once4(const bf16_t* p) {
  const qil_u32x4 v = load_once(p);
  return make_uint4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ uint4 pack8(const float* v) {
  return make_uint4(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]), pack_bf16(v[4], v[5]), pack_bf16(v[6], v[7]));
}
__device__ __forceinline__ uint4 shuffle4(uint4 v, int source) {
  return make_uint4(__shfl(v.x, source, QIL_WAVE), __shfl(v.y, source, QIL_WAVE), __shfl(v.z, source, QIL_WAVE),
                    __shfl(v.w, source, QIL_WAVE));
}

// WHOLE: d == DMAX (always so when FUSED).
template <int DMAX, bool PAIRS, bool FUSED, bool WHOLE = FUSED>
__global__ void __launch_bounds__(DEC_MAX_WAVES * QIL_WAVE)
attn_decode_kernel(FusedQKV fused, const bf16_t* __restrict__ q, int q_stride, const bf16_t* __restrict__ k_cache,
                   const bf16_t* __restrict__ v_cache, const int* __restrict__ block_tables, int table_stride,
                   const int* __restrict__ row_seq, const int* __restrict__ positions,
                   const int* __restrict__ row_index, float* __restrict__ part_acc, float* __restrict__ part_m,
                   float* __restrict__ part_l, bf16_t* __restrict__ out, int heads, int kv_heads, int d,
                   int page_size, int window, float scale, int P, int parts, float softcap,
                   const float* __restrict__ sinks, const float* __restrict__ slopes, int keep) {
  constexpr int QFRAGS = DMAX / 32, DTILES = DMAX / 16;
  if (WHOLE) d = DMAX;                                      // what the host has checked, known to the compiler: no
                                                            // condition on the head size stays in the loops
  extern __shared__ float lds[];
  const int slot_row = blockIdx.x, kvh = blockIdx.y, part = blockIdx.z;
  const int row = row_index ? row_index[slot_row] : slot_row;
  const int g = heads / kv_heads;
  const int pos = positions[row], ctx = pos + 1;
  const KeySpan span(pos, window, keep);
  const int begin = max(part * P, span.first_place()), end = min((part + 1) * P, span.places());      // places
  if (begin >= end) return;
  const int pos_place = pos - span.hole;                   // the row's own key lies behind the hole

  const int lane = threadIdx.x & (QIL_WAVE - 1), wave = threadIdx.x / QIL_WAVE, waves = blockDim.x / QIL_WAVE;
  const int r = lane & 15, kb = lane >> 4;
  const int dt = d / 16;
  const int* table = block_tables + (size_t)row_seq[row] * table_stride;

  const int first_step = begin / 32;                       // steps of 32 places, numbered from the first place
  const int last_step = (end - 1) / 32;
  const float slope = (slopes && r < g) ? slopes[kvh * g + r] : 0.f;

  // Q fragments: B operand, column r = head kvh * g + r (filled below, after the first loads are on their way)
  bf16x8 qb[QFRAGS];
  uint4 new_k = make_uint4(0, 0, 0, 0), new_v = make_uint4(0, 0, 0, 0);   // FUSED: chunk lane % (DMAX / 8) of the new key / value
  bool owner = false;                                      // FUSED: this wave meets the row's own position

  float m = -INFINITY, l = 0.f;
  f32x4 o[DTILES];
#pragma unroll
  for (int t = 0; t < DTILES; ++t) o[t] = (f32x4){0.f, 0.f, 0.f, 0.f};

  // What one 32-key step needs from memory: the K rows of both 16-key sub-tiles and the V^T fragments
  // of every dim tile, found through three entries of the block table.
  struct StepData {
    uint4 k[2][QFRAGS];
    uint4 v[DTILES];                                        // V^T[dim 16 t + r][keys 8 kb .. 8 kb + 7]: 16 bytes of one page row
  };
  auto look_up = [&](int step, int (&page)[3]) {
    const int k0 = span.key(step * 32);
#pragma unroll
    for (int jt = 0; jt < 2; ++jt)
      // row r of sub-tile jt is key 8 (r / 4) + 4 jt + r % 4 of the step, so that a lane's eight
      // scores (rows 4 kb + i of both sub-tiles) are the eight consecutive keys 8 kb .. 8 kb + 7
      page[jt] = table[min(k0 + 8 * (r >> 2) + 4 * jt + (r & 3), ctx - 1) / page_size];   // clamped: an invisible key's score is replaced
    page[2] = table[(min(k0 + 8 * kb, ctx - 1) & ~7) / page_size];
  };
  auto request = [&](int step, const int (&page)[3], StepData& data) {
    const int k0 = span.key(step * 32);
#pragma unroll
    for (int jt = 0; jt < 2; ++jt) {
      const int key = min(k0 + 8 * (r >> 2) + 4 * jt + (r & 3), ctx - 1);
      const bf16_t* krow = k_cache + (((size_t)page[jt] * kv_heads + kvh) * page_size + (key % page_size)) * (size_t)d;
#pragma unroll
      for (int ks = 0; ks < QFRAGS; ++ks) {
        const int dim = ks * 32 + kb * 8;
        data.k[jt][ks] = (ks * 32 < d && dim < d) ? once4(krow + dim) : make_uint4(0, 0, 0, 0);
      }
    }
    const int key = min(k0 + 8 * kb, ctx - 1) & ~7;
    const bf16_t* vbase = v_cache + ((size_t)page[2] * kv_heads + kvh) * (size_t)d * page_size + (key % page_size);
#pragma unroll
    for (int t = 0; t < DTILES; ++t)
      data.v[t] = t < dt ? once4(vbase + (size_t)(t * 16 + r) * page_size) : make_uint4(0, 0, 0, 0);
  };
  auto attend = [&](int step, StepData& data) {
    const int k0 = span.key(step * 32);
    if constexpr (FUSED) {
      if (owner && step == (pos_place >> 5)) {                   // the new key and value come from this wave's registers
        const int local = pos & 31;                          // key 8 (rr / 4) + 4 jt + rr % 4 of the step
        const int jt_new = (local >> 2) & 1, rr = ((local >> 3) << 2) | (local & 3);
#pragma unroll
        for (int ks = 0; ks < QFRAGS; ++ks) {
          const uint4 piece = shuffle4(new_k, 4 * ks + kb);
#pragma unroll
          for (int jt = 0; jt < 2; ++jt)
            if (r == rr && jt == jt_new) data.k[jt][ks] = piece;
        }
        const int j = local & 7;                             // element of the lanes with kb == local / 8
#pragma unroll
        for (int t = 0; t < DTILES; ++t) {
          const uint4 piece = shuffle4(new_v, 2 * t + (r >> 3));             // chunk of dim 16 t + r
          const int e = r & 7;
          const uint32_t word = (e >> 1) == 0 ? piece.x : (e >> 1) == 1 ? piece.y : (e >> 1) == 2 ? piece.z : piece.w;
          const uint32_t value = (word >> ((e & 1) * 16)) & 0xffffu;
          if (kb == (local >> 3)) {
            const uint32_t shift = (j & 1) * 16, keep = ~(0xffffu << shift), put = value << shift;
            uint32_t w[4] = {data.v[t].x, data.v[t].y, data.v[t].z, data.v[t].w};
#pragma unroll
            for (int i = 0; i < 4; ++i)
              if (i == (j >> 1)) w[i] = (w[i] & keep) | put;
            data.v[t] = make_uint4(w[0], w[1], w[2], w[3]);
          }
        }
      }
    }
    // ---- scores
    f32x4 s[2];
#pragma unroll
    for (int jt = 0; jt < 2; ++jt) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < QFRAGS; ++ks)
        if (ks * 32 < d) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, data.k[jt][ks]), qb[ks], acc, 0, 0, 0);
      s[jt] = acc;
    }
    float mx = -INFINITY;
    uint32_t seen[2][4];                                    // 0xffff where the key is visible
#pragma unroll
    for (int jt = 0; jt < 2; ++jt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = k0 + 8 * kb + 4 * jt + i;
        const bool visible = span.visible(key);              // (a part ends at a whole step, or where the keys end)
        seen[jt][i] = visible ? 0xffffu : 0u;
        float v = s[jt][i] * scale;
        if (softcap > 0.f) v = soft_cap_fast(v, softcap, 2.88539008177793f / softcap);
        v = fmaf(slope, (float)(key - pos), v);
        if (!visible) v = -INFINITY;
        s[jt][i] = v;
        mx = fmaxf(mx, v);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, QIL_WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, QIL_WAVE));
    const float m_new = fmaxf(m, mx);
    const float alpha = (m_new == -INFINITY) ? 1.f : __builtin_amdgcn_exp2f((m - m_new) * 1.44269504088896f);
    float psum = 0.f;
#pragma unroll
    for (int jt = 0; jt < 2; ++jt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float p = (s[jt][i] == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f((s[jt][i] - m_new) * 1.44269504088896f);
        s[jt][i] = p;
        psum += p;
      }
    l = l * alpha + psum;
    m = m_new;
    // ---- O^T = O^T alpha + V^T P^T
    uint32_t packed[4];
#pragma unroll
    for (int jt = 0; jt < 2; ++jt)
#pragma unroll
      for (int i = 0; i < 2; ++i)
        packed[jt * 2 + i] = pack_bf16(s[jt][2 * i], s[jt][2 * i + 1]);
    const bf16x8 pb = __builtin_bit_cast(bf16x8, make_uint4(packed[0], packed[1], packed[2], packed[3]));
    const uint32_t mask[4] = {seen[0][0] | (seen[0][1] << 16), seen[0][2] | (seen[0][3] << 16),
                              seen[1][0] | (seen[1][1] << 16), seen[1][2] | (seen[1][3] << 16)};
#pragma unroll
    for (int t = 0; t < DTILES; ++t) {
      if (t < dt) {
        const bf16x8 a = __builtin_bit_cast(bf16x8, make_uint4(data.v[t].x & mask[0], data.v[t].y & mask[1],
                                                                data.v[t].z & mask[2], data.v[t].w & mask[3]));
#pragma unroll
        for (int i = 0; i < 4; ++i) o[t][i] *= alpha;
        o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pb, o[t], 0, 0, 0);
      }
    }
  };
  auto make_queries = [&]() {
    if constexpr (FUSED) {
      constexpr int TG = DMAX / 8, HPP = QIL_WAVE / TG;      // lanes of a head (8 elements each), heads a pass
      const int chunk = lane % TG, sub = lane / TG;
      // the block's waves share the heads (HPP of them a wave and pass); the queries meet in LDS
      uint4* shared_q = reinterpret_cast<uint4*>(lds);       // [g][TG] chunks; the end of the kernel uses the LDS again
      for (int base = wave * HPP; base < g; base += waves * HPP) {
        float x[8];
        const int head = kvh * g + min(base + sub, g - 1);   // lanes past the group repeat its last head
        load8_sum_wide(fused.qkv, (size_t)row * fused.row_elems + (size_t)head * DMAX + chunk * 8, fused.splits, fused.split_stride, x);
        add_bias8(x, fused.bias, head * DMAX + chunk * 8);
        norm_rope8<bf16_t>(x, chunk, TG, fused.q_weight, DMAX, fused.eps, fused.cos_table, fused.sin_table, pos, fused.rot,
                           fused.rotate_first != 0);
        if (fused.temp_every > 0) {
          const float temperature = query_temperature(pos, fused.temp_coef, fused.temp_every);
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] *= temperature;
        }
        if (base + sub < g) shared_q[(base + sub) * TG + chunk] = pack8(x);
      }
      owner = fused.writes && pos_place >= begin && pos_place < end && wave == ((pos_place >> 5) - first_step) % waves;
      if (owner) {                                           // wave-uniform
        float x[8];
        load8_sum_wide(fused.qkv, (size_t)row * fused.row_elems + (size_t)(heads + kvh) * DMAX + chunk * 8, fused.splits, fused.split_stride, x);
        add_bias8(x, fused.bias, (heads + kvh) * DMAX + chunk * 8);
        norm_rope8<bf16_t>(x, chunk, TG, fused.k_weight, DMAX, fused.eps, fused.cos_table, fused.sin_table, pos, fused.rot,
                           fused.rotate_first != 0);
        new_k = pack8(x);
        load8_sum_wide(fused.qkv, (size_t)row * fused.row_elems + (size_t)(fused.v_head + kvh) * DMAX + chunk * 8, fused.splits,
                       fused.split_stride, x);
        add_bias8(x, fused.bias, (fused.v_head + kvh) * DMAX + chunk * 8);
        new_v = pack8(x);
        if (sub == 0) {                                      // into the pages (qil/cache.py:79-82)
          const size_t page = table[pos / page_size];
          const int offset = pos % page_size;
          bf16_t* k_row = const_cast<bf16_t*>(k_cache) + ((page * kv_heads + kvh) * page_size + offset) * (size_t)DMAX;
          *reinterpret_cast<uint4*>(k_row + chunk * 8) = new_k;
          bf16_t* column = const_cast<bf16_t*>(v_cache) + ((page * kv_heads + kvh) * (size_t)DMAX + chunk * 8) * page_size + offset;
          const uint32_t words[4] = {new_v.x, new_v.y, new_v.z, new_v.w};
#pragma unroll
          for (int e = 0; e < 8; ++e) column[(size_t)e * page_size] = (bf16_t)(words[e >> 1] >> ((e & 1) * 16));
        }
      }
      __syncthreads();
#pragma unroll
      for (int ks = 0; ks < QFRAGS; ++ks)                    // fragment ks of head r = chunk 4 ks + kb of that head
        qb[ks] = __builtin_bit_cast(bf16x8, r < g ? shared_q[r * TG + 4 * ks + kb] : make_uint4(0, 0, 0, 0));
      __syncthreads();                                       // the LDS is free again
    } else {
#pragma unroll
      for (int ks = 0; ks < QFRAGS; ++ks) {
        const int dim = ks * 32 + kb * 8;
        uint4 raw = make_uint4(0, 0, 0, 0);
        if (r < g && dim < d) raw = *reinterpret_cast<const uint4*>(q + (size_t)row * q_stride + (size_t)(kvh * g + r) * d + dim);
        qb[ks] = __builtin_bit_cast(bf16x8, raw);
      }
    }
  };
  // The loads of a wave's first step (or pair of steps) go out before its queries are made, so that the
  // two waits overlap; later steps are loaded when the step before is done.
  if (PAIRS) {
    // Two of the wave's steps at a time: both steps' table entries, then both steps' K and V, then the
    // arithmetic; a wave waits for memory twice per pair instead of twice per step.  (Twice the
    // registers: for launches that leave a CU's register file to one block.)
    int step = first_step + wave;
    int page_a[3], page_b[3];
    StepData a, b;
    auto load_pair = [&]() {
      look_up(step, page_a);
      if (step + waves <= last_step) look_up(step + waves, page_b);
      request(step, page_a, a);
      if (step + waves <= last_step) request(step + waves, page_b, b);
    };
    if (step <= last_step) load_pair();
    make_queries();
    while (step <= last_step) {
      attend(step, a);
      if (step + waves <= last_step) attend(step + waves, b);
      step += 2 * waves;
      if (step <= last_step) load_pair();
    }
  } else {
    int step = first_step + wave;
    int page[3];
    StepData data;
    if (step <= last_step) {
      look_up(step, page);
      request(step, page, data);
    }
    make_queries();
    while (step <= last_step) {
      attend(step, data);
      step += waves;
      if (step <= last_step) {
        look_up(step, page);
        request(step, page, data);
      }
    }
  }

  // ---- the waves' (m, l, O) meet in LDS: [wave][head < g][d + 2]
  l += __shfl_xor(l, 16, QIL_WAVE);
  l += __shfl_xor(l, 32, QIL_WAVE);
  const int cell = d + 2;
  if (r < g) {
    float* mine = lds + ((size_t)wave * g + r) * cell;
    if (kb == 0) { mine[d] = m; mine[d + 1] = l; }
#pragma unroll
    for (int t = 0; t < DTILES; ++t)
      if (t < dt)
#pragma unroll
        for (int i = 0; i < 4; ++i) mine[t * 16 + 4 * kb + i] = o[t][i];
  }
  __syncthreads();
  for (int idx = threadIdx.x; idx < g * d; idx += blockDim.x) {
    const int h = idx / d, e = idx - h * d;
    float mm = -INFINITY;
    for (int w = 0; w < waves; ++w) mm = fmaxf(mm, lds[((size_t)w * g + h) * cell + d]);
    float total = 0.f, ll = 0.f;
    for (int w = 0; w < waves; ++w) {                       // fixed order
      const float mw = lds[((size_t)w * g + h) * cell + d];
      const float f = mw == -INFINITY ? 0.f : __builtin_amdgcn_exp2f((mw - mm) * 1.44269504088896f);
      total += lds[((size_t)w * g + h) * cell + e] * f;
      ll += lds[((size_t)w * g + h) * cell + d + 1] * f;
    }
    const int head = kvh * g + h;
    if (parts == 1) {
      out[((size_t)row * heads + head) * d + e] =
          f32_to_bf16(sinks ? total * sink_reciprocal(ll, mm, sinks[head]) : total / ll);
    } else {
      const size_t c = ((size_t)slot_row * heads + head) * parts + part;
      part_acc[c * d + e] = total;
      if (e == 0) { part_m[c] = mm; part_l[c] = ll; }
    }
  }
}

// 1 if the matrix-core decode kernel takes these sizes.
extern "C" int qil_attn_decode_takes(int heads, int kv_heads, int d, int page_size) {
  if (heads % kv_heads || d % 16 || d < 16 || d > 256 || page_size % 8) return 0;
  const int g = heads / kv_heads;
  return g <= 16 && (size_t)DEC_MAX_WAVES * g * (d + 2) * sizeof(float) <= 64 * 1024;
}

// Partial results in the layout of the row kernel (acc [rows, heads, parts, d], then m, then l);
// the caller runs the row kernel's merge when parts > 1.  P must be a multiple of 32; a block has
// `waves` waves (at most 8), best one or two 32-key steps of P for each.  pairs != 0: a wave loads two of
// its steps at a time (twice the registers; for launches of at most one block a CU).  sinks: null, or float32 [heads]:
// exp(sink) joins a head's divisor (here when parts == 1, else in the merge).  slopes: null, or float32 [heads]; keep > 0
// (with a window): the kept first keys, and P and parts count places.
extern "C" int qil_attn_decode(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                               const int* block_tables, int table_stride, const int* row_seq, const int* positions,
                               const int* row_index, void* workspace, void* out, int rows, int heads, int kv_heads,
                               int d, int page_size, int window, float scale, int P, int parts, int waves,
                               int pairs, float softcap, const float* sinks, const float* slopes, int keep,
                               hipStream_t s) {
  if (rows == 0) return 0;
  if (!qil_attn_decode_takes(heads, kv_heads, d, page_size) || P % 32 || P < 32 || parts < 1 || parts > 65535 ||
      kv_heads > 65535 || waves < 1 || waves > DEC_MAX_WAVES || keep < 0 || (keep > 0 && window <= 0))
    return -1;
  const int g = heads / kv_heads;
  float* acc = (float*)workspace;
  float* m = acc ? acc + (size_t)rows * heads * parts * d : nullptr;
  float* l = m ? m + (size_t)rows * heads * parts : nullptr;
  const size_t lds = (size_t)waves * g * (d + 2) * sizeof(float);
  dim3 grid(rows, kv_heads, parts);
  const FusedQKV none = {};
#define QIL_DEC_LAUNCH(DMAX, PAIRS, FUSED, FIELDS)                                                                  \
  hipLaunchKernelGGL((attn_decode_kernel<DMAX, PAIRS, FUSED>), grid, dim3(waves * QIL_WAVE), lds, s, FIELDS,         \
                     (const bf16_t*)q, q_stride, (const bf16_t*)k_cache, (const bf16_t*)v_cache, block_tables,       \
                     table_stride, row_seq, positions, row_index, acc, m, l, (bf16_t*)out, heads, kv_heads, d,        \
                     page_size, window, scale, P, parts, softcap, sinks, slopes, keep)
#define QIL_DEC_WHOLE(DMAX, PAIRS)                                                                                  \
  hipLaunchKernelGGL((attn_decode_kernel<DMAX, PAIRS, false, true>), grid, dim3(waves * QIL_WAVE), lds, s, none,     \
                     (const bf16_t*)q, q_stride, (const bf16_t*)k_cache, (const bf16_t*)v_cache, block_tables,       \
                     table_stride, row_seq, positions, row_index, acc, m, l, (bf16_t*)out, heads, kv_heads, d,        \
                     page_size, window, scale, P, parts, softcap, sinks, slopes, keep)
#define QIL_DEC_CASE(DMAX)                                                                                          \
  if (d == DMAX && pairs) QIL_DEC_WHOLE(DMAX, true);                                                                \
  else if (d == DMAX) QIL_DEC_WHOLE(DMAX, false);                                                                   \
  else if (pairs) QIL_DEC_LAUNCH(DMAX, true, false, none);                                                          \
  else QIL_DEC_LAUNCH(DMAX, false, false, none)
  if (d <= 64) QIL_DEC_CASE(64);
  else if (d <= 128) QIL_DEC_CASE(128);
  else QIL_DEC_CASE(256);
#undef QIL_DEC_CASE
#undef QIL_DEC_WHOLE
  QIL_RETURN_LAUNCH_STATUS();
}

// 1 if the fused kernel (queries, new key and new value made from the q/k/v product's partial sums) takes
// the sizes: a head of exactly 64 or 128 elements (256 would not fit the registers), a rotated width the
// vector kernel of qk_rope.hip takes.
extern "C" int qil_attn_decode_fused_takes(int heads, int kv_heads, int d, int page_size, int rot) {
  if (!qil_attn_decode_takes(heads, kv_heads, d, page_size) || !(d == 64 || d == 128)) return 0;
  const int half_chunks = rot >> 4;
  return rot == 0 || (rot <= d && rot % 16 == 0 && (half_chunks & (half_chunks - 1)) == 0);
}

// qil_attn_decode with qkv [splits][rows][(heads + 2 kv_heads) d] float32 partial sums in the place of q; the
// rows are the step's rows 0 .. rows-1 (no row index).  q_weight, k_weight: both or neither; cos/sin: both
// [positions][rot / 2], or neither, or a cos_table alone that holds the rot / 2 frequencies (the angles are then made
// in the kernel).  rotate_first: rotate, then norm.  softcap > 0: scores are capped softly after the scale.  writes != 0: the new keys and values go into the caches at the rows'
// positions (the page comes from the block table).  has_kv 0: the rows of qkv hold queries only (a reader; writes must be 0).
// extra_columns: so many more columns follow in every row and are skipped.  bias: null, or float32 by column of q, k and v.
// temp_every > 0: the query temperature of qk_rope.hip.  sinks: null, or float32 [heads] (as in qil_attn_decode).
// shared_kv: the rows hold no values of their own; a value is its key as projected, before norm and rotation.
// slopes, keep: as in qil_attn_decode.
extern "C" int qil_attn_decode_fused(const float* qkv, int splits, const float* q_weight, const float* k_weight,
                                     float eps, const float* cos_table, const float* sin_table, int rot, int writes,
                                     void* k_cache, void* v_cache, const int* block_tables, int table_stride,
                                     const int* row_seq, const int* positions, void* workspace, void* out, int rows,
                                     int heads, int kv_heads, int d, int page_size, int window, float scale, int P,
                                     int parts, int waves, int pairs, int rotate_first, float softcap,
                                     int has_kv, int extra_columns, const float* bias, float temp_coef, int temp_every,
                                     const float* sinks, int shared_kv, const float* slopes, int keep, hipStream_t s) {
  if (rows == 0) return 0;
  if (keep < 0 || (keep > 0 && window <= 0) || (shared_kv && !has_kv)) return -1;
  if (extra_columns < 0 || temp_every < 0 || (writes && !has_kv) || ((uintptr_t)bias % 16) || extra_columns % 8) return -1;
  if (!qil_attn_decode_fused_takes(heads, kv_heads, d, page_size, cos_table ? rot : 0) || P % 32 || P < 32 ||
      parts < 1 || parts > 65535 || kv_heads > 65535 || waves < 1 || waves > DEC_MAX_WAVES || splits < 1 ||
      (q_weight == nullptr) != (k_weight == nullptr) || (sin_table != nullptr && cos_table == nullptr) ||
      (((uintptr_t)qkv | (uintptr_t)q_weight | (uintptr_t)k_weight | (uintptr_t)cos_table | (uintptr_t)sin_table |
        (uintptr_t)k_cache) % 16))
    return -1;
  const int g = heads / kv_heads;
  float* acc = (float*)workspace;
  float* m = acc ? acc + (size_t)rows * heads * parts * d : nullptr;
  float* l = m ? m + (size_t)rows * heads * parts : nullptr;
  const size_t lds = (size_t)waves * g * (d + 2) * sizeof(float);
  dim3 grid(rows, kv_heads, parts);
  FusedQKV fused;
  fused.qkv = qkv;
  fused.row_elems = (heads + (has_kv ? (shared_kv ? 1 : 2) * kv_heads : 0)) * d + extra_columns;
  fused.v_head = shared_kv ? heads : heads + kv_heads;
  fused.split_stride = (size_t)rows * fused.row_elems;
  fused.bias = bias; fused.temp_coef = temp_coef; fused.temp_every = temp_every;
  fused.splits = splits;
  fused.q_weight = q_weight; fused.k_weight = k_weight; fused.eps = eps;
  fused.cos_table = cos_table; fused.sin_table = sin_table; fused.rot = cos_table ? rot : 0;
  fused.rotate_first = rotate_first;
  fused.writes = writes;
  const void* q = nullptr;
  const int q_stride = 0;
  const int* row_index = nullptr;
#define QIL_DEC_CASE(DMAX)                                                                                          \
  if (pairs) QIL_DEC_LAUNCH(DMAX, true, true, fused);                                                               \
  else QIL_DEC_LAUNCH(DMAX, false, true, fused)
  if (d == 64) QIL_DEC_CASE(64);
  else QIL_DEC_CASE(128);
#undef QIL_DEC_CASE
#undef QIL_DEC_LAUNCH
  QIL_RETURN_LAUNCH_STATUS();
}
