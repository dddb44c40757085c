// Attention with two softmax maps a head over the same values, o = norm(a1 - factor a2): what surrounds the attention
// kernels, which run as they are on paired heads.  A key/value head's two keys lie one behind the other in one cached key
// [k1 | k2 | 0], and a head's two queries become the rows [q1 | 0 | 0] and [0 | q2 | 0] of two query heads of that size:
// their products with the cached key are q1 . k1 and q2 . k2 exactly (the rest of a sum are zeros), both rows read the
// same values, and neither key nor value is held or read twice.
//
//   pair_store          a row of the stacked product [q1 q2 a head | k1 k2 a kv head | v a kv head | ..] -> the two query
//                       rows a head, the key and the value (transposed in its page) in the cache;
//   difference_combine  the two results a head (or, for split contexts, the parts' unmerged results) -> their difference,
//                       over its root mean square, times a constant and sigmoid(gate logit), rounded once.
#include "common.h"
#include "operand.h"
#include "merge_parts.h"

// grid (tiles of 16 rows, pieces): a thread takes one row of the tile and one piece of V elements of an output head; 16
// neighbouring threads take the tile's rows, so that the transposed values of one page leave as runs of tokens.
template <typename T, int V>
__global__ void __launch_bounds__(256)
pair_store_kernel(Operand x, size_t row_elems, T* __restrict__ q, const int* __restrict__ slots, T* __restrict__ k_cache,
                  T* __restrict__ v_cache, int n, int heads, int kv_heads, int dim, int vdim, int padded, int page_size,
                  int pieces) {
  const int local = threadIdx.x & 15, piece = blockIdx.y * (256 / 16) + (threadIdx.x >> 4), row = blockIdx.x * 16 + local;
  if (row >= n || piece >= pieces) return;
  const int a_head = padded / V, head = piece / a_head, e = (piece - head * a_head) * V;
  // output head -> first source column of its element 0, and the range of elements that come from there
  int source, first, last;
  if (head < 2 * heads) {
    const int map = head & 1;
    first = map * dim;
    last = first + dim;
    source = (head >> 1) * 2 * dim;
  } else if (head < 2 * heads + kv_heads) {
    first = 0;
    last = 2 * dim;
    source = heads * 2 * dim + (head - 2 * heads) * 2 * dim;
  } else {
    first = 0;
    last = vdim;
    source = (heads + kv_heads) * 2 * dim + (head - 2 * heads - kv_heads) * vdim;
  }
  float v[V];
  const size_t at = (size_t)row * row_elems + source + e;
  if constexpr (V == 8) {                                   // (sizes in pieces of 8: a piece lies inside or outside)
    if (e >= first && e < last) {
      if (x.code == QIL_BF16) {
        ld8(reinterpret_cast<const bf16_t*>(x.data) + at, v);
      } else {
        const float4 a = operand_at4(x, at), b = operand_at4(x, at + 4);
        v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
      }
    } else {
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] = 0.f;
    }
  } else {
    v[0] = e >= first && e < last ? operand_at(x, at) : 0.f;
  }
  auto put = [&](T* to) {
    if constexpr (V == 8) {
      st4(to, make_float4(v[0], v[1], v[2], v[3]));
      st4(to + 4, make_float4(v[4], v[5], v[6], v[7]));
    } else {
      st(to, v[0]);
    }
  };
  if (head < 2 * heads) {
    put(q + ((size_t)row * 2 * heads + head) * padded + e);
    return;
  }
  if (!slots) return;
  const size_t slot = (size_t)slots[row], page = slot / page_size, in_page = slot % page_size;
  if (head < 2 * heads + kv_heads) {
    put(k_cache + ((page * kv_heads + head - 2 * heads) * page_size + in_page) * padded + e);
  } else {
    T* to = v_cache + ((page * kv_heads + head - 2 * heads - kv_heads) * padded + e) * page_size + in_page;
#pragma unroll
    for (int i = 0; i < V; ++i) st(to + (size_t)i * page_size, v[i]);
  }
}

// A (row, head) takes 2 L lanes, the first L the first map's elements, the others the second's, eight a lane (L = 16 up to 128
// elements, 32 up to 256): a lane and its partner L lanes away hold the same elements of both maps.  PARTS: the maps are the
// unmerged parts of a split context.
template <typename T, bool PARTS, int L>
__global__ void __launch_bounds__(256)
difference_combine_kernel(const T* __restrict__ maps, UnmergedA parts, Operand gate, size_t gate_row, float factor, float post,
                          float eps, T* __restrict__ out, int rows, int heads, int vdim, int padded, int vec_out) {
  const int item = blockIdx.x * (256 / (2 * L)) + threadIdx.x / (2 * L);
  const bool there = item < rows * heads;                   // (every lane takes part in the exchanges)
  const int row = there ? item / heads : 0, head = there ? item - row * heads : 0;
  const int map = (threadIdx.x / L) & 1, e = (threadIdx.x % L) * 8;
  const float g = operand_at(gate, (size_t)row * gate_row + head);
  float v[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = 0.f;
  if (e < padded) {
    if constexpr (PARTS) merged_values<8>(parts, row, (head * 2 + map) * padded + e, v);
    else ld8(maps + ((size_t)row * 2 * heads + head * 2 + map) * padded + e, v);
  }
  float squares = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float other = __shfl_xor(v[i], L, QIL_WAVE);
    const float d = map ? other - factor * v[i] : v[i] - factor * other;
    v[i] = e + i < vdim ? d : 0.f;
    squares += v[i] * v[i];
  }
#pragma unroll
  for (int o = 1; o < L; o <<= 1) squares += __shfl_xor(squares, o, QIL_WAVE);
  const float scale = post / sqrtf(squares / (float)vdim + eps) / (1.f + expf(-g));
  // both partners hold the difference: the first stores its first four elements, the second the last four
  const int first = map * 4;
  if (!there || e + first >= vdim) return;
  T* to = out + ((size_t)row * heads + head) * vdim + e + first;
  const float y[4] = {(map ? v[4] : v[0]) * scale, (map ? v[5] : v[1]) * scale, (map ? v[6] : v[2]) * scale, (map ? v[7] : v[3]) * scale};
  if (vec_out) {
    st4(to, make_float4(y[0], y[1], y[2], y[3]));
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (e + first + i < vdim) st(to + i, y[i]);
  }
}

extern "C" {

// x: an operand of n rows of row_elems elements (split stride n * row_elems), columns [heads * 2 * dim queries | kv_heads *
// 2 * dim keys | kv_heads * vdim values | ..] (kv_heads 0: queries only).  padded >= max(2 dim, vdim), a multiple of 8.
int qil_pair_store(const void* x, int code, int splits, int row_elems, void* q, const int* slots, void* k_cache, void* v_cache,
                   int n, int heads, int kv_heads, int dim, int vdim, int padded, int page_size, int dtype, hipStream_t s) {
  if (n == 0) return 0;
  if (heads < 1 || kv_heads < 0 || dim < 1 || vdim < 1 || padded % 8 || padded < 2 * dim || (kv_heads && padded < vdim) ||
      row_elems < (heads + kv_heads) * 2 * dim + kv_heads * vdim || splits < 1 || (code == QIL_BF16 && splits != 1) ||
      (dtype == QIL_F32 && code != QIL_F32) || (slots && (page_size < 1 || !k_cache || !v_cache || kv_heads < 1)))
    return -1;
  const Operand in{x, code, splits, (size_t)n * row_elems};
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && row_elems % 8 == 0 &&
                   (((uintptr_t)x | (uintptr_t)q | (uintptr_t)k_cache) % 16) == 0;
  const int pieces = (2 * heads + (slots ? 2 * kv_heads : 0)) * (padded / (vec ? 8 : 1));
  const dim3 grid((n + 15) / 16, (pieces + 15) / 16);
  if (grid.y > 65535) return -1;
#define QIL_PS(T, V)                                                                                                  \
  hipLaunchKernelGGL((pair_store_kernel<T, V>), grid, dim3(256), 0, s, in, (size_t)row_elems, (T*)q, slots, (T*)k_cache, \
                     (T*)v_cache, n, heads, kv_heads, dim, vdim, padded, page_size, pieces)
  if (dtype == QIL_F32) { if (vec) QIL_PS(float, 8); else QIL_PS(float, 1); }
  else { if (vec) QIL_PS(bf16_t, 8); else QIL_PS(bf16_t, 1); }
#undef QIL_PS
  QIL_RETURN_LAUNCH_STATUS();
}

// maps [rows, 2 heads, padded] of dtype (a head's two results one behind the other), or workspace: the unmerged parts of a
// split context as attn_rows leaves them (acc [rows, 2 heads, n_parts, padded], m, l), part keys each.  gate: an operand of
// rows of gate_row elements, head h's logit at column h.  out [rows, heads * vdim].
int qil_difference_combine(const void* maps, const float* workspace, const int* positions, int window, int part, int n_parts,
                           const void* gate, int gate_code, int gate_splits, int gate_row, float factor, float post, float eps,
                           void* out, int rows, int heads, int vdim, int padded, int dtype, hipStream_t s) {
  if (rows == 0) return 0;
  if ((!maps) == (!workspace) || !gate || gate_splits < 1 || (gate_code == QIL_BF16 && gate_splits != 1) || gate_row < heads ||
      padded % 8 || padded > 256 || vdim > padded || vdim < 1 || (workspace && (!positions || part < 1 || n_parts < 1)))
    return -1;
  UnmergedA u{};
  if (workspace) {
    const size_t cells = (size_t)rows * 2 * heads * n_parts;
    u = UnmergedA{workspace, workspace + cells * padded, workspace + cells * (padded + 1), positions, 2 * heads, padded, n_parts, part, window};
  }
  const Operand g{gate, gate_code, gate_splits, (size_t)rows * gate_row};
  const int vec_out = vdim % 4 == 0 && (uintptr_t)out % 16 == 0;
  const int a_block = padded <= 128 ? 8 : 4;
  const dim3 grid((rows * heads + a_block - 1) / a_block);
#define QIL_DC(T, P)                                                                                                  \
  do {                                                                                                                \
    if (padded <= 128)                                                                                                \
      hipLaunchKernelGGL((difference_combine_kernel<T, P, 16>), grid, dim3(256), 0, s, (const T*)maps, u, g, (size_t)gate_row, \
                         factor, post, eps, (T*)out, rows, heads, vdim, padded, vec_out);                              \
    else                                                                                                              \
      hipLaunchKernelGGL((difference_combine_kernel<T, P, 32>), grid, dim3(256), 0, s, (const T*)maps, u, g, (size_t)gate_row, \
                         factor, post, eps, (T*)out, rows, heads, vdim, padded, vec_out);                              \
  } while (0)
  if (dtype == QIL_F32) { if (workspace) QIL_DC(float, true); else QIL_DC(float, false); }
  else { if (workspace) QIL_DC(bf16_t, true); else QIL_DC(bf16_t, false); }
#undef QIL_DC
  QIL_RETURN_LAUNCH_STATUS();
}

}  // extern "C"
