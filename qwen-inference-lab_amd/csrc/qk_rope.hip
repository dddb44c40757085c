// Fused per-head RMSNorm of q and k, rotary encoding, and the write of k and v into the pages.
//
// qkv[N, (heads + 2 kv_heads) * d]: head h of q at columns [h d, (h+1) d), then the k heads, then the
// v heads; in the model's type T, or float32 partial sums [splits][N][..] of a K-split product, added
// here in split order.  One wave per (token, head).  All arithmetic is float32 and a value is
// rounded to T once, when it is stored (the reference rounds after the norm, of cos and sin, and
// after every product: qil/model.py:15-23,42-46,52-55).
//   q heads: norm -> rotate -> stored into q_out[N, heads * d]
//   k heads: norm -> rotate -> stored into k_cache at the token's slot
//   v heads: copied into v_cache at the token's slot
// Cache layouts, slot = page * page_size + offset (qil/cache.py:79-82):
//   K [pages, kv_heads, page_size, d]   a key's d elements are contiguous (the score product sums over d)
//   V [pages, kv_heads, d, page_size]   a dim's keys are contiguous (the value product sums over keys), so
//                                       the attention kernels load matrix-core operands for P V directly
// Rotation pairs (i, i + rot/2), i < rot/2 (qil/model.py:42-46); elements from rot on pass unrotated.
#include "common.h"
#include "qk_math.h"

#define QIL_MAX_HEAD_DIM 512

// Loads go out eight at a time before the first is used; the additions stay in split order.
template <typename TD>
__device__ __forceinline__ float load_sum(const TD* __restrict__ base, size_t index, int splits, size_t stride) {
  float v = 0.f;
  for (int s0 = 0; s0 < splits; s0 += 8) {
    float part[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) part[u] = s0 + u < splits ? ld(base + (s0 + u) * stride + index) : 0.f;
#pragma unroll
    for (int u = 0; u < 8; ++u) v += part[u];
  }
  return v;
}

template <typename TD, typename T>
__global__ void qk_norm_rope_store_kernel(
    const TD* __restrict__ qkv, int splits, size_t split_stride, T* __restrict__ q_out,
    const float* __restrict__ q_weight, const float* __restrict__ k_weight,
    const float* __restrict__ cos_table, const float* __restrict__ sin_table, const int* __restrict__ positions,
    const int* __restrict__ slots, T* __restrict__ k_cache, T* __restrict__ v_cache,
    int heads, int kv_heads, int d, int rot, int page_size, float eps, int norm_dim, int rotate_first, int row_elems,
    float temp_coef, int temp_every, const float* __restrict__ bias, int v_head) {
  __shared__ float vec[QIL_MAX_HEAD_DIM];
  const int n = blockIdx.x, head = blockIdx.y, lane = threadIdx.x;
  const int piece = head < heads + kv_heads ? head : head - heads - kv_heads + v_head;     // head-sized piece of the row
  const size_t src = (size_t)n * row_elems + (size_t)piece * d;   // index into qkv
  const bool is_q = head < heads, is_k = !is_q && head < heads + kv_heads;
  if (!is_q && slots == nullptr) return;                 // a reader of another entry's cache writes no k/v

  T* dst = q_out + ((size_t)n * heads + head) * d;
  if (!is_q) {
    const int kvh = is_k ? head - heads : head - heads - kv_heads;
    const int slot = slots[n];
    const size_t page = slot / page_size, offset = slot % page_size;
    if (is_k) {
      dst = k_cache + ((page * kv_heads + kvh) * page_size + offset) * d;
    } else {                                             // v: copy, transposed within the page
      T* column = v_cache + (page * kv_heads + kvh) * (size_t)d * page_size + offset;
      for (int i = lane; i < d; i += QIL_WAVE)
        st(column + (size_t)i * page_size, load_sum(qkv, src + i, splits, split_stride) + (bias ? bias[piece * d + i] : 0.f));
      return;
    }
  }

  const float* weight = is_q ? q_weight : k_weight;
  for (int i = lane; i < d; i += QIL_WAVE)
    vec[i] = load_sum(qkv, src + i, splits, split_stride) + (bias ? bias[piece * d + i] : 0.f);
  __syncthreads();
  const int half = rot / 2;
  const int position = positions[n];
  const float temperature = is_q ? query_temperature(position, temp_coef, temp_every) : 1.f;
  const bool rotates = cos_table && rot > 0;
  // one element of the rotated head: from the tables, or (no sine table) from the frequencies the cosine table's place holds
  auto turned = [&](int i) {
    if (!rotates || i >= rot) return vec[i];
    const int f = i < half ? i : i - half;
    float sn, cs;
    if (sin_table) { cs = cos_table[(size_t)position * half + f]; sn = sin_table[(size_t)position * half + f]; }
    else sincosf((float)position * cos_table[f], &sn, &cs);
    return i < half ? vec[i] * cs - vec[i + half] * sn : vec[i - half] * sn + vec[i] * cs;
  };
  if (rotate_first) {                                    // rotate, then norm what was rotated
    float mine[QIL_MAX_HEAD_DIM / QIL_WAVE], sum = 0.f;
#pragma unroll
    for (int u = 0; u < QIL_MAX_HEAD_DIM / QIL_WAVE; ++u) {
      const int i = lane + u * QIL_WAVE;
      mine[u] = i < d ? turned(i) : 0.f;
      sum += mine[u] * mine[u];
    }
    float rstd = 1.f;
    if (weight) rstd = rsqrtf(wave_sum(sum) / (float)norm_dim + eps);
#pragma unroll
    for (int u = 0; u < QIL_MAX_HEAD_DIM / QIL_WAVE; ++u) {
      const int i = lane + u * QIL_WAVE;
      if (i < d) st(dst + i, (weight ? round_to<T>(mine[u] * rstd) * weight[i] : mine[u]) * temperature);
    }
    return;
  }
  if (weight) {
    float sum = 0.f;
    for (int i = lane; i < d; i += QIL_WAVE) sum += vec[i] * vec[i];
    sum = wave_sum(sum);
    const float rstd = rsqrtf(sum / (float)norm_dim + eps);
    for (int i = lane; i < d; i += QIL_WAVE) vec[i] = round_to<T>(vec[i] * rstd) * weight[i];
    __syncthreads();
  }
  for (int i = lane; i < d; i += QIL_WAVE) st(dst + i, turned(i) * temperature);
}

// The same work with eight consecutive elements a lane (16-byte vectors) and no LDS: a head is spread
// over TG = d / 8 lanes (a power of two), a wave serves 64 / TG (token, head) pairs, the statistics are
// reduced and the rotation partner (TG lanes... rot / 16 lanes away) is fetched with lane shuffles.
// Takes d in {16, 32, 64, 128, 256} and a rotated width whose half is a power-of-two number of
// 8-element chunks (rot == d always qualifies).
template <typename TD, typename T>
__global__ void __launch_bounds__(256)
qk_norm_rope_store_vec_kernel(
    const TD* __restrict__ qkv, int splits, size_t split_stride, T* __restrict__ q_out,
    const float* __restrict__ q_weight, const float* __restrict__ k_weight, const float* __restrict__ cos_table,
    const float* __restrict__ sin_table, const int* __restrict__ positions, const int* __restrict__ slots,
    T* __restrict__ k_cache, T* __restrict__ v_cache, int n, int heads, int kv_heads, int d, int rot, int page_size,
    float eps, int tg_log2, unsigned v_first_block, int norm_dim, int rotate_first, int row_elems, float temp_coef,
    int temp_every, const float* __restrict__ bias, int v_head) {
  const int total_heads = heads + 2 * kv_heads;
  const int TG = 1 << tg_log2;
  if (blockIdx.x >= v_first_block) {
    // v apart (TG >= 4): a wave takes 16 tokens x 4 chunks of one head, so that a store instruction (one
    // element of every lane's chunk) fills 32 contiguous bytes per chunk when the tokens follow each other
    // in a page, instead of touching 64 lines with 2 bytes each.  v: copy, transposed within the page.
    const int lane = threadIdx.x & (QIL_WAVE - 1);
    const size_t wave = (size_t)(blockIdx.x - v_first_block) * (blockDim.x / QIL_WAVE) + threadIdx.x / QIL_WAVE;
    const int quads = TG >> 2;
    const int quad = (int)(wave % quads), kvh = (int)(wave / quads % kv_heads);
    const size_t group = wave / quads / kv_heads;
    const size_t token = group * 16 + (lane >> 2);
    const int chunk = quad * 4 + (lane & 3);
    if (token >= (size_t)n) return;
    float x[8];
    load8_sum(qkv, token * row_elems + (size_t)(v_head + kvh) * d + chunk * 8, splits, split_stride, x);
    add_bias8(x, bias, (v_head + kvh) * d + chunk * 8);
    const int slot = slots[token];
    const size_t page = slot / page_size, offset = slot % page_size;
    T* column = v_cache + ((page * kv_heads + kvh) * (size_t)d + chunk * 8) * page_size + offset;
#pragma unroll
    for (int e = 0; e < 8; ++e) st(column + (size_t)e * page_size, x[e]);
    return;
  }
  const int pair_heads = v_first_block != 0xffffffffu ? heads + kv_heads : total_heads;   // v apart: q and k only here
  const int pair = (int)((blockIdx.x * (size_t)blockDim.x + threadIdx.x) >> tg_log2);    // (token, head) pair
  const int chunk = threadIdx.x & (TG - 1);
  if (pair >= n * pair_heads) return;                   // whole lane groups leave together
  const int token = pair / pair_heads, head = pair - token * pair_heads;
  const bool is_q = head < heads, is_k = !is_q && head < heads + kv_heads;
  if (!is_q && slots == nullptr) return;
  float x[8];
  const int piece = is_q || is_k ? head : head - heads - kv_heads + v_head;
  load8_sum(qkv, (size_t)token * row_elems + (size_t)piece * d + chunk * 8, splits, split_stride, x);
  add_bias8(x, bias, piece * d + chunk * 8);

  if (!is_q && !is_k) {                                 // v: copy, transposed within the page
    const int kvh = head - heads - kv_heads, slot = slots[token];
    const size_t page = slot / page_size, offset = slot % page_size;
    T* column = v_cache + ((page * kv_heads + kvh) * (size_t)d + chunk * 8) * page_size + offset;
#pragma unroll
    for (int e = 0; e < 8; ++e) st(column + (size_t)e * page_size, x[e]);
    return;
  }
  norm_rope8<T>(x, chunk, TG, is_q ? q_weight : k_weight, norm_dim, eps, cos_table, sin_table, positions[token], rot,
                rotate_first != 0);
  if (is_q) {
    if (temp_every > 0) {
      const float temperature = query_temperature(positions[token], temp_coef, temp_every);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] *= temperature;
    }
    store8(q_out + ((size_t)token * heads + head) * d + chunk * 8, x);
  } else {
    const int kvh = head - heads, slot = slots[token];
    const size_t page = slot / page_size, offset = slot % page_size;
    store8(k_cache + ((page * kv_heads + kvh) * page_size + offset) * (size_t)d + chunk * 8, x);
  }
}

// sin_table null with a cos_table: cos_table holds the rot / 2 float32 frequencies and the kernels make the angle
// position * frequency, its cosine and sine themselves.  rotate_first: rotate, then norm (else norm, then rotate).
// qkv: in_dtype QIL_BF16 (one array, splits == 1) or QIL_F32 ([splits][n][..] partial sums).  dtype: type
// of q_out and of the caches.  norm_dim: the number of elements the head norm's mean runs over (0: d); smaller
// than d when the heads are padded with zeros to a size the attention kernels take.
// extra_columns: so many more columns follow the v heads in every row of qkv (another branch's part of a stacked
// product); they are skipped.  kv_heads 0: the rows hold queries only (a reader of another entry's cache).
// bias: null, or float32 [(heads + 2 kv_heads) d]: the projection's bias, added to the sums as they are loaded (the
// product before this kernel then needs none, and may leave partial sums).
// shared_kv: the rows hold no values of their own; a value is its key as projected, before norm and rotation.
// temp_every > 0: the query at position p is multiplied by 1 + temp_coef * ln(floor((p + 1) / temp_every) + 1) last.
extern "C" int qil_qk_norm_rope_store(
    const void* qkv, int in_dtype, int splits, void* q_out, const float* q_weight, const float* k_weight,
    const float* cos_table, const float* sin_table, const int* positions, const int* slots, void* k_cache,
    void* v_cache, int n, int heads, int kv_heads, int d, int rot, int page_size, float eps, int norm_dim, int rotate_first,
    int extra_columns, float temp_coef, int temp_every, const float* bias, int shared_kv, int dtype, hipStream_t s) {
  if (n == 0) return 0;
  if (extra_columns < 0 || temp_every < 0 || kv_heads < 0 || (kv_heads == 0 && slots)) return -1;
  const int row_elems = (heads + (shared_kv ? 1 : 2) * kv_heads) * d + extra_columns;
  const int v_head = shared_kv ? heads : heads + kv_heads;
  if (norm_dim == 0) norm_dim = d;
  if (norm_dim < 1 || norm_dim > d) return -1;
  if (d > QIL_MAX_HEAD_DIM || rot > d || (rot & 1) || splits < 1 || (in_dtype == QIL_BF16 && splits != 1)) return -1;
  if (dtype == QIL_F32 && in_dtype != QIL_F32) return -1;
  const size_t stride = (size_t)n * row_elems;
  dim3 grid(n, heads + 2 * kv_heads);
  // vector kernel: d / 8 a power of two up to 32, half of the rotated width a power-of-two number of chunks
  int tg_log2 = -1;
  for (int b = 1; b <= 5; ++b)
    if (d == (8 << b)) tg_log2 = b;
  const int half_chunks = rot >> 4;
  const bool rot_fits = rot == 0 || !cos_table || (rot % 16 == 0 && (half_chunks & (half_chunks - 1)) == 0);
  const bool aligned = row_elems % 8 == 0 &&
                       (((uintptr_t)qkv | (uintptr_t)q_out | (uintptr_t)k_cache | (uintptr_t)q_weight | (uintptr_t)k_weight |
                         (uintptr_t)cos_table | (uintptr_t)sin_table | (uintptr_t)bias) % 16) == 0;
  if (tg_log2 > 0 && rot_fits && aligned) {
    // v in blocks of its own behind the others when a head has at least four chunks and there is a cache to write
    const bool v_apart = tg_log2 >= 2 && slots != nullptr;
    const size_t lanes = (size_t)n * (v_apart ? heads + kv_heads : heads + 2 * kv_heads) << tg_log2;
    const unsigned pair_blocks = (unsigned)((lanes + 255) / 256);
    const size_t v_waves = v_apart ? (size_t)((n + 15) / 16) * kv_heads * ((size_t)1 << (tg_log2 - 2)) : 0;
    const unsigned v_first_block = v_apart ? pair_blocks : 0xffffffffu;
    const unsigned blocks = pair_blocks + (unsigned)((v_waves + 3) / 4);
#define QIL_QKV_CASE(TD, T)                                                                                           \
  hipLaunchKernelGGL((qk_norm_rope_store_vec_kernel<TD, T>), dim3(blocks), dim3(256), 0, s, (const TD*)qkv, splits,    \
                     stride, (T*)q_out, q_weight, k_weight, cos_table, sin_table, positions, slots, (T*)k_cache,       \
                     (T*)v_cache, n, heads, kv_heads, d, rot, page_size, eps, tg_log2, v_first_block, norm_dim, rotate_first,       \
                     row_elems, temp_coef, temp_every, bias, v_head)
    if (dtype == QIL_F32) QIL_QKV_CASE(float, float);
    else if (in_dtype == QIL_F32) QIL_QKV_CASE(float, bf16_t);
    else QIL_QKV_CASE(bf16_t, bf16_t);
#undef QIL_QKV_CASE
    QIL_RETURN_LAUNCH_STATUS();
  }
#define QIL_QK_CASE(TD, T)                                                                                            \
  hipLaunchKernelGGL((qk_norm_rope_store_kernel<TD, T>), grid, dim3(QIL_WAVE), 0, s, (const TD*)qkv, splits, stride,   \
                     (T*)q_out, q_weight, k_weight, cos_table, sin_table, positions, slots, (T*)k_cache, (T*)v_cache,  \
                     heads, kv_heads, d, rot, page_size, eps, norm_dim, rotate_first, row_elems, temp_coef, temp_every, bias, \
                     v_head)
  if (dtype == QIL_F32) QIL_QK_CASE(float, float);
  else if (in_dtype == QIL_F32) QIL_QK_CASE(float, bf16_t);
  else QIL_QK_CASE(bf16_t, bf16_t);
#undef QIL_QK_CASE
  QIL_RETURN_LAUNCH_STATUS();
}

// The same task with ONE norm over all query heads of a row and one over all its key heads (a norm of the whole
// projection, before it is split into heads): x / sqrt(sum(x^2) / norm_elems + eps) * weight[column], then the rotation, in
// float32 and rounded once.  Blocks 0 .. 2 n - 1 take a row's queries (even) or keys (odd), the row waiting in LDS
// between the statistics and the result; the blocks behind them take the values, a wave 16 tokens x 4 chunks of 8
// elements of one head, as in the vector kernel above.
template <typename TD, typename T>
__global__ void __launch_bounds__(256)
qk_row_norm_store_kernel(const TD* __restrict__ qkv, int splits, size_t split_stride, T* __restrict__ q_out,
                         const float* __restrict__ q_weight, const float* __restrict__ k_weight,
                         const float* __restrict__ cos_table, const float* __restrict__ sin_table,
                         const int* __restrict__ positions, const int* __restrict__ slots, T* __restrict__ k_cache,
                         T* __restrict__ v_cache, int n, int heads, int kv_heads, int d, int rot, int page_size, float eps,
                         float q_elems, float k_elems, int row_elems, int v_head) {
  extern __shared__ __align__(16) float row[];
  __shared__ float scratch[16];
  const int chunks = d / 8;
  if ((int)blockIdx.x >= 2 * n) {                        // values: copied, transposed within the page
    const int lane = threadIdx.x & (QIL_WAVE - 1), quads = (chunks + 3) / 4;
    const size_t wave = (size_t)(blockIdx.x - 2 * n) * (blockDim.x / QIL_WAVE) + threadIdx.x / QIL_WAVE;
    const int quad = (int)(wave % quads), kvh = (int)(wave / quads % kv_heads);
    const size_t token = wave / quads / kv_heads * 16 + (lane >> 2);
    const int chunk = quad * 4 + (lane & 3);
    if (token >= (size_t)n || chunk >= chunks) return;
    float x[8];
    load8_sum(qkv, token * row_elems + (size_t)(v_head + kvh) * d + chunk * 8, splits, split_stride, x);
    const int slot = slots[token];
    const size_t page = slot / page_size, offset = slot % page_size;
    T* column = v_cache + ((page * kv_heads + kvh) * (size_t)d + chunk * 8) * page_size + offset;
#pragma unroll
    for (int e = 0; e < 8; ++e) st(column + (size_t)e * page_size, x[e]);
    return;
  }
  const int token = blockIdx.x >> 1;
  const bool is_k = blockIdx.x & 1;
  if (is_k && slots == nullptr) return;                  // a reader of another entry's cache (the whole block)
  const int count = (is_k ? kv_heads : heads) * chunks;
  const size_t src = (size_t)token * row_elems + (is_k ? (size_t)heads * d : 0);
  float sum = 0.f;
  for (int c = threadIdx.x; c < count; c += blockDim.x) {
    float x[8];
    load8_sum(qkv, src + (size_t)c * 8, splits, split_stride, x);
#pragma unroll
    for (int e = 0; e < 8; ++e) sum += x[e] * x[e];
    store8(row + c * 8, x);
  }
  sum = block_sum(sum, scratch);                         // (its barriers also make the row whole)
  const float rstd = 1.f / sqrtf(sum / (is_k ? k_elems : q_elems) + eps);
  const float* weight = is_k ? k_weight : q_weight;
  const int half = rot / 2, position = positions[token];
  const bool rotates = cos_table && rot > 0;
  size_t page = 0, offset = 0;
  if (is_k) { page = slots[token] / page_size; offset = slots[token] % page_size; }
  for (int c = threadIdx.x; c < count; c += blockDim.x) {
    const int head = c / chunks, e0 = (c - head * chunks) * 8, base = head * d;
    float y[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int i = e0 + e;
      y[e] = row[base + i] * rstd * weight[base + i];
      if (rotates && i < rot) {
        const int f = i < half ? i : i - half, other = base + (i < half ? i + half : i - half);
        float sn, cs;
        if (sin_table) { cs = cos_table[(size_t)position * half + f]; sn = sin_table[(size_t)position * half + f]; }
        else sincosf((float)position * cos_table[f], &sn, &cs);
        const float z = row[other] * rstd * weight[other];
        y[e] = i < half ? y[e] * cs - z * sn : z * sn + y[e] * cs;
      }
    }
    T* dst = is_k ? k_cache + ((page * kv_heads + head) * page_size + offset) * (size_t)d + e0
                  : q_out + ((size_t)token * heads + head) * d + e0;
    store8(dst, y);
  }
}

// The same without a rotation, the row in registers: a block a row of queries (up to JQ chunks of 8 a thread), a wave a
// row of keys (up to JK chunks a lane, four tokens a block), then the values as above.
template <typename TD, typename T, int JQ, int JK>
__global__ void __launch_bounds__(256)
qk_row_norm_store_vec_kernel(const TD* __restrict__ qkv, int splits, size_t split_stride, T* __restrict__ q_out,
                             const float* __restrict__ q_weight, const float* __restrict__ k_weight,
                             const int* __restrict__ slots, T* __restrict__ k_cache, T* __restrict__ v_cache, int n, int heads,
                             int kv_heads, int d, int page_size, float eps, float q_elems, float k_elems, int row_elems,
                             int v_head, int k_blocks) {
  __shared__ float scratch[16];
  const int chunks = d / 8, lane = threadIdx.x & (QIL_WAVE - 1), wave_in_block = threadIdx.x / QIL_WAVE;
  if ((int)blockIdx.x < n) {                             // queries
    const int token = blockIdx.x, count = heads * chunks;
    const size_t src = (size_t)token * row_elems;
    float x[JQ][8], sum = 0.f;
#pragma unroll
    for (int j = 0; j < JQ; ++j) {
      const int c = min((int)threadIdx.x + j * 256, count - 1);
      load8_sum(qkv, src + (size_t)c * 8, splits, split_stride, x[j]);
    }
#pragma unroll
    for (int j = 0; j < JQ; ++j)
      if ((int)threadIdx.x + j * 256 < count) {
#pragma unroll
        for (int e = 0; e < 8; ++e) sum += x[j][e] * x[j][e];
      }
    sum = block_sum(sum, scratch);
    const float rstd = 1.f / sqrtf(sum / q_elems + eps);
#pragma unroll
    for (int j = 0; j < JQ; ++j) {
      const int c = threadIdx.x + j * 256;
      if (c < count) {
        float w[8];
        ld8(q_weight + (size_t)c * 8, w);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] = x[j][e] * rstd * w[e];
        store8(q_out + (size_t)token * heads * d + (size_t)c * 8, x[j]);
      }
    }
    return;
  }
  if ((int)blockIdx.x < n + k_blocks) {                  // keys
    const int token = ((int)blockIdx.x - n) * 4 + wave_in_block, count = kv_heads * chunks;
    if (token >= n) return;
    const size_t src = (size_t)token * row_elems + (size_t)heads * d;
    float x[JK][8], sum = 0.f;
#pragma unroll
    for (int j = 0; j < JK; ++j) {
      const int c = min(lane + j * QIL_WAVE, count - 1);
      load8_sum(qkv, src + (size_t)c * 8, splits, split_stride, x[j]);
    }
    const int slot = slots[token];
    const size_t page = slot / page_size, offset = slot % page_size;
#pragma unroll
    for (int j = 0; j < JK; ++j)
      if (lane + j * QIL_WAVE < count) {
#pragma unroll
        for (int e = 0; e < 8; ++e) sum += x[j][e] * x[j][e];
      }
    sum = wave_sum(sum);
    const float rstd = 1.f / sqrtf(sum / k_elems + eps);
#pragma unroll
    for (int j = 0; j < JK; ++j) {
      const int c = lane + j * QIL_WAVE;
      if (c < count) {
        float w[8];
        ld8(k_weight + (size_t)c * 8, w);
        const int head = c / chunks, e0 = (c - head * chunks) * 8;
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] = x[j][e] * rstd * w[e];
        store8(k_cache + ((page * kv_heads + head) * page_size + offset) * (size_t)d + e0, x[j]);
      }
    }
    return;
  }
  const int quads = (chunks + 3) / 4;                    // values: copied, transposed within the page
  const size_t wave = (size_t)((int)blockIdx.x - n - k_blocks) * 4 + wave_in_block;
  const int quad = (int)(wave % quads), kvh = (int)(wave / quads % kv_heads);
  const size_t token = wave / quads / kv_heads * 16 + (lane >> 2);
  const int chunk = quad * 4 + (lane & 3);
  if (token >= (size_t)n || chunk >= chunks) return;
  float x[8];
  load8_sum(qkv, token * row_elems + (size_t)(v_head + kvh) * d + chunk * 8, splits, split_stride, x);
  const int slot = slots[token];
  const size_t page = slot / page_size, offset = slot % page_size;
  T* column = v_cache + ((page * kv_heads + kvh) * (size_t)d + chunk * 8) * page_size + offset;
#pragma unroll
  for (int e = 0; e < 8; ++e) st(column + (size_t)e * page_size, x[e]);
}

// qkv, caches, slots, rotation, shared_kv, extra_columns: as in qil_qk_norm_rope_store (no bias, no temperature).
// q_weight float32 [heads * d], k_weight float32 [kv_heads * d]; q_elems, k_elems: the numbers of elements the two means
// run over (fewer than heads * d where the heads are padded with zeros).  d % 8 == 0 and 16-byte aligned rows.
extern "C" int qil_qk_row_norm_store(
    const void* qkv, int in_dtype, int splits, void* q_out, const float* q_weight, const float* k_weight,
    const float* cos_table, const float* sin_table, const int* positions, const int* slots, void* k_cache,
    void* v_cache, int n, int heads, int kv_heads, int d, int rot, int page_size, float eps, int q_elems, int k_elems,
    int extra_columns, int shared_kv, int dtype, hipStream_t s) {
  if (n == 0) return 0;
  if (heads < 1 || kv_heads < 1 || d < 8 || d % 8 || rot > d || (rot & 1) || splits < 1 || extra_columns < 0 ||
      extra_columns % 8 || (in_dtype == QIL_BF16 && splits != 1) || (dtype == QIL_F32 && in_dtype != QIL_F32) ||
      q_elems < 1 || q_elems > heads * d || k_elems < 1 || k_elems > kv_heads * d || !q_weight || !k_weight)
    return -1;
  const int row_elems = (heads + (shared_kv ? 1 : 2) * kv_heads) * d + extra_columns;
  const int v_head = shared_kv ? heads : heads + kv_heads;
  if (((uintptr_t)qkv | (uintptr_t)q_out | (uintptr_t)k_cache | (uintptr_t)q_weight | (uintptr_t)k_weight) % 16) return -1;
  const size_t lds = (size_t)(heads > kv_heads ? heads : kv_heads) * d * sizeof(float);
  if (lds > 128 * 1024) return -1;
  const size_t v_waves = slots ? (size_t)((n + 15) / 16) * kv_heads * ((d / 8 + 3) / 4) : 0;
  const dim3 grid((unsigned)(2 * (size_t)n + (v_waves + 3) / 4));
  const size_t stride = (size_t)n * row_elems;
  const int q_chunks = heads * d / 8, k_chunks = kv_heads * d / 8;
  if ((!cos_table || rot == 0) && q_chunks <= 1024 && k_chunks <= 256) {
    const int k_blocks = slots ? (n + 3) / 4 : 0;
    const dim3 blocks((unsigned)((size_t)n + k_blocks + (v_waves + 3) / 4));
#define QIL_ROW_VEC(TD, T, JQ, JK)                                                                                    \
  hipLaunchKernelGGL((qk_row_norm_store_vec_kernel<TD, T, JQ, JK>), blocks, dim3(256), 0, s, (const TD*)qkv, splits,   \
                     stride, (T*)q_out, q_weight, k_weight, slots, (T*)k_cache, (T*)v_cache, n, heads, kv_heads, d,    \
                     page_size, eps, (float)q_elems, (float)k_elems, row_elems, v_head, k_blocks)
#define QIL_ROW_VEC_J(TD, T)                                                                                          \
  do {                                                                                                                \
    if (q_chunks <= 256 && k_chunks <= 64) QIL_ROW_VEC(TD, T, 1, 1);                                                   \
    else if (q_chunks <= 512 && k_chunks <= 128) QIL_ROW_VEC(TD, T, 2, 2);                                             \
    else QIL_ROW_VEC(TD, T, 4, 4);                                                                                     \
  } while (0)
    if (dtype == QIL_F32) QIL_ROW_VEC_J(float, float);
    else if (in_dtype == QIL_F32) QIL_ROW_VEC_J(float, bf16_t);
    else QIL_ROW_VEC_J(bf16_t, bf16_t);
#undef QIL_ROW_VEC_J
#undef QIL_ROW_VEC
    QIL_RETURN_LAUNCH_STATUS();
  }
#define QIL_ROW_NORM(TD, T)                                                                                           \
  do {                                                                                                                \
    if (lds > 60 * 1024) {                                                                                            \
      hipError_t e = hipFuncSetAttribute((const void*)qk_row_norm_store_kernel<TD, T>,                                \
                                         hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                       \
      if (e != hipSuccess) return (int)e;                                                                             \
    }                                                                                                                 \
    hipLaunchKernelGGL((qk_row_norm_store_kernel<TD, T>), grid, dim3(256), lds, s, (const TD*)qkv, splits, stride,     \
                       (T*)q_out, q_weight, k_weight, cos_table, sin_table, positions, slots, (T*)k_cache,            \
                       (T*)v_cache, n, heads, kv_heads, d, rot, page_size, eps, (float)q_elems, (float)k_elems,        \
                       row_elems, v_head);                                                                            \
  } while (0)
  if (dtype == QIL_F32) QIL_ROW_NORM(float, float);
  else if (in_dtype == QIL_F32) QIL_ROW_NORM(float, bf16_t);
  else QIL_ROW_NORM(bf16_t, bf16_t);
#undef QIL_ROW_NORM
  QIL_RETURN_LAUNCH_STATUS();
}
