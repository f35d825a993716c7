// Geometry shared by the kernels of windowed attention with pooled blocks (pooled_attn.hip, pooled_prefill.hip).
//
// A query at position i sees the tokens j with 0 <= i - j < size and one mean key / mean value for every block of
// `pool` consecutive tokens that lies wholly before that window.  Token rows live in the paged K/V cache; the means
// live in a second paged cache with the same page numbers: a page of `bs` tokens owns C = ceil(bs / pool) mean rows,
// and a block's row is in the page of its last token.
#pragma once
#include "elem.h"

namespace tlf {

struct PooledCache {
  const void *k, *v;    // [pages, bs, G, Dp]
  const void *pk, *pv;  // [pages, C, G, Dp]
  const int32_t *bt;    // block tables, one row per sequence
  int64_t bt_stride;
  int32_t bs, pool, C, size;
  int32_t G, D, Dp;     // KV heads, head dimension, padded head dimension (a multiple of 32; pads hold zeros)
  int64_t pages;
  int32_t bs_shift;     // log2 of bs, -1 if it is no power of two
};
inline void pooled_cache_finish(PooledCache &c) {
  c.C = (c.bs + c.pool - 1) / c.pool;
  c.bs_shift = (c.bs & (c.bs - 1)) == 0 ? __builtin_ctz(c.bs) : -1;
}
__device__ __forceinline__ int page_of(const PooledCache &c, int j) { return c.bs_shift >= 0 ? j >> c.bs_shift : j / c.bs; }

// Blocks visible to position i.
__device__ __forceinline__ int pooled_visible(int i, int size, int pool) {
  const int past = i - size + 1;
  return past > 0 ? past / pool : 0;
}
// Cache row (units of G * Dp elements) of token j and of block b; an unmapped page reads row 0 (never visible).
__device__ __forceinline__ int64_t token_row(const PooledCache &c, const int32_t *bt, int j) {
  const int pg = page_of(c, j);
  const int64_t page = bt[pg];
  const bool ok = page >= 0 && page < c.pages;
  return ok ? page * c.bs + (j - pg * c.bs) : 0;
}
__device__ __forceinline__ int64_t block_row(const PooledCache &c, const int32_t *bt, int b) {
  const int pg = page_of(c, b * c.pool + c.pool - 1);
  const int64_t page = bt[pg];
  const bool ok = page >= 0 && page < c.pages;
  return ok ? page * c.C + (b - (pg * c.bs) / c.pool) : 0;
}

// Mean of the rows of block b, one KV head, written to the pooled cache: work item t of 2 * Dp / 8 (K chunks, then V).
template <typename T>
__device__ __forceinline__ void pool_block_chunk(const PooledCache &c, const int32_t *bt, int b, int kvh, int t) {
  const int nch = c.Dp / 8;
  const bool is_v = t >= nch;
  const int ch = is_v ? t - nch : t;
  const T *src = static_cast<const T *>(is_v ? c.v : c.k) + kvh * c.Dp + ch * 8;
  const int64_t rs = static_cast<int64_t>(c.G) * c.Dp;
  float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int r = 0; r < c.pool; ++r) {
    float f[8];
    Elem<T>::ld8(src + token_row(c, bt, b * c.pool + r) * rs, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] += f[e];
  }
  const float inv = 1.0f / static_cast<float>(c.pool);
#pragma unroll
  for (int e = 0; e < 8; ++e) acc[e] *= inv;
  T *dst = static_cast<T *>(const_cast<void *>(is_v ? c.pv : c.pk)) + kvh * c.Dp + ch * 8;
  Elem<T>::st8(dst + block_row(c, bt, b) * rs, acc);
}

// Unnormalised attention weight sigmoid(score), argument in units of log 2 with the sign already flipped.
__device__ __forceinline__ float sigmoid_neg_log2(float neg_score_log2) {
  return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(neg_score_log2));
}
constexpr float kLog2e = 1.4426950408889634f;

int pooled_cache_check(const PooledCache &c, int32_t dtype);

}  // namespace tlf
