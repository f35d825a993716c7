// Geometry shared by the kernels of causal grouped-query attention with a sink, a score cap and an output gate
// (sink_attn.hip, sink_decode.hip, sink_prefill.hip).
//
// A query at position i sees the tokens 0 .. i.  Its score with a key is s = scale (q . k), capped to cap tanh(s / cap) where
// there is a cap; the weights are exp(s) / (sum of exp(s) + exp(sink)), sink a number per query head; each head's mix of
// values is multiplied element by element with sigmoid(gate).
//
// Caches are paged and head-major, K [pages, G, bs, Dp] and V [pages, G, bs, Vp]: the tokens of a page that one KV head
// reads are one contiguous piece.  Dp, Vp are the head dimensions rounded up to 32; pads hold zeros.
#pragma once
#include "elem.h"

namespace tlf {

struct SinkCache {
  const void *k, *v;
  const int32_t *bt;      // block tables, one row per sequence
  int64_t bt_stride;
  int32_t bs, G, D, Dv, Dp, Vp;
  int64_t pages;
  int32_t bs_shift;       // log2 of bs, -1 if it is no power of two
};

constexpr float kSinkLog2e = 1.4426950408889634f;

__device__ __forceinline__ int sink_page_of(const SinkCache &c, int j) { return c.bs_shift >= 0 ? j >> c.bs_shift : j / c.bs; }
// Cache row (units of Dp or Vp elements) of token j of a page's KV head; an unmapped page reads page 0 (never visible).
__device__ __forceinline__ int64_t sink_row(const SinkCache &c, int page, int pg, int kvh, int j) {
  const int64_t p = page >= 0 && page < c.pages ? page : 0;
  return (p * c.G + kvh) * c.bs + (j - pg * c.bs);
}

// Scores in units of log 2.  With a cap: cap log2(e) tanh(s / cap) from one exponential and one reciprocal.
struct SinkScore {
  float scale_log2;       // scale * log2(e)
  float cap_log2, turn;   // cap * log2(e), 2 scale log2(e) / cap; cap_log2 0: no cap
};
inline SinkScore sink_score(float scale, float cap) {
  return SinkScore{scale * kSinkLog2e, cap > 0.f ? cap * kSinkLog2e : 0.f, cap > 0.f ? 2.f * scale * kSinkLog2e / cap : 0.f};
}
template <bool CAP>
__device__ __forceinline__ float sink_score_log2(float dot, const SinkScore &s) {
  if (!CAP) return dot * s.scale_log2;
  return fmaf(-2.f * s.cap_log2, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(dot * s.turn)), s.cap_log2);
}

inline int sink_cache_make(SinkCache &c, const void *k, const void *v, const int32_t *bt, int64_t bt_stride, int32_t bs, int32_t G,
                           int32_t D, int32_t Dv, int64_t pages) {
  if (bs <= 0 || bs % 64 || G <= 0 || D <= 0 || Dv <= 0 || D > 512 || Dv > 512 || pages <= 0) return TLF_E_SHAPE;
  if (pages * G * bs > (int64_t{1} << 40)) return TLF_E_SHAPE;
  if (!k || !v) return TLF_E_NULL;
  if (!aligned16(k) || !aligned16(v)) return TLF_E_ALIGN;
  c = SinkCache{k, v, bt, bt_stride, bs, G, D, Dv, (D + 31) / 32 * 32, (Dv + 31) / 32 * 32, pages,
                (bs & (bs - 1)) == 0 ? __builtin_ctz(bs) : -1};
  return TLF_OK;
}

}  // namespace tlf
