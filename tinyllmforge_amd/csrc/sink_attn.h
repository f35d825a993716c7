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

// Queries are stored with the score's constants in them: q . k is the score times log2(e), or with a cap 2 log2(e) / cap times
// the score, so that cap log2(e) tanh(score / cap) takes one exponential and one reciprocal.
inline float sink_query_scale(float scale, float cap) { return scale * kSinkLog2e * (cap > 0.f ? 2.f / cap : 1.f); }
// The capped score (or the score) in units of log 2.
template <bool CAP>
__device__ __forceinline__ float sink_score_log2(float dot, float cap_log2) {
  if (!CAP) return dot;
  return fmaf(-2.f * cap_log2, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(dot)), cap_log2);
}

// acc *= back unless back is 1 in every lane.  Branch and multiplies are one block, so that the accumulators stay in their
// registers: behind a C++ branch the scaled values land in new ones, and the path that skips the rescale copies them all.
__device__ __forceinline__ void sink_rescale(floatx4 &x, floatx4 &y, float back) {
  const unsigned long long moved = __builtin_amdgcn_ballot_w64(back != 1.0f);
  float t[8] = {x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]};
  asm volatile(
      "s_cmp_eq_u64 %[m], 0\n\t"
      "s_cbranch_scc1 .Ltlf_sink_keep%=\n\t"
      "v_mul_f32_e32 %0, %[a], %0\n\tv_mul_f32_e32 %1, %[a], %1\n\tv_mul_f32_e32 %2, %[a], %2\n\tv_mul_f32_e32 %3, %[a], %3\n\t"
      "v_mul_f32_e32 %4, %[a], %4\n\tv_mul_f32_e32 %5, %[a], %5\n\tv_mul_f32_e32 %6, %[a], %6\n\tv_mul_f32_e32 %7, %[a], %7\n"
      ".Ltlf_sink_keep%=:"
      : "+v"(t[0]), "+v"(t[1]), "+v"(t[2]), "+v"(t[3]), "+v"(t[4]), "+v"(t[5]), "+v"(t[6]), "+v"(t[7])
      : [a] "v"(back), [m] "s"(moved)
      : "scc");
  x = floatx4{t[0], t[1], t[2], t[3]};
  y = floatx4{t[4], t[5], t[6], t[7]};
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
