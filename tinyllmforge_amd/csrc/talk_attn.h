// Geometry shared by the kernels of causal grouped-query attention whose heads mix their weights after the softmax
// (talk_attn.hip, talk_decode.hip, talk_prefill.hip).
//
//   w_h(i, j) = softmax over j <= i of scale temp_h (q_h . k);  out_h = sum_j (sum_g talk[h, g] w_g(i, j)) v_(h / group)(j)
//
// A head's output needs every head's denominator, so scores come first, mixes second.  Caches are those of sink_attn.h:
// K [pages, G, bs, Dp] and V [pages, G, bs, Vp], Dp and Vp the head dimensions rounded up to 32, pads are zeros.  Queries are
// stored with the score's constants in them: q . k is the score in units of log 2.
#pragma once
#include "sink_attn.h"

namespace tlf {

struct TalkRowsArgs {
  SinkCache c;
  const void *q;             // [rows, H, Dp]
  const void *talk;          // [H, H]
  const int64_t *positions;  // [rows]
  const int32_t *slots;      // [rows], negative: padding row
  const int32_t *row_seq;    // [rows] or NULL: row r belongs to sequence r
  void *out;                 // [rows, ldo]
  int64_t ldo;
  float *scores;             // [rows, H, keys] log 2 units
  float *part_ml;            // [splits, rows, H, 2]: maximum, sum
  float *part_o;             // [splits, rows, H, Vp]
  int32_t keys;              // max_len rounded up to 64
  int32_t rows, H, group, per_pass, passes, splits, least, max_len;
};

// A row's keys are cut into pieces of equal length, a multiple of 64 and at least `least`, so short rows use few of the splits.
// Split `split` has keys [lo, hi); returns how many splits the row uses, 0 for a padding row.
__device__ __forceinline__ int talk_split(const TalkRowsArgs &a, int64_t row, int split, int &lo, int &hi) {
  const int64_t i = a.positions[row];
  lo = hi = 0;
  if (a.slots[row] < 0 || i < 0 || i >= a.max_len) return 0;
  const int total = static_cast<int>(i) + 1, per = max(((total + a.splits - 1) / a.splits + 63) & ~63, a.least);
  lo = min(total, split * per);
  hi = min(total, lo + per);
  return (total + per - 1) / per;
}

__device__ __forceinline__ shortx4 talk_read_tr16(const unsigned short *p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p));
}

// Eight fp32 values as a bf16 pair, hi + lo: 16 significant bits.
__device__ __forceinline__ void talk_pair(const float (&w)[8], bf16x8 &hi, bf16x8 &lo) {
  unsigned int h[4], l[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    h[e] = pack_bf16x2(w[2 * e], w[2 * e + 1]);
    l[e] = pack_bf16x2(w[2 * e] - __uint_as_float(h[e] << 16), w[2 * e + 1] - __uint_as_float(h[e] & 0xffff0000u));
  }
  hi = __builtin_bit_cast(bf16x8, make_uint4(h[0], h[1], h[2], h[3]));
  lo = __builtin_bit_cast(bf16x8, make_uint4(l[0], l[1], l[2], l[3]));
}

}  // namespace tlf
