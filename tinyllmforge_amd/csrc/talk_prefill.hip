// Attention of talk_attn.h for prompt portions, bf16, on the matrix cores, from the paged cache.
//
// A workgroup owns one portion and 16 query rows with all their heads, four heads per wave: mixing needs every head's weights,
// and weights need their denominators.  Two walks over the keys up to the last row, 32 at a time:
//   1  S^T[key, row] = K . Q^T per head, K straight from the caches in operand order; each lane keeps the maximum and sum of
//      the keys it sees, joined at the end.  No exchange between waves.
//   2  S^T again; W = 2^(S - m) / l, complete weights, as a bf16 hi + lo pair (16 significant bits) into LDS, [row][key][head];
//      per row (dealt to the waves) M^T[key, head] = W^T . talk^T, back into the row's place in LDS as a pair, [row][head][key];
//      O^T[dim, row] += V^T . M^T per head, V^T by LDS transpose reads of a tile that all waves filled.
// Weights need no rescaling: the denominators are known.  The rows of two 16-key tiles are picked so that their accumulators are
// eight consecutive keys.
#include "talk_attn.h"

namespace tlf {

constexpr int kTQ = 16, kTK = 32;   // query rows per workgroup, keys per tile

struct TalkPrefillArgs {
  SinkCache c;
  const unsigned short *q;          // [rows, H, Dp]
  const unsigned short *talk;       // [H, H]
  const int32_t *cu_q, *starts;
  unsigned short *out;
  int64_t ldo;
  int32_t H, group;
  int32_t xtiles, total, first_seq, per_xcd, table_cols;
};

// One buffer per row, first W [key][head], then M [head][key]; hi and lo apart.  HT: heads in units of 16.
template <int HT>
struct TalkLds {
  static constexpr int kW = HT * 16 + 8;                             // head stride of a key
  static constexpr int kM = kTK + 8;                                 // key stride of a head
  static constexpr int kRow = (kTK * kW > HT * 16 * kM ? kTK * kW : HT * 16 * kM) + 8;   // rows begin in different banks
};

// WV waves, DC, VC: key and value dimensions in units of 32
template <int WV, int DC, int VC>
__global__ __launch_bounds__(WV * 64) void talk_prefill_kernel(const TalkPrefillArgs p) {
  constexpr int HT = (WV + 3) / 4, VP = VC * 32, LV = VP + 16;
  constexpr int KH = (HT + 1) / 2;                                   // heads in units of 32: steps of the mix
  using L = TalkLds<HT>;
  extern __shared__ __attribute__((aligned(16))) unsigned short lds[];
  unsigned short *Wh = lds, *Wl = lds + kTQ * L::kRow, *Vs = lds + 2 * kTQ * L::kRow;   // Vs [G][32][LV]
  const int id = (blockIdx.x & 7) * p.per_xcd + (blockIdx.x >> 3);   // neighbours in rows share keys: the same XCD
  if (id >= p.total) return;
  const SinkCache &c = p.c;
  const int xt = p.xtiles - 1 - id % p.xtiles, seq = p.first_seq + id / p.xtiles;       // the longest first
  const int q0 = p.cu_q[seq], lq = p.cu_q[seq + 1] - q0, start = p.starts[seq];
  const int row0 = xt * kTQ;
  if (row0 >= lq || start + lq > static_cast<int64_t>(p.table_cols) * c.bs) return;
  const int32_t *bt = c.bt + seq * c.bt_stride;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int last_row = min(row0 + kTQ, lq) - 1, i_last = start + last_row;
  const int my_row = min(row0 + n, last_row), my_pos = start + my_row;
  const int h0 = wave * 4, G = c.G;
  const int tiles = i_last / kTK + 1;

  // heads that no wave has are read by the mix (times zero)
  for (int i = tid; i < 2 * kTQ * L::kRow / 8; i += WV * 64) reinterpret_cast<uint4 *>(lds)[i] = make_uint4(0, 0, 0, 0);
  lds_barrier();
  bf16x8 qf[4][DC];
  int kvh[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int h = min(h0 + e, p.H - 1);
    kvh[e] = h / p.group;
    const unsigned short *qp = p.q + (static_cast<int64_t>(q0 + my_row) * p.H + h) * c.Dp + g * 8;
#pragma unroll
    for (int kc = 0; kc < DC; ++kc) {
      Pack16 t;
      t.u = kc * 32 < c.Dp ? *reinterpret_cast<const uint4 *>(qp + kc * 32) : make_uint4(0, 0, 0, 0);
      qf[e][kc] = t.v;
    }
  }
  const int krow = (n >> 2) * 8 + (n & 3);
  bf16x8 kf[2][DC];
  auto load_k = [&](int j0, int page, int kv) __attribute__((always_inline)) {
    const unsigned short *kp = static_cast<const unsigned short *>(c.k) + (sink_row(c, page, sink_page_of(c, j0), kv, j0) + krow) * c.Dp + g * 8;
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int kc = 0; kc < DC; ++kc) {
        Pack16 t;
        t.u = kc * 32 < c.Dp ? *reinterpret_cast<const uint4 *>(kp + s * 4 * c.Dp + kc * 32) : make_uint4(0, 0, 0, 0);
        kf[s][kc] = t.v;
      }
  };
  // lane (n, g): keys j0 + g * 8 + 0 .. 7 of row n
  auto scores = [&](int e, int j0, float (&w)[8]) __attribute__((always_inline)) {
    floatx4 s0 = floatx4{0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
    for (int kc = 0; kc < DC; ++kc) {
      s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[0][kc], qf[e][kc], s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[1][kc], qf[e][kc], s1, 0, 0, 0);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) w[j] = j < 4 ? s0[j & 3] : s1[j & 3];
    if (j0 + kTK - 1 > start + row0) {                               // the diagonal cuts the tile
#pragma unroll
      for (int j = 0; j < 8; ++j) w[j] = j0 + g * 8 + j <= my_pos ? w[j] : -INFINITY;
    }
  };

  float m[4], l[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) { m[e] = -INFINITY; l[e] = 0.f; }
  {
    int page = bt[0];
    for (int t = 0; t < tiles; ++t) {
      const int j0 = t * kTK;
      const int next = bt[sink_page_of(c, min(j0 + kTK, i_last))];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        if (e == 0 || kvh[e] != kvh[e - 1]) load_k(j0, page, kvh[e]);
        float w[8];
        scores(e, j0, w);
        float x = w[0];
#pragma unroll
        for (int j = 1; j < 8; ++j) x = fmaxf(x, w[j]);
        const float mn = fmaxf(m[e], x), ms = mn == -INFINITY ? 0.f : mn;
        l[e] *= __builtin_amdgcn_exp2f(m[e] - ms);
        m[e] = mn;
#pragma unroll
        for (int j = 0; j < 8; ++j) l[e] += __builtin_amdgcn_exp2f(w[j] - ms);
      }
      page = next;
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float top = max_lanes_16_32_48(m[e]);                    // a row sees itself: finite
      l[e] = sum_lanes_16_32_48(l[e] * __builtin_amdgcn_exp2f(m[e] - top));
      m[e] = top;
      l[e] = h0 + e < p.H ? 1.0f / l[e] : 0.f;
    }
  }

  // talk^T as the mix's B operand: lane (n, g) of tile t holds talk[16 t + n][32 k + 8 g ..]
  bf16x8 tf[HT][KH];
#pragma unroll
  for (int t = 0; t < HT; ++t)
#pragma unroll
    for (int k = 0; k < KH; ++k) {
      Pack16 x;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int h = t * 16 + n, gg = k * 32 + g * 8 + j;
        x.s[j] = h < p.H && gg < p.H ? p.talk[h * p.H + gg] : 0;
      }
      tf[t][k] = x.v;
    }

  floatx4 acc[4][2 * VC];
#pragma unroll
  for (int e = 0; e < 4; ++e)
#pragma unroll
    for (int d = 0; d < 2 * VC; ++d) acc[e][d] = floatx4{0.f, 0.f, 0.f, 0.f};

  const int vpieces = G * kTK * (VP / 8);
  int page = bt[0];
  for (int t = 0; t < tiles; ++t) {
    const int j0 = t * kTK;
    const int next = bt[sink_page_of(c, min(j0 + kTK, i_last))], pg = sink_page_of(c, j0);
    // the last tile's V and M have been read by all (barrier at the end)
    for (int item = tid; item < vpieces; item += WV * 64) {
      const int kv = item / (kTK * (VP / 8)), rest = item % (kTK * (VP / 8)), r = rest / (VP / 8), ch = rest % (VP / 8);
      uint4 v = make_uint4(0, 0, 0, 0);
      if (ch * 8 < c.Vp) v = *reinterpret_cast<const uint4 *>(static_cast<const unsigned short *>(c.v) + (sink_row(c, page, pg, kv, j0) + r) * c.Vp + ch * 8);
      *reinterpret_cast<uint4 *>(Vs + (kv * kTK + r) * LV + ch * 8) = v;
    }
    float w[4][8];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (e == 0 || kvh[e] != kvh[e - 1]) load_k(j0, page, kvh[e]);
      scores(e, j0, w[e]);
#pragma unroll
      for (int j = 0; j < 8; ++j) w[e][j] = __builtin_amdgcn_exp2f(w[e][j] - m[e]) * l[e];
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {                                    // four heads of one key: 8 bytes
      const unsigned int a = pack_bf16x2(w[0][j], w[1][j]), b = pack_bf16x2(w[2][j], w[3][j]);
      const int at = n * L::kRow + (g * 8 + j) * L::kW + h0;
      *reinterpret_cast<uint2 *>(Wh + at) = make_uint2(a, b);
      *reinterpret_cast<uint2 *>(Wl + at) =
          make_uint2(pack_bf16x2(w[0][j] - __uint_as_float(a << 16), w[1][j] - __uint_as_float(a & 0xffff0000u)),
                     pack_bf16x2(w[2][j] - __uint_as_float(b << 16), w[3][j] - __uint_as_float(b & 0xffff0000u)));
    }
    lds_barrier();
    for (int i = wave; i < kTQ; i += WV) {                           // a row's W is read and its M written by the same wave
      unsigned short *wh = Wh + i * L::kRow, *wl = Wl + i * L::kRow;
      floatx4 mx[HT][2];
#pragma unroll
      for (int ht = 0; ht < HT; ++ht) mx[ht][0] = mx[ht][1] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KH; ++k)
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          Pack16 hi, lo;
          hi.u = lo.u = make_uint4(0, 0, 0, 0);
          if (k * 32 + g * 8 < HT * 16) {                            // heads there are room for
            hi.u = *reinterpret_cast<const uint4 *>(wh + (krow + s * 4) * L::kW + k * 32 + g * 8);
            lo.u = *reinterpret_cast<const uint4 *>(wl + (krow + s * 4) * L::kW + k * 32 + g * 8);
          }
#pragma unroll
          for (int ht = 0; ht < HT; ++ht) {
            mx[ht][s] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi.v, tf[ht][k], mx[ht][s], 0, 0, 0);
            mx[ht][s] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo.v, tf[ht][k], mx[ht][s], 0, 0, 0);
          }
        }
      wave_lds_fence();
#pragma unroll
      for (int ht = 0; ht < HT; ++ht) {                              // lane (n, g): head 16 ht + n, keys 8 g ..
        const float x[8] = {mx[ht][0][0], mx[ht][0][1], mx[ht][0][2], mx[ht][0][3], mx[ht][1][0], mx[ht][1][1], mx[ht][1][2], mx[ht][1][3]};
        bf16x8 hi, lo;
        talk_pair(x, hi, lo);
        *reinterpret_cast<bf16x8 *>(wh + (ht * 16 + n) * L::kM + g * 8) = hi;
        *reinterpret_cast<bf16x8 *>(wl + (ht * 16 + n) * L::kM + g * 8) = lo;
      }
    }
    lds_barrier();
    const int vrow = g * 8 + (n >> 2), vcol = (n & 3) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (h0 + e >= p.H) continue;                                   // wave uniform
      const bf16x8 mh = *reinterpret_cast<const bf16x8 *>(Wh + n * L::kRow + (h0 + e) * L::kM + g * 8);
      const bf16x8 ml = *reinterpret_cast<const bf16x8 *>(Wl + n * L::kRow + (h0 + e) * L::kM + g * 8);
      const unsigned short *vp = Vs + (kvh[e] * kTK + vrow) * LV + vcol;
#pragma unroll
      for (int d = 0; d < 2 * VC; ++d) {
        const uint2 v0 = __builtin_bit_cast(uint2, talk_read_tr16(vp + d * 16)), v1 = __builtin_bit_cast(uint2, talk_read_tr16(vp + 4 * LV + d * 16));
        const bf16x8 vb = __builtin_bit_cast(bf16x8, make_uint4(v0.x, v0.y, v1.x, v1.y));
        acc[e][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, mh, acc[e][d], 0, 0, 0);
        acc[e][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, ml, acc[e][d], 0, 0, 0);
      }
    }
    lds_barrier();
    page = next;
  }

  const bool vec = (c.Dv & 3) == 0 && (p.ldo & 3) == 0 && (reinterpret_cast<uintptr_t>(p.out) & 7) == 0;
  if (row0 + n > last_row) return;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    if (h0 + e >= p.H) return;
    unsigned short *o = p.out + static_cast<int64_t>(q0 + row0 + n) * p.ldo + static_cast<int64_t>(h0 + e) * c.Dv;
#pragma unroll
    for (int d = 0; d < 2 * VC; ++d) {
      const int col = d * 16 + g * 4;
      const uint2 v = make_uint2(pack_bf16x2(acc[e][d][0], acc[e][d][1]), pack_bf16x2(acc[e][d][2], acc[e][d][3]));
      if (vec) {
        if (col < c.Dv) *reinterpret_cast<uint2 *>(o + col) = v;
      } else {
        const unsigned int x[2] = {v.x, v.y};
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (col + r < c.Dv) o[col + r] = static_cast<unsigned short>(x[r / 2] >> (16 * (r & 1)));
      }
    }
  }
}

// Waves as instantiated for H heads, 0: too many.
inline int talk_waves(int heads) { return heads <= 4 ? 1 : heads <= 8 ? 2 : heads <= 16 ? 4 : heads <= 32 ? 8 : 0; }
inline int talk_units(int dim) { return dim <= 64 ? 2 : 4; }          // of 32, as instantiated
size_t talk_prefill_lds(int heads, int G, int vdim) {
  const size_t row = talk_waves(heads) <= 4 ? TalkLds<1>::kRow : TalkLds<2>::kRow;
  return 2 * (2 * kTQ * row + static_cast<size_t>(G) * kTK * (talk_units(vdim) * 32 + 16));
}

template <int WV, int DC, int VC>
int launch_talk_prefill(const TalkPrefillArgs &a, size_t lds, hipStream_t s) {
  static const hipError_t allowed = hipFuncSetAttribute(reinterpret_cast<const void *>(&talk_prefill_kernel<WV, DC, VC>),
                                                        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  if (allowed != hipSuccess) return static_cast<int>(allowed);
  TLF_LAUNCH((talk_prefill_kernel<WV, DC, VC>), dim3(a.per_xcd * 8), dim3(WV * 64), lds, s, a);
  return launch_status();
}

}  // namespace tlf

extern "C" int tlf_talk_attn_prefill_supported(int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim) {
  return heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0 && heads <= 32 && dim <= 128 && vdim <= 128 &&
         tlf::talk_prefill_lds(heads, kv_heads, vdim) <= 160 * 1024;
}

extern "C" int tlf_talk_attn_prefill(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables,
                                     int64_t bt_stride, const int32_t *cu_seqlens_q, const int32_t *seq_starts, int32_t first_seq,
                                     int32_t num_seqs, int32_t max_tokens, const void *talk, void *out, int64_t out_stride,
                                     int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size,
                                     int64_t num_pages, void *stream) {
  using namespace tlf;
  if (num_seqs < 0 || max_tokens < 0 || first_seq < 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads) return TLF_E_SHAPE;
  if (out_stride < static_cast<int64_t>(heads) * vdim || bt_stride <= 0) return TLF_E_SHAPE;
  if (num_seqs == 0 || max_tokens == 0) return TLF_OK;
  TalkPrefillArgs a{};
  if (int rc = sink_cache_make(a.c, k_cache, v_cache, block_tables, bt_stride, block_size, kv_heads, dim, vdim, num_pages)) return rc;
  if (!tlf_talk_attn_prefill_supported(heads, kv_heads, dim, vdim)) return TLF_E_UNSUPPORTED;
  if (!q || !block_tables || !cu_seqlens_q || !seq_starts || !talk || !out) return TLF_E_NULL;
  if (!aligned16(q)) return TLF_E_ALIGN;
  a.q = static_cast<const unsigned short *>(q); a.talk = static_cast<const unsigned short *>(talk); a.cu_q = cu_seqlens_q;
  a.starts = seq_starts; a.out = static_cast<unsigned short *>(out); a.ldo = out_stride; a.H = heads; a.group = heads / kv_heads;
  a.xtiles = (max_tokens + kTQ - 1) / kTQ;
  a.first_seq = first_seq; a.table_cols = static_cast<int32_t>(bt_stride);
  const int64_t total = static_cast<int64_t>(a.xtiles) * num_seqs;
  if (total > (1 << 30)) return TLF_E_SHAPE;
  a.total = static_cast<int32_t>(total);
  a.per_xcd = (a.total + 7) / 8;
  const size_t lds = talk_prefill_lds(heads, kv_heads, vdim);
  hipStream_t s = static_cast<hipStream_t>(stream);
  const bool d4 = talk_units(dim) == 4, v4 = talk_units(vdim) == 4;
#define TLF_TP(WV)                                                      \
  case WV:                                                              \
    if (d4 && v4) return launch_talk_prefill<WV, 4, 4>(a, lds, s);      \
    if (d4) return launch_talk_prefill<WV, 4, 2>(a, lds, s);            \
    if (v4) return launch_talk_prefill<WV, 2, 4>(a, lds, s);            \
    return launch_talk_prefill<WV, 2, 2>(a, lds, s);
  switch (talk_waves(heads)) {
    TLF_TP(1) TLF_TP(2) TLF_TP(4) TLF_TP(8)
    default: return TLF_E_UNSUPPORTED;
  }
#undef TLF_TP
}
