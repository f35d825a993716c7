// What lies between the projections and the attention of sink_attn.h:
//
//   sink_prep_kernel   projection row [q | k | v | gate] -> biases, short causal convolution over time per channel, RMS norm
//                      per head of q and k, a factor per position on q, rotation of the first rot_dims dimensions in halves
//                      (i with i + rot_dims / 2), K and V stores, q with the score's constants; the gate where the projection exists as partial sums
//   conv_tail_kernel   the last projected rows of a step's portions into the convolution's state
//
// Convolution state: a ring of `taps` projected rows per sequence (bias not yet added), position p in row p mod taps.  A
// single token writes its row while it reads the taps - 1 before it, which lie in other rows; portions read the ring for their
// first tokens and their last rows go there in a second launch.  Positions below 0 are zeros, so a ring is never cleared.
// HBM bound: a row is read once (from the caches again for the convolution of its neighbours) and written once.
#include "sink_attn.h"

namespace tlf {

struct SinkPrepArgs {
  const void *proj;            // [n, ld]: q heads, k heads, v heads, gate
  Partials part;               // or its partial sums
  int64_t ld;
  const void *bias;            // [channels of q, k, v] or NULL
  const void *conv;            // [taps, channels] or NULL
  void *ring;                  // [state slots, taps, channels]
  const int32_t *state_slots;  // per sequence
  int64_t num_state_slots;
  const int32_t *row_seq, *cu_q;   // NULL: row r is the one row of sequence r
  const void *q_norm, *k_norm;     // [D] or NULL
  const int64_t *positions;
  const float *cos_sin;        // [max_pos, rot_dims]: cos of the pairs, then sin
  const float *q_mult;         // [max_pos] or NULL
  int32_t max_pos, rot_dims;
  const int32_t *slots;        // cache slot per token, negative: no store
  void *q_out, *gate_out;      // [n, H, Dp]; [n, H * Dv] or NULL
  SinkCache c;
  int32_t n, H, taps, channels, heads;
  float eps, q_scale;
};

// Eight values that came from memory as T: held as they were, exact.
template <typename T, bool PACK>
struct Few {
  float f[8];
  __device__ __forceinline__ void put(const float (&v)[8]) {
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = v[e];
  }
  __device__ __forceinline__ float operator[](int e) const { return f[e]; }
};
template <>
struct Few<unsigned short, true> {
  unsigned int w[4];
  __device__ __forceinline__ void put(const float (&v)[8]) {
#pragma unroll
    for (int e = 0; e < 4; ++e) w[e] = (__float_as_uint(v[2 * e]) >> 16) | (__float_as_uint(v[2 * e + 1]) & 0xffff0000u);
  }
  __device__ __forceinline__ float operator[](int e) const { return __uint_as_float(e & 1 ? w[e / 2] & 0xffff0000u : w[e / 2] << 16); }
};

// 16 lanes per (token, head), MAXC chunks of 8 elements per lane.  TAPS: 0 no convolution, -1 any (neighbours read again),
// otherwise a window of that many rows stays in registers over TOK consecutive tokens.  VEC: all sizes are multiples of 8.
template <typename T, int MAXC, int TOK, int TAPS, bool PART, bool VEC>
__global__ __launch_bounds__(256) void sink_prep_kernel(const SinkPrepArgs a) {
  __shared__ __attribute__((aligned(16))) float turn[16][MAXC * 128 + 8];
  constexpr int kBack = TAPS > 0 ? TAPS - 1 : 1;
  const SinkCache &c = a.c;
  const int head = blockIdx.y * 16 + threadIdx.x / 16, j = threadIdx.x % 16;
  if (head >= a.heads) return;                      // whole 16-lane groups leave together
  const int G = c.G;
  const int kind = head < a.H ? 0 : head < a.H + G ? 1 : head < a.H + 2 * G ? 2 : 3;
  const int dims = kind < 2 ? c.D : c.Dv, nch = (kind < 2 ? c.Dp : c.Vp) / 8;
  const int chan = kind < 2 ? head * c.D : (a.H + G) * c.D + (head - a.H - G) * c.Dv;
  const int64_t tok0 = static_cast<int64_t>(blockIdx.x) * TOK;
  const T *proj = static_cast<const T *>(a.proj);

  auto at8 = [&](const T *p, int ch, float (&f)[8]) __attribute__((always_inline)) {   // p: the head's first element
    if constexpr (VEC) {
      Elem<T>::ld8(p + min(ch * 8, dims - 8), f);
      if (ch * 8 >= dims) {
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = 0.f;
      }
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) f[e] = ch * 8 + e < dims ? Elem<T>::ld(p + ch * 8 + e) : 0.f;
    }
  };
  auto row8 = [&](int64_t row, int ch, float (&f)[8]) __attribute__((always_inline)) {
    if constexpr (PART) {
      a.part.ld8(row, chan + min(ch * 8, dims - 8), f);
      if (ch * 8 >= dims) {
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = 0.f;
      }
    } else {
      at8(proj + row * a.ld + chan, ch, f);
    }
  };

  if (kind == 3) {
    for (int64_t tok = tok0; tok < min(tok0 + TOK, static_cast<int64_t>(a.n)); ++tok) {
#pragma unroll
      for (int q = 0; q < MAXC; ++q) {
        const int ch = j + q * 16;
        if (ch * 8 >= dims) continue;
        float f[8];
        row8(tok, ch, f);
        T *o = static_cast<T *>(a.gate_out) + tok * (static_cast<int64_t>(a.H) * c.Dv) + static_cast<int64_t>(head - a.H - 2 * G) * c.Dv + ch * 8;
        if constexpr (VEC) Elem<T>::st8(o, f);
        else
          for (int e = 0; e < 8; ++e)
            if (ch * 8 + e < dims) Elem<T>::st(o + e, f[e]);
      }
    }
    return;
  }

  // the weights stay packed: registers decide how many waves hide the loads
  Few<T, VEC> bias[MAXC], wn[MAXC], wc[TAPS > 0 ? TAPS : 1][MAXC];
  float hist[kBack][MAXC][8];
  const T *norm = static_cast<const T *>(kind == 0 ? a.q_norm : kind == 1 ? a.k_norm : nullptr);
#pragma unroll
  for (int q = 0; q < MAXC; ++q) {
    const int ch = j + q * 16;
    float f[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = 0.f;
    if (a.bias) at8(static_cast<const T *>(a.bias) + chan, ch, f);
    bias[q].put(f);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = 1.f;
    if (norm) at8(norm, ch, f);
    wn[q].put(f);
    if constexpr (TAPS > 0) {
#pragma unroll
      for (int t = 0; t < TAPS; ++t) {
        at8(static_cast<const T *>(a.conv) + static_cast<int64_t>(t) * a.channels + chan, ch, f);
        wc[t][q].put(f);
      }
    }
  }
  // the loads of all tokens are in flight before the first is touched
  typename Elem<T>::Raw8 raw[TOK][MAXC];
  if constexpr (VEC && !PART) {
#pragma unroll
    for (int k = 0; k < TOK; ++k)
#pragma unroll
      for (int q = 0; q < MAXC; ++q)
        Elem<T>::raw8(proj + min(tok0 + k, static_cast<int64_t>(a.n) - 1) * a.ld + chan + min((j + q * 16) * 8, dims - 8), raw[k][q]);
  }

  // and of the rows before them, of the same sequence or not
  typename Elem<T>::Raw8 back_rows[kBack][MAXC];
  if constexpr (VEC && !PART && TAPS > 0 && TOK > 1) {
#pragma unroll
    for (int b = 0; b < kBack; ++b)
#pragma unroll
      for (int q = 0; q < MAXC; ++q)
        Elem<T>::raw8(proj + max(tok0 - 1 - b, static_cast<int64_t>(0)) * a.ld + chan + min((j + q * 16) * 8, dims - 8), back_rows[b][q]);
  }
  int64_t poss[TOK], slots[TOK];
  int32_t firsts[TOK], states[TOK];
  bool singles[TOK];
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const int64_t tok = min(tok0 + k, static_cast<int64_t>(a.n) - 1);
    poss[k] = a.positions[tok];
    slots[k] = a.slots[tok];
    if constexpr (TAPS != 0) {
      const int seq = a.row_seq ? a.row_seq[tok] : static_cast<int>(tok);
      firsts[k] = a.row_seq ? a.cu_q[seq] : static_cast<int>(tok);
      singles[k] = !a.row_seq || a.cu_q[seq + 1] - firsts[k] == 1;
      states[k] = a.state_slots[seq];
    }
  }
  const int half = a.rot_dims / 2;
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const int64_t tok = tok0 + k;
    if (tok >= a.n) return;
    const int64_t pos = poss[k], slot = slots[k];
    float x[MAXC][8];
#pragma unroll
    for (int q = 0; q < MAXC; ++q) {
      if constexpr (VEC && !PART) {
        Elem<T>::cvt8(raw[k][q], x[q]);
        if ((j + q * 16) * 8 >= dims) {
#pragma unroll
          for (int e = 0; e < 8; ++e) x[q][e] = 0.f;
        }
      } else {
        row8(tok, j + q * 16, x[q]);
      }
    }
    if constexpr (TAPS != 0) {
      const int taps = TAPS > 0 ? TAPS : a.taps;
      const int64_t first = firsts[k], st = states[k];
      const bool single = singles[k];
      const bool held = st >= 0 && st < a.num_state_slots && pos >= 0;
      T *ring = static_cast<T *>(a.ring) + (held ? st : 0) * taps * a.channels + chan;
      // projected value `back` tokens earlier, with its bias
      auto earlier = [&](int back, int q, float (&f)[8]) __attribute__((always_inline)) {
        const int ch = j + q * 16;
        if (pos < back || !held) {
#pragma unroll
          for (int e = 0; e < 8; ++e) f[e] = 0.f;
          return;
        }
        if (tok - back >= first) {
          if (VEC && !PART && TOK > 1 && TAPS > 0 && k == 0) {
            Elem<T>::cvt8(back_rows[TAPS > 0 ? back - 1 : 0][q], f);
            if (ch * 8 >= dims) {
#pragma unroll
              for (int e = 0; e < 8; ++e) f[e] = 0.f;
            }
          } else row8(tok - back, ch, f);
        } else at8(ring + (pos - back) % taps * a.channels, ch, f);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] += bias[q][e];
      };
      if (single && held) {
        T *w = ring + pos % taps * a.channels;
#pragma unroll
        for (int q = 0; q < MAXC; ++q) {
          const int ch = j + q * 16;
          if (ch * 8 >= dims) continue;
          if constexpr (VEC) Elem<T>::st8(w + ch * 8, x[q]);
          else
            for (int e = 0; e < 8; ++e)
              if (ch * 8 + e < dims) Elem<T>::st(w + ch * 8 + e, x[q][e]);
        }
      }
#pragma unroll
      for (int q = 0; q < MAXC; ++q)
#pragma unroll
        for (int e = 0; e < 8; ++e) x[q][e] += bias[q][e];
      if constexpr (TAPS > 0) {
        if (k == 0 || tok == first) {
#pragma unroll
          for (int b = 0; b < kBack; ++b)
#pragma unroll
            for (int q = 0; q < MAXC; ++q) earlier(b + 1, q, hist[b][q]);
        }
#pragma unroll
        for (int q = 0; q < MAXC; ++q)
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            float y = 0.f;
#pragma unroll
            for (int b = kBack - 1; b >= 0; --b) y = fmaf(wc[TAPS - 2 - b][q][e], hist[b][q][e], y);
            const float now = x[q][e];
            x[q][e] = fmaf(wc[TAPS - 1][q][e], now, y);
#pragma unroll
            for (int b = kBack - 1; b > 0; --b) hist[b][q][e] = hist[b - 1][q][e];
            hist[0][q][e] = now;
          }
      } else {
        const T *w = static_cast<const T *>(a.conv) + chan;
#pragma unroll
        for (int q = 0; q < MAXC; ++q) {
          float y[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, f[8], wt[8];
          for (int b = taps - 1; b > 0; --b) {
            earlier(b, q, f);
            at8(w + static_cast<int64_t>(taps - 1 - b) * a.channels, j + q * 16, wt);
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] = fmaf(wt[e], f[e], y[e]);
          }
          at8(w + static_cast<int64_t>(taps - 1) * a.channels, j + q * 16, wt);
#pragma unroll
          for (int e = 0; e < 8; ++e) x[q][e] = fmaf(wt[e], x[q][e], y[e]);
        }
      }
    } else {
#pragma unroll
      for (int q = 0; q < MAXC; ++q)
#pragma unroll
        for (int e = 0; e < 8; ++e) x[q][e] += bias[q][e];
    }

    const bool store = slot >= 0 && slot < c.pages * c.bs;
    const int64_t page = store ? slot / c.bs : 0;
    const int64_t crow = (page * G + (head - a.H) % G) * c.bs + (slot - page * c.bs);
    if (kind == 2) {
#pragma unroll
      for (int q = 0; q < MAXC; ++q)
        if (store && j + q * 16 < nch) Elem<T>::st8(static_cast<T *>(const_cast<void *>(c.v)) + crow * c.Vp + (j + q * 16) * 8, x[q]);
      continue;
    }
    float ss = 0.f;
#pragma unroll
    for (int q = 0; q < MAXC; ++q)
#pragma unroll
      for (int e = 0; e < 8; ++e) ss = fmaf(x[q][e], x[q][e], ss);
    ss = group_sum<16>(ss);
    const bool pos_ok = pos >= 0 && pos < a.max_pos;
    float inv = 1.0f / sqrtf(ss / static_cast<float>(c.D) + a.eps);
#pragma unroll
    for (int q = 0; q < MAXC; ++q)
#pragma unroll
      for (int e = 0; e < 8; ++e) x[q][e] = x[q][e] * inv * wn[q][e];
    if (kind == 0) {
      const float m = a.q_mult ? a.q_mult[pos_ok ? pos : 0] * a.q_scale : a.q_scale;
#pragma unroll
      for (int q = 0; q < MAXC; ++q)
#pragma unroll
        for (int e = 0; e < 8; ++e) x[q][e] *= m;
    }
    if (a.rot_dims > 0 && pos_ok) {                  // the same for the lanes of a team
      float *xs = turn[threadIdx.x / 16];
      const float *cs = a.cos_sin + pos * a.rot_dims;
      wave_lds_fence();
#pragma unroll
      for (int q = 0; q < MAXC; ++q) {
        float4 *d = reinterpret_cast<float4 *>(xs + (j + q * 16) * 8);
        d[0] = make_float4(x[q][0], x[q][1], x[q][2], x[q][3]);
        d[1] = make_float4(x[q][4], x[q][5], x[q][6], x[q][7]);
      }
      wave_lds_fence();
#pragma unroll
      for (int q = 0; q < MAXC; ++q) {
        const int at = (j + q * 16) * 8;
        if (at >= a.rot_dims) continue;
        if (VEC && half % 8 == 0) {
          const bool low = at < half;
          const float *ps = xs + (low ? at + half : at - half), *cp = cs + (low ? at : at - half);
          const float sign = low ? -1.f : 1.f;
          float p[8], cv[8], sv[8];
          Elem<float>::ld8(ps, p);
          Elem<float>::ld8(cp, cv);
          Elem<float>::ld8(cp + half, sv);
#pragma unroll
          for (int e = 0; e < 8; ++e) x[q][e] = __fmul_rn(x[q][e], cv[e]) + sign * __fmul_rn(p[e], sv[e]);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const int i = at + e;
            if (i < half) x[q][e] = __fmul_rn(x[q][e], cs[i]) - __fmul_rn(xs[i + half], cs[half + i]);
            else if (i < a.rot_dims) x[q][e] = __fmul_rn(x[q][e], cs[i - half]) + __fmul_rn(xs[i - half], cs[i]);
          }
        }
      }
    }
#pragma unroll
    for (int q = 0; q < MAXC; ++q) {
      const int ch = j + q * 16;
      if (ch >= nch) continue;
      if (kind == 0) Elem<T>::st8(static_cast<T *>(a.q_out) + (tok * a.H + head) * c.Dp + ch * 8, x[q]);
      else if (store) Elem<T>::st8(static_cast<T *>(const_cast<void *>(c.k)) + crow * c.Dp + ch * 8, x[q]);
    }
  }
}

template <typename T>
int launch_sink_prep(const SinkPrepArgs &a, bool vec, bool part, hipStream_t s) {
  const int most = a.c.Dp > a.c.Vp ? a.c.Dp : a.c.Vp;
  const unsigned hy = (a.heads + 15) / 16;
#define TLF_PREP(MAXC, TOK, TAPS, PART, VEC)                                                                       \
  TLF_LAUNCH((sink_prep_kernel<T, MAXC, TOK, TAPS, PART, VEC>), dim3((a.n + (TOK) - 1) / (TOK), hy), dim3(256), 0, s, a)
#define TLF_PREP_ANY(TAPS)                                \
  do {                                                    \
    if (most <= 128) TLF_PREP(1, 1, TAPS, false, false);  \
    else TLF_PREP(4, 1, TAPS, false, false);              \
  } while (0)
  if constexpr (sizeof(T) == 2) {
    if (vec && most <= 256) {
#define TLF_PREP_C(MAXC, TAPS)                                     \
  do {                                                             \
    if (part) TLF_PREP(MAXC, 1, TAPS, true, true);                 \
    else if (a.n > 1024 && (TAPS) >= 0) TLF_PREP(MAXC, (TAPS) >= 0 ? 4 : 1, TAPS, false, true); \
    else TLF_PREP(MAXC, 1, TAPS, false, true);                     \
  } while (0)
#define TLF_PREP_T(TAPS)                     \
  do {                                       \
    if (most <= 128) TLF_PREP_C(1, TAPS);    \
    else TLF_PREP_C(2, TAPS);                \
  } while (0)
      switch (a.conv ? a.taps : 0) {
        case 0: TLF_PREP_T(0); break;
        case 2: TLF_PREP_T(2); break;
        case 3: TLF_PREP_T(3); break;
        case 4: TLF_PREP_T(4); break;
        default: TLF_PREP_T(-1); break;
      }
#undef TLF_PREP_T
#undef TLF_PREP_C
      return launch_status();
    }
  }
  if (part) return TLF_E_UNSUPPORTED;
  if (a.conv) TLF_PREP_ANY(-1);
  else TLF_PREP_ANY(0);
#undef TLF_PREP_ANY
#undef TLF_PREP
  return launch_status();
}

template <typename T>
__global__ __launch_bounds__(256) void conv_tail_kernel(const T *proj, int64_t ld, T *ring, const int32_t *state_slots,
                                                        int64_t num_state_slots, const int32_t *cu_q, const int32_t *starts,
                                                        int32_t first_seq, int32_t taps, int32_t channels) {
  const int seq = first_seq + blockIdx.y;
  const int64_t end = cu_q[seq + 1], n = end - cu_q[seq], st = state_slots[seq];
  if (st < 0 || st >= num_state_slots) return;
  const int col = blockIdx.x * 256 + threadIdx.x;
  if (col >= channels) return;
  const int64_t last = starts[seq] + n - 1;
  const int keep = static_cast<int>(min(n, static_cast<int64_t>(taps - 1)));
  for (int d = 0; d < keep; ++d) ring[(st * taps + (last - d) % taps) * channels + col] = proj[(end - 1 - d) * ld + col];
}

}  // namespace tlf

extern "C" int tlf_sink_prep(const void *proj, int64_t proj_stride, const float *partials, int32_t splits, const float *scale,
                             const void *bias, const void *conv, int32_t taps, void *ring, const int32_t *state_slots,
                             int64_t num_state_slots, const int32_t *row_seq, const int32_t *cu_seqlens_q, const void *q_norm,
                             const void *k_norm, const int64_t *positions, const float *cos_sin, const float *q_mult,
                             int32_t max_pos, int32_t rot_dims, const int32_t *slot_mapping, void *q_out, void *k_cache,
                             void *v_cache, void *gate_out, int32_t n, int32_t heads, int32_t kv_heads, int32_t dim,
                             int32_t vdim, int32_t block_size, int64_t num_pages, float eps, float score_scale, float cap, int32_t dtype, void *stream) {
  using namespace tlf;
  SinkPrepArgs a{};
  if (n < 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || rot_dims < 0 || rot_dims % 2 || rot_dims > dim) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (cap < 0.f || (conv && (taps < 1 || taps > 64))) return TLF_E_SHAPE;
  if (n == 0) return TLF_OK;
  if (int rc = partials_check(partials, scale, splits, dtype)) return rc;
  if (int rc = sink_cache_make(a.c, k_cache, v_cache, nullptr, 0, block_size, kv_heads, dim, vdim, num_pages)) return rc;
  const int64_t channels = static_cast<int64_t>(heads + kv_heads) * dim + static_cast<int64_t>(kv_heads) * vdim;
  if (proj_stride < channels + static_cast<int64_t>(heads) * vdim || proj_stride > (1 << 28)) return TLF_E_SHAPE;
  if ((!proj && splits <= 1) || !positions || !slot_mapping || !q_out || (rot_dims && !cos_sin)) return TLF_E_NULL;
  if (conv && (!ring || !state_slots || (row_seq && !cu_seqlens_q))) return TLF_E_NULL;
  if (splits > 1 && (!gate_out || row_seq)) return TLF_E_UNSUPPORTED;
  if (!aligned16(q_out)) return TLF_E_ALIGN;
  a.proj = proj; a.ld = proj_stride;
  a.part = Partials{partials, scale, n * proj_stride, static_cast<int32_t>(proj_stride), splits};
  a.bias = bias; a.conv = conv; a.ring = ring; a.state_slots = state_slots; a.num_state_slots = num_state_slots;
  a.row_seq = row_seq; a.cu_q = cu_seqlens_q; a.q_norm = q_norm; a.k_norm = k_norm; a.positions = positions;
  a.cos_sin = cos_sin; a.q_mult = q_mult; a.max_pos = max_pos; a.rot_dims = rot_dims; a.slots = slot_mapping;
  a.q_out = q_out; a.gate_out = gate_out; a.n = n; a.H = heads; a.taps = conv ? taps : 0;
  a.channels = static_cast<int32_t>(channels); a.eps = eps; a.q_scale = sink_query_scale(score_scale, cap);
  a.heads = heads + 2 * kv_heads + (gate_out ? heads : 0);
  if ((a.heads + 15) / 16 > 65535) return TLF_E_SHAPE;
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && proj_stride % 8 == 0 && (splits > 1 || aligned16(proj)) && aligned16(bias) &&
                   aligned16(conv) && aligned16(ring) && aligned16(q_norm) && aligned16(k_norm) && aligned16(gate_out) &&
                   (rot_dims % 16 || aligned16(cos_sin));
  hipStream_t s = static_cast<hipStream_t>(stream);
  return dtype == TLF_DT_BF16 ? launch_sink_prep<unsigned short>(a, vec, splits > 1, s) : launch_sink_prep<float>(a, vec, false, s);
}

extern "C" int tlf_conv_tail(const void *proj, int64_t proj_stride, void *ring, const int32_t *state_slots, int64_t num_state_slots,
                             const int32_t *cu_seqlens_q, const int32_t *seq_starts, int32_t first_seq, int32_t num_seqs,
                             int32_t taps, int32_t channels, int32_t dtype, void *stream) {
  using namespace tlf;
  if (num_seqs < 0 || num_seqs > 65535 || first_seq < 0 || taps < 1 || taps > 64 || channels <= 0 || proj_stride < channels) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (num_seqs == 0 || taps == 1) return TLF_OK;
  if (!proj || !ring || !state_slots || !cu_seqlens_q || !seq_starts) return TLF_E_NULL;
  const dim3 grid((channels + 255) / 256, num_seqs);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == TLF_DT_BF16)
    TLF_LAUNCH((conv_tail_kernel<unsigned short>), grid, dim3(256), 0, s, static_cast<const unsigned short *>(proj), proj_stride,
               static_cast<unsigned short *>(ring), state_slots, num_state_slots, cu_seqlens_q, seq_starts, first_seq, taps, channels);
  else
    TLF_LAUNCH((conv_tail_kernel<float>), grid, dim3(256), 0, s, static_cast<const float *>(proj), proj_stride,
               static_cast<float *>(ring), state_slots, num_state_slots, cu_seqlens_q, seq_starts, first_seq, taps, channels);
  return launch_status();
}
