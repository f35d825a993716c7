// Norms behind the sum (post-norm), with what precedes and follows them in one pass:
//
//   embed:  v = embed_scale * table[id]
//   post:   v = rms_norm(alpha * x + layer_scale * y) * w
//   then    x' = v (fp32) and  h = v | v + (v_before - v) * mix (token shift) | rms_norm(v) * w_next
//
// v_before is the row of the token before, zeros for a sequence's first one.  For a portion's rows it is computed again from
// the row's own inputs: a team of threads takes `run` rows in a row and keeps the last one, so only the row in front of them
// is read twice (x' must not overwrite x then).  A portion's first row, and a single token, take it from the sequence's state:
// a ring of two fp32 rows, position p in row p mod 2.  Single tokens store theirs here; conv_tail_kernel stores those of
// portions afterwards.  HBM bound: y and x are read once, x' and h written once; arithmetic is fp32.
//
//   rows_rmsnorm_kernel   rows of `cols` values in `groups` equal parts, each divided by its own root mean square, times w
#include "elem.h"

namespace tlf {

struct PostNormArgs {
  const void *y;             // [rows, y_stride]
  Partials part;             // or its partial sums
  int64_t y_stride;
  const void *layer_scale, *w;   // [width]
  const int64_t *ids;        // embed
  const void *table;
  int32_t vocab;
  float alpha;               // of x; of the table's rows for embed
  const float *x;
  float *x_out;
  const void *mix;           // [width]: token shift
  float *ring;               // [slots, 2, width]
  int64_t num_slots;
  const int32_t *state_slots, *row_seq, *cu_q;   // row_seq NULL: row r is the one row of sequence r
  const int64_t *positions;
  const void *w_next;        // [width]: norm
  void *h;                   // [rows, width] or NULL
  int32_t rows, width, run;
  float eps;
};

template <int TPR>
__device__ __forceinline__ float post_sum(float v, float *part) {
  v = wave_sum(v);
  if (TPR <= 64) return v;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
  __syncthreads();
  return (part[0] + part[1]) + (part[2] + part[3]);
}
template <typename T, int VEC>
__device__ __forceinline__ void post_ld(const T *p, float (&f)[VEC]) {
  if constexpr (VEC == 8) Elem<T>::ld8(p, f);
  else f[0] = Elem<T>::ld(p);
}
template <typename T, int VEC>
__device__ __forceinline__ void post_st(T *p, const float (&f)[VEC]) {
  if constexpr (VEC == 8) Elem<T>::st8(p, f);
  else Elem<T>::st(p, f[0]);
}

// TPR threads (64: a wave, 256: the workgroup) per team.  MODE 0: embed, 1: y, 2: y as partial sums
template <typename T, int VEC, int TPR, int MAXC, int MODE, bool SHIFT>
__global__ __launch_bounds__(256) void postnorm_kernel(const PostNormArgs a) {
  __shared__ float part[4];
  const int sub = threadIdx.x % TPR, nch = a.width / VEC;
  const int64_t first = (static_cast<int64_t>(blockIdx.x) * (256 / TPR) + threadIdx.x / TPR) * a.run;
  if (first >= a.rows) return;                       // whole teams leave together
  const float inv_cols = 1.0f / static_cast<float>(a.width);
  const T *ls = static_cast<const T *>(a.layer_scale), *wp = static_cast<const T *>(a.w);

  auto value = [&](int64_t row, float (&v)[MAXC][VEC]) __attribute__((always_inline)) {
    if constexpr (MODE == 0) {
      const int64_t id = a.ids[row];
      const bool ok = id >= 0 && id < a.vocab;
      const T *src = static_cast<const T *>(a.table) + (ok ? id : 0) * a.width;
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        post_ld<T, VEC>(src + min(sub + c * TPR, nch - 1) * VEC, v[c]);
#pragma unroll
        for (int i = 0; i < VEC; ++i) v[c][i] = ok ? v[c][i] * a.alpha : 0.f;
      }
    } else {
      float ss = 0.f, xo[MAXC][VEC];
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        const int at = min(sub + c * TPR, nch - 1) * VEC;
        if constexpr (MODE == 1) post_ld<T, VEC>(static_cast<const T *>(a.y) + row * a.y_stride + at, v[c]);
        else if constexpr (VEC == 8) a.part.ld8(row, at, v[c]);
        else v[c][0] = a.part.ld(row, at);
        post_ld<float, VEC>(a.x + row * a.width + at, xo[c]);
      }
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        const int ch = sub + c * TPR;
        float s[VEC];
        post_ld<T, VEC>(ls + min(ch, nch - 1) * VEC, s);
#pragma unroll
        for (int i = 0; i < VEC; ++i) {
          v[c][i] = fmaf(v[c][i], s[i], a.alpha * xo[c][i]);
          ss = fmaf(v[c][i], ch < nch ? v[c][i] : 0.f, ss);
        }
      }
      ss = post_sum<TPR>(ss, part);
      const float inv = 1.0f / sqrtf(ss * inv_cols + a.eps);
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        float w[VEC];
        post_ld<T, VEC>(wp + min(sub + c * TPR, nch - 1) * VEC, w);
#pragma unroll
        for (int i = 0; i < VEC; ++i) v[c][i] = v[c][i] * inv * w[i];
      }
    }
  };

  float before[SHIFT ? MAXC : 1][VEC];
  int64_t known = -1;                                // row whose value `before` holds
  for (int k = 0; k < a.run; ++k) {
    const int64_t row = first + k;
    if (row >= a.rows) return;
    float v[MAXC][VEC];
    bool single = false, held = false;
    int64_t pos = 0;
    float *ring = nullptr;
    if constexpr (SHIFT) {
      const int seq = a.row_seq ? a.row_seq[row] : static_cast<int>(row);
      const int64_t begin = a.row_seq ? a.cu_q[seq] : row;
      single = !a.row_seq || a.cu_q[seq + 1] - begin == 1;
      const int64_t slot = a.state_slots[seq];
      pos = a.positions[row];
      held = slot >= 0 && slot < a.num_slots && pos >= 0;
      ring = a.ring + (held ? slot : 0) * 2 * a.width;
      if (row > begin) {
        if (known != row - 1) value(row - 1, before);
      } else {
#pragma unroll
        for (int c = 0; c < MAXC; ++c) {
          post_ld<float, VEC>(ring + ((pos + 1) & 1) * a.width + min(sub + c * TPR, nch - 1) * VEC, before[c]);
          if (!held || pos == 0) {
#pragma unroll
            for (int i = 0; i < VEC; ++i) before[c][i] = 0.f;
          }
        }
      }
    }
    value(row, v);
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int ch = sub + c * TPR;
      if (ch < nch) {
        post_st<float, VEC>(a.x_out + row * a.width + ch * VEC, v[c]);
        if (SHIFT && single && held) post_st<float, VEC>(ring + (pos & 1) * a.width + ch * VEC, v[c]);
      }
    }
    T *hr = static_cast<T *>(a.h) + row * a.width;
    if constexpr (SHIFT) {
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        const int ch = sub + c * TPR;
        float m[VEC];
        post_ld<T, VEC>(static_cast<const T *>(a.mix) + min(ch, nch - 1) * VEC, m);
#pragma unroll
        for (int i = 0; i < VEC; ++i) {
          m[i] = fmaf(before[c][i] - v[c][i], m[i], v[c][i]);
          before[c][i] = v[c][i];
        }
        if (ch < nch) post_st<T, VEC>(hr + ch * VEC, m);
      }
      known = row;
    } else {
      if (a.w_next) {
        float ss = 0.f;
#pragma unroll
        for (int c = 0; c < MAXC; ++c)
          if (sub + c * TPR < nch)
#pragma unroll
            for (int i = 0; i < VEC; ++i) ss = fmaf(v[c][i], v[c][i], ss);
        ss = post_sum<TPR>(ss, part);
        const float inv = 1.0f / sqrtf(ss * inv_cols + a.eps);
#pragma unroll
        for (int c = 0; c < MAXC; ++c) {
          float w[VEC];
          post_ld<T, VEC>(static_cast<const T *>(a.w_next) + min(sub + c * TPR, nch - 1) * VEC, w);
#pragma unroll
          for (int i = 0; i < VEC; ++i) v[c][i] = v[c][i] * inv * w[i];
        }
      }
      if (a.h) {
#pragma unroll
        for (int c = 0; c < MAXC; ++c)
          if (sub + c * TPR < nch) post_st<T, VEC>(hr + (sub + c * TPR) * VEC, v[c]);
      }
    }
  }
}

template <typename T, int MODE, bool SHIFT>
int launch_postnorm(PostNormArgs &a, bool vec8, hipStream_t stream) {
  // a portion's rows: long enough runs to read little twice, enough teams to fill the chip
  a.run = SHIFT && a.row_seq ? (a.rows >= 4096 ? 8 : a.rows >= 1024 ? 4 : a.rows >= 256 ? 2 : 1) : 1;
#define TLF_PN(VEC, TPR, MAXC)                                                                                    \
  TLF_LAUNCH((postnorm_kernel<T, VEC, TPR, MAXC, MODE, SHIFT>),                                                   \
             dim3(static_cast<unsigned>((a.rows + (256 / TPR) * a.run - 1) / ((256 / TPR) * a.run))), dim3(256), 0, stream, a)
  if (vec8) {
    if (a.width <= 512) TLF_PN(8, 64, 1);
    else if (a.width <= 1024) TLF_PN(8, 64, 2);
    else if (a.width <= 2048) TLF_PN(8, 256, 1);
    else if (a.width <= 4096) TLF_PN(8, 256, 2);
    else if (a.width <= 8192) TLF_PN(8, 256, 4);
    else TLF_PN(8, 256, 8);
  } else {
    if (a.width <= 256) TLF_PN(1, 64, 4);
    else if (a.width <= 2048) TLF_PN(1, 256, 8);
    else TLF_PN(1, 256, 64);
  }
#undef TLF_PN
  return launch_status();
}

// kMode 0: embed, 1: post
template <int kMode>
int postnorm_entry(PostNormArgs &a, int32_t dtype, hipStream_t stream) {
  if (a.rows < 0 || a.width <= 0 || a.width > 16384) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (a.mix && a.w_next) return TLF_E_UNSUPPORTED;
  if (a.rows == 0) return TLF_OK;
  if (!a.x_out || (!a.h && (a.mix || a.w_next))) return TLF_E_NULL;
  if (a.mix && (!a.ring || !a.state_slots || !a.positions || (a.row_seq && !a.cu_q))) return TLF_E_NULL;
  if (kMode == 1 && a.mix && a.row_seq && a.x_out == a.x) return TLF_E_UNSUPPORTED;   // rows are read again
  if (a.row_seq && a.part.splits > 1 && a.part.n < a.width) return TLF_E_SHAPE;
  bool vec8 = a.width % 8 == 0 && aligned16(a.x_out) && aligned16(a.h) && aligned16(a.mix) && aligned16(a.ring) && aligned16(a.w_next);
  if (kMode == 0) vec8 = vec8 && aligned16(a.table);
  else vec8 = vec8 && aligned16(a.y) && aligned16(a.x) && aligned16(a.layer_scale) && aligned16(a.w) && a.y_stride % 8 == 0;
#define TLF_PN_T(T, MODE) (a.mix ? launch_postnorm<T, MODE, true>(a, vec8, stream) : launch_postnorm<T, MODE, false>(a, vec8, stream))
  if constexpr (kMode == 1)
    if (a.part.splits > 1) return TLF_PN_T(unsigned short, 2);
  return dtype == TLF_DT_BF16 ? TLF_PN_T(unsigned short, kMode) : TLF_PN_T(float, kMode);
#undef TLF_PN_T
}

// ---------------------------------------------------------------------------------------------------------------
struct RowsNormArgs {
  const void *x;         // [rows, ld]
  const void *w;         // [cols]
  void *out;             // [rows, ldo], zeros from cols on
  int64_t ld, ldo;
  int64_t units;         // rows * groups
  int32_t groups, part;  // values of a group
  float eps;
};

template <typename T, int VEC, int TPR, int MAXC>
__global__ __launch_bounds__(256) void rows_rmsnorm_kernel(const RowsNormArgs a) {
  __shared__ float part[4];
  const int sub = threadIdx.x % TPR, nch = a.part / VEC;
  const int64_t unit = static_cast<int64_t>(blockIdx.x) * (256 / TPR) + threadIdx.x / TPR;
  if (unit >= a.units) return;                       // whole teams leave together
  const int64_t row = unit / a.groups;
  const int grp = static_cast<int>(unit - row * a.groups), col0 = grp * a.part;
  const T *src = static_cast<const T *>(a.x) + row * a.ld + col0;
  T *dst = static_cast<T *>(a.out) + row * a.ldo + col0;
  float v[MAXC][VEC], ss = 0.f;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) post_ld<T, VEC>(src + min(sub + c * TPR, nch - 1) * VEC, v[c]);
#pragma unroll
  for (int c = 0; c < MAXC; ++c)
    if (sub + c * TPR < nch)
#pragma unroll
      for (int i = 0; i < VEC; ++i) ss = fmaf(v[c][i], v[c][i], ss);
  ss = post_sum<TPR>(ss, part);
  const float inv = 1.0f / sqrtf(ss / static_cast<float>(a.part) + a.eps);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = sub + c * TPR;
    if (ch < nch) {
      float w[VEC];
      post_ld<T, VEC>(static_cast<const T *>(a.w) + col0 + ch * VEC, w);
#pragma unroll
      for (int i = 0; i < VEC; ++i) w[i] = v[c][i] * inv * w[i];
      post_st<T, VEC>(dst + ch * VEC, w);
    }
  }
  if (grp == a.groups - 1)
    for (int64_t d = a.part + sub; col0 + d < a.ldo; d += TPR) Elem<T>::st(dst + d, 0.f);
}

template <typename T>
int launch_rows_norm(const RowsNormArgs &a, bool vec8, hipStream_t stream) {
#define TLF_RN(VEC, TPR, MAXC) \
  TLF_LAUNCH((rows_rmsnorm_kernel<T, VEC, TPR, MAXC>), dim3(static_cast<unsigned>((a.units + (256 / TPR) - 1) / (256 / TPR))), dim3(256), 0, stream, a)
  if (vec8) {
    if (a.part <= 512) TLF_RN(8, 64, 1);
    else if (a.part <= 1024) TLF_RN(8, 64, 2);
    else if (a.part <= 2048) TLF_RN(8, 256, 1);
    else if (a.part <= 4096) TLF_RN(8, 256, 2);
    else if (a.part <= 8192) TLF_RN(8, 256, 4);
    else TLF_RN(8, 256, 8);
  } else {
    if (a.part <= 256) TLF_RN(1, 64, 4);
    else if (a.part <= 2048) TLF_RN(1, 256, 8);
    else TLF_RN(1, 256, 64);
  }
#undef TLF_RN
  return launch_status();
}

}  // namespace tlf

extern "C" int tlf_post_rmsnorm(const void *y, int64_t y_stride, const float *partials, int32_t splits, const float *scale,
                                const void *layer_scale, float alpha, const float *x, const void *w, float eps, float *x_out,
                                const void *mix, float *ring, int64_t num_slots, const int32_t *state_slots,
                                const int32_t *row_seq, const int32_t *cu_seqlens_q, const int64_t *positions,
                                const void *w_next, void *h, int32_t rows, int32_t width, int32_t dtype, void *stream) {
  tlf::PostNormArgs a{};
  if (int rc = tlf::partials_check(partials, scale, splits, dtype)) return rc;
  if (y_stride < width) return TLF_E_SHAPE;
  if (rows > 0 && ((!y && splits <= 1) || !layer_scale || !x || !w)) return TLF_E_NULL;
  a.part = tlf::Partials{partials, scale, rows * y_stride, static_cast<int32_t>(y_stride), splits};
  a.y = y; a.y_stride = y_stride; a.layer_scale = layer_scale; a.alpha = alpha; a.x = x; a.w = w; a.eps = eps; a.x_out = x_out;
  a.mix = mix; a.ring = ring; a.num_slots = num_slots; a.state_slots = state_slots; a.row_seq = row_seq; a.cu_q = cu_seqlens_q;
  a.positions = positions; a.w_next = w_next; a.h = h; a.rows = rows; a.width = width;
  return tlf::postnorm_entry<1>(a, dtype, static_cast<hipStream_t>(stream));
}

extern "C" int tlf_embed_shift(const int64_t *ids, const void *table, int32_t vocab, float embed_scale, float *x_out,
                               const void *mix, float *ring, int64_t num_slots, const int32_t *state_slots,
                               const int32_t *row_seq, const int32_t *cu_seqlens_q, const int64_t *positions, void *h,
                               int32_t rows, int32_t width, int32_t dtype, void *stream) {
  tlf::PostNormArgs a{};
  if (vocab <= 0) return TLF_E_SHAPE;
  if (rows > 0 && (!ids || !table || !mix)) return TLF_E_NULL;
  a.ids = ids; a.table = table; a.vocab = vocab; a.alpha = embed_scale; a.x_out = x_out; a.mix = mix; a.ring = ring;
  a.num_slots = num_slots; a.state_slots = state_slots; a.row_seq = row_seq; a.cu_q = cu_seqlens_q; a.positions = positions;
  a.h = h; a.rows = rows; a.width = width;
  return tlf::postnorm_entry<0>(a, dtype, static_cast<hipStream_t>(stream));
}

extern "C" int tlf_rows_rmsnorm(const void *x, int64_t x_stride, const void *w, void *out, int64_t out_stride, int32_t rows,
                                int32_t cols, int32_t groups, float eps, int32_t dtype, void *stream) {
  using namespace tlf;
  if (rows < 0 || cols <= 0 || groups <= 0 || cols % groups || cols / groups > 16384 || x_stride < cols || out_stride < cols) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (rows == 0) return TLF_OK;
  if (!x || !w || !out) return TLF_E_NULL;
  const RowsNormArgs a{x, w, out, x_stride, out_stride, static_cast<int64_t>(rows) * groups, groups, cols / groups, eps};
  const bool vec8 = a.part % 8 == 0 && x_stride % 8 == 0 && out_stride % 8 == 0 && aligned16(x) && aligned16(w) && aligned16(out);
  hipStream_t s = static_cast<hipStream_t>(stream);
  return dtype == TLF_DT_BF16 ? launch_rows_norm<unsigned short>(a, vec8, s) : launch_rows_norm<float>(a, vec8, s);
}
