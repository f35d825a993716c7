// Grouped RMSNorm around an fp32 residual stream (sandwich norms): a row of `width` values is split into `groups`
// equal parts and each part is divided by its own root mean square.
//
//   mode embed:  x = table[id];                              h = norm(x) * w_next
//   mode add:    x = x + norm(y + y_bias) * w_post;           h = norm(x) * w_next
//   mode plain:  x = x + mult * (y + sum of extra rows);      h = norm(x) * (w_next + w_offset)
//
// (w_offset 1: a weight stored around zero.  The extra rows are a mixture of experts' results, found through an index, each
// with a weight of its own where there are weights; a negative index stands for the row of another tensor, the experts' input.)
// Modes embed and plain also exist with layer norm: h = ((x - mean) / sqrt(variance + eps) * w_next + b_next) * out_scale.
// The norm after a sublayer, the residual add and the norm in front of the next sublayer share their grouping, so a
// (row, group) pair is one independent unit: the three steps are one pass over memory.  HBM bound: y and x are read
// once, x and h written once.  The residual is fp32; y, h and the weights are T (bf16 or fp32); arithmetic is fp32.
#include "elem.h"

namespace tlf {

struct GroupNormArgs {
  const void *y;        // [rows, width] sublayer output, row stride y_stride (add mode)
  Partials part;        // or its partial sums
  int64_t y_stride;
  const void *y_bias;   // [width] or NULL
  const void *w_post;   // [width]
  const int64_t *ids;   // embed mode
  const void *table;    // [vocab, width]
  int32_t vocab;
  float *x;             // [rows, width] fp32 residual, updated in place
  const void *w_next;   // [width] or NULL: no h
  void *h;              // [rows, width]
  const void *extra;    // [*, extra_stride] or NULL: rows extra_rows[row * top + k], k < top (plain mode)
  const int32_t *extra_rows;
  const float *extra_weights;   // [rows, top] or NULL: 1
  const void *self;             // [rows, self_stride]: what a negative index stands for
  const void *b_next;           // [width], layer norm
  float out_scale;              // layer norm
  int64_t extra_stride, self_stride;
  int32_t top;
  float mult, w_offset;
  int64_t units;        // rows * groups
  int32_t width, groups, cols;
  float eps;
};

template <int TPR>
__device__ __forceinline__ float unit_sum(float v, float *part) {
  if (TPR <= 64) {
#pragma unroll
    for (int o = TPR / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
  }
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
  __syncthreads();
  v = 0.f;
#pragma unroll
  for (int w = 0; w < TPR / 64; ++w) v += part[w];
  return v;
}

template <typename T, int VEC>
__device__ __forceinline__ void ldv(const T *p, float (&f)[VEC]) {
  if constexpr (VEC == 8) Elem<T>::ld8(p, f);
  else f[0] = Elem<T>::ld(p);
}
template <typename T, int VEC>
__device__ __forceinline__ void stv(T *p, const float (&f)[VEC]) {
  if constexpr (VEC == 8) Elem<T>::st8(p, f);
  else Elem<T>::st(p, f[0]);
}

// MODE 0: embed, 1: add, 2: add with y as partial sums, 3: plain, 4: plain with y as partial sums
template <typename T, int VEC, int TPR, int MAXC, int MODE, bool LN>
__global__ __launch_bounds__(256) void groupnorm_kernel(const GroupNormArgs a) {
  __shared__ float part[4];
  const int tid = threadIdx.x, sub = tid % TPR;
  const int64_t unit = static_cast<int64_t>(blockIdx.x) * (256 / TPR) + tid / TPR;
  const bool active = unit < a.units;
  const int64_t safe = active ? unit : 0;
  const int64_t row = safe / a.groups;
  const int grp = static_cast<int>(safe - row * a.groups);
  const int nch = a.cols / VEC;
  const int col0 = grp * a.cols;
  float v[MAXC][VEC];
  float *xr = a.x + row * a.width + col0;
  const float inv_cols = 1.0f / static_cast<float>(a.cols);
  if constexpr (MODE == 0) {
    const int64_t id = a.ids[row];
    const bool ok = id >= 0 && id < a.vocab;
    const T *src = static_cast<const T *>(a.table) + (ok ? id : 0) * a.width + col0;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int ch = sub + c * TPR;
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[c][i] = 0.f;
      if (ch < nch && ok) ldv<T, VEC>(src + ch * VEC, v[c]);
    }
  } else if constexpr (MODE >= 3) {
    const T *yr = MODE == 3 ? static_cast<const T *>(a.y) + row * a.y_stride + col0 : nullptr;
    float xo[MAXC][VEC];
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int at = min(sub + c * TPR, nch - 1) * VEC;
      if constexpr (MODE == 3) {
        if (a.y) ldv<T, VEC>(yr + at, v[c]);
        else
#pragma unroll
          for (int i = 0; i < VEC; ++i) v[c][i] = 0.f;
      } else if constexpr (VEC == 8) a.part.ld8(row, col0 + at, v[c]);
      else v[c][0] = a.part.ld(row, col0 + at);
      ldv<float, VEC>(xr + at, xo[c]);
    }
    for (int k = 0; k < a.top; ++k) {
      const int64_t at = a.extra_rows[row * a.top + k];
      const T *er = (at >= 0 ? static_cast<const T *>(a.extra) + at * a.extra_stride : static_cast<const T *>(a.self) + row * a.self_stride) + col0;
      const float f0 = a.extra_weights ? a.extra_weights[row * a.top + k] : 1.f;
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        float f[VEC];
        ldv<T, VEC>(er + min(sub + c * TPR, nch - 1) * VEC, f);
#pragma unroll
        for (int i = 0; i < VEC; ++i) v[c][i] = fmaf(f[i], f0, v[c][i]);
      }
    }
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[c][i] = fmaf(v[c][i], a.mult, xo[c][i]);
  } else {
    const T *yr = MODE == 1 ? static_cast<const T *>(a.y) + row * a.y_stride + col0 : nullptr;
    const T *wp = static_cast<const T *>(a.w_post) + col0;
    const T *yb = a.y_bias ? static_cast<const T *>(a.y_bias) + col0 : nullptr;
    float xo[MAXC][VEC], w[MAXC][VEC];
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int at = min(sub + c * TPR, nch - 1) * VEC;
      if constexpr (MODE == 1) ldv<T, VEC>(yr + at, v[c]);
      else if constexpr (VEC == 8) a.part.ld8(row, col0 + at, v[c]);
      else v[c][0] = a.part.ld(row, col0 + at);
      ldv<float, VEC>(xr + at, xo[c]);
      ldv<T, VEC>(wp + at, w[c]);
    }
    if (yb) {
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        float b[VEC];
        ldv<T, VEC>(yb + min(sub + c * TPR, nch - 1) * VEC, b);
#pragma unroll
        for (int i = 0; i < VEC; ++i) v[c][i] += b[i];
      }
    }
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
      if (sub + c * TPR < nch)
#pragma unroll
        for (int i = 0; i < VEC; ++i) ss = fmaf(v[c][i], v[c][i], ss);
    ss = unit_sum<TPR>(ss, part);
    const float inv = 1.0f / sqrtf(ss * inv_cols + a.eps);
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[c][i] = fmaf(v[c][i] * inv, w[c][i], xo[c][i]);
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = sub + c * TPR;
    if (ch < nch) {
      if (active) stv<float, VEC>(xr + ch * VEC, v[c]);
#pragma unroll
      for (int i = 0; i < VEC; ++i) ss = LN ? ss + v[c][i] : fmaf(v[c][i], v[c][i], ss);
    }
  }
  if (a.w_next == nullptr) return;  // uniform
  ss = unit_sum<TPR>(ss, part);
  if constexpr (LN) {               // centred first: the variance is the mean of the squared deviations
    const float mean = ss * inv_cols;
    ss = 0.f;
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
      if (sub + c * TPR < nch)
#pragma unroll
        for (int i = 0; i < VEC; ++i) {
          v[c][i] -= mean;
          ss = fmaf(v[c][i], v[c][i], ss);
        }
    ss = unit_sum<TPR>(ss, part);
  }
  const float inv = 1.0f / sqrtf(ss * inv_cols + a.eps);
  const T *wn = static_cast<const T *>(a.w_next) + col0;
  T *hr = static_cast<T *>(a.h) + row * a.width + col0;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = sub + c * TPR;
    if (active && ch < nch) {
      float w[VEC];
      ldv<T, VEC>(wn + ch * VEC, w);
#pragma unroll
      for (int i = 0; i < VEC; ++i) w[i] = v[c][i] * inv * (w[i] + a.w_offset);
      if constexpr (LN) {
        float b[VEC];
        ldv<T, VEC>(static_cast<const T *>(a.b_next) + col0 + ch * VEC, b);
#pragma unroll
        for (int i = 0; i < VEC; ++i) w[i] = (w[i] + b[i]) * a.out_scale;
      }
      stv<T, VEC>(hr + ch * VEC, w);
    }
  }
}

template <typename T, int MODE, bool LN>
int launch_groupnorm(const GroupNormArgs &a, bool vec8, hipStream_t stream) {
#define TLF_GN(VEC, TPR, MAXC)                                                                               \
  TLF_LAUNCH((groupnorm_kernel<T, VEC, TPR, MAXC, MODE, LN>),                                                   \
             dim3(static_cast<unsigned>((a.units + (256 / TPR) - 1) / (256 / TPR))), dim3(256), 0, stream, a)
  if (vec8) {
    if (a.cols <= 128) TLF_GN(8, 16, 1);
    else if (a.cols <= 512) TLF_GN(8, 64, 1);
    else if (a.cols <= 1024) TLF_GN(8, 64, 2);
    else if (a.cols <= 2048) TLF_GN(8, 256, 1);
    else if (a.cols <= 4096) TLF_GN(8, 256, 2);
    else if (a.cols <= 8192) TLF_GN(8, 256, 4);
    else TLF_GN(8, 256, 8);
  } else {
    if (a.cols <= 256) TLF_GN(1, 64, 4);
    else if (a.cols <= 2048) TLF_GN(1, 256, 8);
    else TLF_GN(1, 256, 64);
  }
#undef TLF_GN
  return launch_status();
}

// kMode 0: embed, 1: add, 3: plain
template <int kMode, bool LN = false>
int groupnorm_entry(GroupNormArgs &a, int32_t rows, int32_t dtype, hipStream_t stream) {
  if (rows < 0 || a.width <= 0 || a.groups <= 0 || a.width % a.groups) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (rows == 0) return TLF_OK;
  if (!a.x || (a.w_next && !a.h)) return TLF_E_NULL;
  a.cols = a.width / a.groups;
  if (a.cols > 16384) return TLF_E_SHAPE;
  a.units = static_cast<int64_t>(rows) * a.groups;
  bool vec8 = a.cols % 8 == 0 && aligned16(a.x) && aligned16(a.w_next) && aligned16(a.h);
  if (kMode == 0)
    vec8 = vec8 && aligned16(a.table);
  else
    vec8 = vec8 && aligned16(a.y) && aligned16(a.y_bias) && aligned16(a.w_post) && a.y_stride % 8 == 0;
  if (kMode == 3) vec8 = vec8 && aligned16(a.extra) && a.extra_stride % 8 == 0 && aligned16(a.self) && a.self_stride % 8 == 0;
  if (LN) vec8 = vec8 && aligned16(a.b_next);
  if constexpr (kMode != 0)
    if (a.part.splits > 1) return launch_groupnorm<unsigned short, kMode + 1, LN>(a, vec8, stream);
  return dtype == TLF_DT_BF16 ? launch_groupnorm<unsigned short, kMode, LN>(a, vec8, stream)
                              : launch_groupnorm<float, kMode, LN>(a, vec8, stream);
}

}  // namespace tlf

extern "C" int tlf_group_rmsnorm_add(const void *y, int64_t y_stride, const float *partials, int32_t splits,
                                     const float *scale, const void *y_bias, const void *w_post, float *x,
                                     const void *w_next, void *h, int32_t rows, int32_t width, int32_t groups,
                                     float eps, int32_t dtype, void *stream) {
  tlf::GroupNormArgs a{};
  if (int rc = tlf::partials_check(partials, scale, splits, dtype)) return rc;
  if (rows > 0 && ((!y && splits <= 1) || !w_post)) return TLF_E_NULL;
  if (y_stride < width) return TLF_E_SHAPE;
  a.part = tlf::Partials{partials, scale, rows * y_stride, static_cast<int32_t>(y_stride), splits};
  a.y = y; a.y_stride = y_stride; a.y_bias = y_bias; a.w_post = w_post; a.x = x; a.w_next = w_next; a.h = h;
  a.width = width; a.groups = groups; a.eps = eps;
  return tlf::groupnorm_entry<1>(a, rows, dtype, static_cast<hipStream_t>(stream));
}

extern "C" int tlf_embed_group_rmsnorm(const int64_t *ids, const void *table, int32_t vocab, float *x,
                                       const void *w_next, float w_offset, void *h, int32_t rows, int32_t width,
                                       int32_t groups, float eps, int32_t dtype, void *stream) {
  tlf::GroupNormArgs a{};
  if (rows > 0 && (!ids || !table)) return TLF_E_NULL;
  if (vocab <= 0) return TLF_E_SHAPE;
  a.w_offset = w_offset;
  a.ids = ids; a.table = table; a.vocab = vocab; a.x = x; a.w_next = w_next; a.h = h;
  a.width = width; a.groups = groups; a.eps = eps;
  return tlf::groupnorm_entry<0>(a, rows, dtype, static_cast<hipStream_t>(stream));
}

extern "C" int tlf_residual_rmsnorm(const void *y, int64_t y_stride, const float *partials, int32_t splits,
                                    const float *scale, const void *extra, int64_t extra_stride, const int32_t *extra_rows,
                                    int32_t top, float mult, float *x, const void *w_next, float w_offset, void *h,
                                    int32_t rows, int32_t width, float eps, int32_t dtype, void *stream) {
  tlf::GroupNormArgs a{};
  if (int rc = tlf::partials_check(partials, scale, splits, dtype)) return rc;
  if (rows > 0 && ((!y && splits <= 1) || (top > 0 && (!extra || !extra_rows)))) return TLF_E_NULL;
  if (y_stride < width || top < 0 || (top > 0 && extra_stride < width)) return TLF_E_SHAPE;
  a.part = tlf::Partials{partials, scale, rows * y_stride, static_cast<int32_t>(y_stride), splits};
  a.y = y; a.y_stride = y_stride; a.x = x; a.w_next = w_next; a.h = h;
  a.extra = extra; a.extra_stride = extra_stride; a.extra_rows = extra_rows; a.top = top; a.mult = mult; a.w_offset = w_offset;
  a.width = width; a.groups = 1; a.eps = eps;
  return tlf::groupnorm_entry<3>(a, rows, dtype, static_cast<hipStream_t>(stream));
}

extern "C" int tlf_embed_layernorm(const int64_t *ids, const void *table, int32_t vocab, float *x, const void *w_next,
                                   const void *b_next, float out_scale, void *h, int32_t rows, int32_t width, float eps,
                                   int32_t dtype, void *stream) {
  tlf::GroupNormArgs a{};
  if (rows > 0 && (!ids || !table || !w_next || !b_next)) return TLF_E_NULL;
  if (vocab <= 0) return TLF_E_SHAPE;
  a.ids = ids; a.table = table; a.vocab = vocab; a.x = x; a.w_next = w_next; a.b_next = b_next; a.out_scale = out_scale; a.h = h;
  a.width = width; a.groups = 1; a.eps = eps;
  return tlf::groupnorm_entry<0, true>(a, rows, dtype, static_cast<hipStream_t>(stream));
}

extern "C" int tlf_residual_layernorm(const void *y, int64_t y_stride, const float *partials, int32_t splits, const float *scale,
                                      const void *extra, int64_t extra_stride, const int32_t *extra_rows,
                                      const float *extra_weights, int32_t top, const void *self, int64_t self_stride, float *x,
                                      const void *w_next, const void *b_next, float out_scale, void *h, int32_t rows,
                                      int32_t width, float eps, int32_t dtype, void *stream) {
  tlf::GroupNormArgs a{};
  if (int rc = tlf::partials_check(partials, scale, splits, dtype)) return rc;
  if (rows > 0 && (!w_next || !b_next || (top > 0 && (!extra || !extra_rows || !self)))) return TLF_E_NULL;
  if ((y && y_stride < width) || top < 0 || (top > 0 && (extra_stride < width || self_stride < width))) return TLF_E_SHAPE;
  a.part = tlf::Partials{partials, scale, rows * y_stride, static_cast<int32_t>(y_stride), splits};
  a.y = y; a.y_stride = y_stride; a.x = x; a.w_next = w_next; a.b_next = b_next; a.out_scale = out_scale; a.h = h;
  a.extra = extra; a.extra_stride = extra_stride; a.extra_rows = extra_rows; a.extra_weights = extra_weights; a.top = top;
  a.self = self; a.self_stride = self_stride; a.mult = 1.f;
  a.width = width; a.groups = 1; a.eps = eps;
  return tlf::groupnorm_entry<3, true>(a, rows, dtype, static_cast<hipStream_t>(stream));
}
