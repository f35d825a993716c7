// In front of the attention of talk_attn.h: projection row [q | k | v] -> RMS norm over all of q and over all of k, rotation of
// the first rot_dims dimensions of every head in pairs (2 i, 2 i + 1), the score's constants (with a temperature per head) into
// q, keys and values into the paged caches.  One workgroup per token and part.  HBM bound: a row is read once and written once.
#include "talk_attn.h"

namespace tlf {

struct TalkPrepArgs {
  const void *proj;            // [n, ld]: q heads, k heads, v heads
  Partials part;               // or its partial sums
  int64_t ld;
  const void *q_norm, *k_norm; // [H * D], [G * D]
  const void *temp;            // [H] or NULL
  const int64_t *positions;
  const float *cos_sin;        // [max_pos, rot_dims]: cos of the pairs, then sin
  int32_t max_pos, rot_dims;
  const int32_t *slots;        // cache slot per token, negative: no store
  void *q_out;                 // [n, H, Dp]
  SinkCache c;
  int32_t n, H, vec;
  float eps, q_scale;
};

// blockIdx.y 0: q, 1: k, 2: v; pieces of 8 elements of a head, MAXC per thread
template <typename T, int MAXC, bool PART>
__global__ __launch_bounds__(256) void talk_prep_kernel(const TalkPrepArgs a) {
  __shared__ float part[4];
  const SinkCache &c = a.c;
  const int64_t tok = blockIdx.x;
  const int kind = blockIdx.y, heads = kind == 0 ? a.H : c.G, dims = kind < 2 ? c.D : c.Dv, padded = kind < 2 ? c.Dp : c.Vp;
  const int col0 = kind == 0 ? 0 : kind == 1 ? a.H * c.D : (a.H + c.G) * c.D;
  const int nch = padded / 8, pieces = heads * nch;
  const int64_t pos = a.positions[tok], slot = a.slots[tok];
  float x[MAXC][8], ss = 0.f;
#pragma unroll
  for (int q = 0; q < MAXC; ++q) {
    const int piece = static_cast<int>(threadIdx.x) + q * 256, head = piece / nch, d = (piece - head * nch) * 8;
#pragma unroll
    for (int e = 0; e < 8; ++e) x[q][e] = 0.f;
    if (piece >= pieces || d >= dims) continue;
    const int col = col0 + head * dims + d;
    if (a.vec) {
      if constexpr (PART) a.part.ld8(tok, col, x[q]);
      else Elem<T>::ld8(static_cast<const T *>(a.proj) + tok * a.ld + col, x[q]);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (d + e < dims) x[q][e] = PART ? a.part.ld(tok, col + e) : Elem<T>::ld(static_cast<const T *>(a.proj) + tok * a.ld + col + e);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = fmaf(x[q][e], x[q][e], ss);
  }
  float inv = 1.f;
  if (kind < 2) {
    ss = wave_sum(ss);
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = (part[0] + part[1]) + (part[2] + part[3]);
    inv = 1.0f / sqrtf(ss / static_cast<float>(heads * dims) + a.eps);
  }
  const bool store = slot >= 0 && slot < c.pages * c.bs;
  if (kind > 0 && !store) return;
  const int64_t page = store ? slot / c.bs : 0;
  const T *w = static_cast<const T *>(kind == 0 ? a.q_norm : a.k_norm);
  const int half = a.rot_dims / 2;
  const float *cs = pos >= 0 && pos < a.max_pos && half ? a.cos_sin + pos * a.rot_dims : nullptr;
#pragma unroll
  for (int q = 0; q < MAXC; ++q) {
    const int piece = static_cast<int>(threadIdx.x) + q * 256, head = piece / nch, d = (piece - head * nch) * 8;
    if (piece >= pieces) continue;
    if (kind < 2 && d < dims) {
      float wn[8];
      if (a.vec) Elem<T>::ld8(w + head * dims + d, wn);
      else
#pragma unroll
        for (int e = 0; e < 8; ++e) wn[e] = d + e < dims ? Elem<T>::ld(w + head * dims + d + e) : 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) x[q][e] = x[q][e] * inv * wn[e];
      if (cs && d < a.rot_dims) {
#pragma unroll
        for (int e = 0; e < 8; e += 2) {
          const int i = (d + e) / 2;
          if (i < half) {
            const float co = cs[i], si = cs[half + i], u = x[q][e], v = x[q][e + 1];
            x[q][e] = __fmul_rn(u, co) - __fmul_rn(v, si);
            x[q][e + 1] = __fmul_rn(v, co) + __fmul_rn(u, si);
          }
        }
      }
    }
    if (kind == 0) {
      const float m = a.q_scale * (a.temp ? Elem<T>::ld(static_cast<const T *>(a.temp) + head) : 1.f);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[q][e] *= m;
      Elem<T>::st8(static_cast<T *>(a.q_out) + (tok * a.H + head) * c.Dp + d, x[q]);
    } else {
      const int64_t crow = (page * c.G + head) * c.bs + (slot - page * c.bs);
      T *dst = static_cast<T *>(const_cast<void *>(kind == 1 ? c.k : c.v));
      Elem<T>::st8(dst + crow * padded + d, x[q]);
    }
  }
}

template <typename T, bool PART>
int launch_talk_prep(const TalkPrepArgs &a, int pieces, hipStream_t s) {
  const dim3 grid(a.n, 3);
  if (pieces <= 256) TLF_LAUNCH((talk_prep_kernel<T, 1, PART>), grid, dim3(256), 0, s, a);
  else if (pieces <= 512) TLF_LAUNCH((talk_prep_kernel<T, 2, PART>), grid, dim3(256), 0, s, a);
  else if (pieces <= 1024) TLF_LAUNCH((talk_prep_kernel<T, 4, PART>), grid, dim3(256), 0, s, a);
  else TLF_LAUNCH((talk_prep_kernel<T, 16, PART>), grid, dim3(256), 0, s, a);
  return launch_status();
}

}  // namespace tlf

extern "C" int tlf_talk_prep(const void *proj, int64_t proj_stride, const float *partials, int32_t splits, const float *scale,
                             const void *q_norm, const void *k_norm, const void *temp, const int64_t *positions,
                             const float *cos_sin, int32_t max_pos, int32_t rot_dims, const int32_t *slot_mapping, void *q_out,
                             void *k_cache, void *v_cache, int32_t n, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim,
                             int32_t block_size, int64_t num_pages, float eps, float score_scale, int32_t dtype, void *stream) {
  using namespace tlf;
  TalkPrepArgs a{};
  if (n < 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || rot_dims < 0 || rot_dims % 2 || rot_dims > dim) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (n == 0) return TLF_OK;
  if (int rc = partials_check(partials, scale, splits, dtype)) return rc;
  if (int rc = sink_cache_make(a.c, k_cache, v_cache, nullptr, 0, block_size, kv_heads, dim, vdim, num_pages)) return rc;
  const int64_t cols = static_cast<int64_t>(heads + kv_heads) * dim + static_cast<int64_t>(kv_heads) * vdim;
  if (proj_stride < cols || proj_stride > (1 << 28)) return TLF_E_SHAPE;
  const int64_t pq = static_cast<int64_t>(heads) * (a.c.Dp / 8), pv = static_cast<int64_t>(kv_heads) * (a.c.Vp / 8), pieces = pq > pv ? pq : pv;
  if (pieces > 4096) return TLF_E_SHAPE;
  if ((!proj && splits <= 1) || !q_norm || !k_norm || !positions || !slot_mapping || !q_out || (rot_dims && !cos_sin)) return TLF_E_NULL;
  if (!aligned16(q_out)) return TLF_E_ALIGN;
  a.proj = proj; a.ld = proj_stride;
  a.part = Partials{partials, scale, n * proj_stride, static_cast<int32_t>(proj_stride), splits};
  a.q_norm = q_norm; a.k_norm = k_norm; a.temp = temp; a.positions = positions; a.cos_sin = cos_sin; a.max_pos = max_pos;
  a.rot_dims = rot_dims; a.slots = slot_mapping; a.q_out = q_out; a.n = n; a.H = heads; a.eps = eps;
  a.q_scale = score_scale * kSinkLog2e;
  a.vec = dim % 8 == 0 && vdim % 8 == 0 && proj_stride % 8 == 0 && (splits > 1 || aligned16(proj)) && aligned16(q_norm) && aligned16(k_norm);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (splits > 1) return launch_talk_prep<unsigned short, true>(a, static_cast<int>(pieces), s);
  return dtype == TLF_DT_BF16 ? launch_talk_prep<unsigned short, false>(a, static_cast<int>(pieces), s)
                              : launch_talk_prep<float, false>(a, static_cast<int>(pieces), s);
}
