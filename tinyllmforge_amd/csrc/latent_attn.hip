// Latent attention (geometry in latent_attn.h): everything but the two matrix-core attention kernels.
//
//   latent_prep_kernel    projection row [q | latent | rotated key] -> rotated queries, normed latent and rotated key into
//                         the paged cache; where queries come through a latent of their own, that one normed; output gates
//   head_gemm_kernel      y[row, h] = W[h] x[row, h] for every head (the queries' way into the latent space)
//   latent_rows_kernel    one workgroup per (query row, head): 32-bit mode, and sizes the matrix-core kernel does not take
//   latent_values_kernel  sum of the key splits, softmax denominator, Uv_h
//   latent_gather_kernel  cache rows of a step's long portions as one dense matrix (input of the expansion)
#include "latent_attn.h"

namespace tlf {

struct LatentPrepArgs {
  LatentShape s;
  const void *proj;
  Partials part;
  int64_t ld;
  int32_t off;              // column of the latent in a projection row
  const void *norm;         // [rank]
  const int64_t *positions;
  const float *cos_sin;     // [max_pos, rot]: cos of the pairs, then sin
  int32_t max_pos;
  const int32_t *slots;     // cache row per token, negative: no store
  int64_t num_slots;
  void *q_out;              // [n, H, Dq]
  void *cache;              // [slots, Lp]
  int32_t n, vec;           // vec: parts of a projection row may be read 8 elements at a time
  float eps;
  int32_t halves;           // rotation: pairs (i, i + rot / 2) instead of (2 i, 2 i + 1)
  int32_t latents;          // blockIdx.y == 0 prepares latents (and gates); then query latents, then queries
  const void *cq_norm;      // [cq_rank] or NULL
  void *cq_out;             // [n, cq_ld], zeros from cq_rank on
  int32_t cq_col, cq_rank, cq_ld, gate_col;
  float *gate_out;          // [n, H] or NULL: sigmoid
};

template <typename T, bool PART>
__device__ __forceinline__ float prep_ld(const LatentPrepArgs &a, int64_t tok, int col) {
  return PART ? a.part.ld(tok, col) : Elem<T>::ld(static_cast<const T *>(a.proj) + tok * a.ld + col);
}
// 8 values from column `col` on of a part of `len` values (zeros past its end), starting at value `d`
template <typename T, bool PART>
__device__ __forceinline__ void prep_ld8(const LatentPrepArgs &a, int64_t tok, int col, int d, int len, float (&f)[8]) {
  if (a.vec) {
    if constexpr (PART) a.part.ld8(tok, col + d, f);
    else Elem<T>::ld8(static_cast<const T *>(a.proj) + tok * a.ld + col + d, f);
    return;
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) f[e] = d + e < len ? prep_ld<T, PART>(a, tok, col + d + e) : 0.f;
}
__device__ __forceinline__ void turn8(const LatentPrepArgs &a, const float *cs, int d, float (&f)[8]) {
  if (cs == nullptr) return;
  const int half = a.s.rot / 2;
#pragma unroll
  for (int e = 0; e < 8; e += 2) {
    const int i = (d + e) / 2;
    if (i < half) {
      const float co = cs[i], si = cs[half + i], u = f[e], v = f[e + 1];
      f[e] = __fmul_rn(u, co) - __fmul_rn(v, si);
      f[e + 1] = __fmul_rn(v, co) + __fmul_rn(u, si);
    }
  }
}

// The partners, rot / 2 away, of piece d .. d + 7 of the rotated part that begins at column `col`.
template <typename T, bool PART>
__device__ __forceinline__ void partner8(const LatentPrepArgs &a, int64_t tok, int col, int d, float (&p)[8]) {
  const int half = a.s.rot / 2;
  if (a.vec && half % 8 == 0) {
    prep_ld8<T, PART>(a, tok, col, d < half ? d + half : d - half, a.s.rot, p);
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int i = d + e;
      p[e] = i < a.s.rot ? prep_ld<T, PART>(a, tok, col + (i < half ? i + half : i - half)) : 0.f;
    }
  }
}

__device__ __forceinline__ void turn8_halves(const LatentPrepArgs &a, const float *cs, int d, const float (&p)[8], float (&f)[8]) {
  if (cs == nullptr) return;
  const int half = a.s.rot / 2;
  if (half % 8 == 0) {                                     // the piece lies on one side
    const float *c = cs + (d < half ? d : d - half);
    const float sign = d < half ? -1.f : 1.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = __fmul_rn(f[e], c[e]) + sign * __fmul_rn(p[e], c[half + e]);
    return;
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const int i = d + e;
    if (i < half) f[e] = __fmul_rn(f[e], cs[i]) - __fmul_rn(p[e], cs[half + i]);
    else if (i < a.s.rot) f[e] = __fmul_rn(f[e], cs[i - half]) + __fmul_rn(p[e], cs[i]);
  }
}

// blockIdx.y == 0 with `latents`: the latents of TOK tokens, a wave each; then, with cq_norm, their query latents; then 256
// 8-value pieces of those tokens' queries, all loads in flight before the first is used
template <typename T, bool PART, int TOK>
__global__ __launch_bounds__(256) void latent_prep_kernel(const LatentPrepArgs a) {
  const LatentShape &s = a.s;
  const int64_t tok0 = static_cast<int64_t>(blockIdx.x) * TOK;
  if (a.cq_norm && static_cast<int>(blockIdx.y) == a.latents) {
    const int64_t tok = tok0 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if ((threadIdx.x >> 6) >= TOK || tok >= a.n) return;   // whole waves leave together
    const T *w = static_cast<const T *>(a.cq_norm);
    T *row = static_cast<T *>(a.cq_out) + tok * a.cq_ld;
    constexpr int kKeep = 2;                               // pieces of 8 a lane holds, longer rows are read twice
    float f[kKeep][8], ss = 0.f;
#pragma unroll
    for (int k = 0; k < kKeep; ++k) {
      const int d = (lane + k * 64) * 8;
#pragma unroll
      for (int e = 0; e < 8; ++e) f[k][e] = 0.f;
      if (d < a.cq_rank) prep_ld8<T, PART>(a, tok, a.cq_col, d, a.cq_rank, f[k]);
#pragma unroll
      for (int e = 0; e < 8; ++e) ss = fmaf(f[k][e], f[k][e], ss);
    }
    for (int d = (lane + kKeep * 64) * 8; d < a.cq_rank; d += 512) {
      float t[8];
      prep_ld8<T, PART>(a, tok, a.cq_col, d, a.cq_rank, t);
#pragma unroll
      for (int e = 0; e < 8; ++e) ss = fmaf(t[e], t[e], ss);
    }
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / static_cast<float>(a.cq_rank) + a.eps);
    for (int d = lane * 8, k = 0; d < a.cq_ld; d += 512, ++k) {
      float t[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (d < a.cq_rank) {
        if (k >= kKeep) prep_ld8<T, PART>(a, tok, a.cq_col, d, a.cq_rank, t);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          if (k < kKeep) t[e] = k == 0 ? f[0][e] : f[1][e];
          t[e] = d + e < a.cq_rank ? t[e] * inv * Elem<T>::ld(w + d + e) : 0.f;
        }
      }
      Elem<T>::st8(row + d, t);
    }
    return;
  }
  if (a.latents && blockIdx.y == 0) {
    const int64_t tok = tok0 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if ((threadIdx.x >> 6) >= TOK || tok >= a.n) return;   // whole waves leave together
    if (a.gate_out)
      for (int h = lane; h < s.H; h += 64) a.gate_out[tok * s.H + h] = sigmoid_f32(prep_ld<T, PART>(a, tok, a.gate_col + h));
    const int64_t slot = a.slots[tok], pos = a.positions[tok];
    const float *cs = pos >= 0 && pos < a.max_pos ? a.cos_sin + pos * s.rot : nullptr;
    constexpr int kKeep = 3;   // pieces of 8 a lane holds: rank <= 1536
    const T *w = static_cast<const T *>(a.norm);
    float f[kKeep][8], t[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < kKeep; ++k) {
      const int d = (lane + k * 64) * 8;
      if (d < s.rank) prep_ld8<T, PART>(a, tok, a.off, d, s.rank, f[k]);
    }
    if (lane * 8 < s.rot) prep_ld8<T, PART>(a, tok, a.off + s.rank, lane * 8, s.rot, t);
    if (slot < 0 || slot >= a.num_slots) return;
    T *row = static_cast<T *>(a.cache) + slot * s.Lp;
#pragma unroll
    for (int k = 0; k < kKeep; ++k)
      if ((lane + k * 64) * 8 < s.rank) {
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = fmaf(f[k][e], f[k][e], ss);
      }
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / static_cast<float>(s.rank) + a.eps);
#pragma unroll
    for (int k = 0; k < kKeep; ++k) {
      const int d = (lane + k * 64) * 8;
      if (d < s.rank) {
#pragma unroll
        for (int e = 0; e < 8; ++e) f[k][e] = d + e < s.rank ? f[k][e] * inv * Elem<T>::ld(w + d + e) : 0.f;
        Elem<T>::st8(row + d, f[k]);
      }
    }
    for (int d = lane * 8; d < s.Lp - s.Ra; d += 512) {
      if (d >= 512) {           // rot > 512
#pragma unroll
        for (int e = 0; e < 8; ++e) t[e] = 0.f;
        if (d < s.rot) prep_ld8<T, PART>(a, tok, a.off + s.rank, d, s.rot, t);
      }
      if (d < s.rot) {
        if (a.halves) {
          float p[8];
          partner8<T, PART>(a, tok, a.off + s.rank, d, p);
          turn8_halves(a, cs, d, p, t);
        } else {
          turn8(a, cs, d, t);
        }
      }
      Elem<T>::st8(row + s.Ra + d, t);
    }
    return;
  }
  const int nch = s.Dq / 8;
  const int item = (blockIdx.y - a.latents - (a.cq_norm ? 1 : 0)) * 256 + threadIdx.x;
  if (item >= s.H * nch) return;
  const int h = item / nch, d = (item - h * nch) * 8;
  const int col = h * (s.dim + s.rot);
  const bool own = d < s.Da, turned = !own && d < s.Da + s.rot;
  float f[TOK][8], p[TOK][8];
  int64_t pos[TOK];
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const int64_t tok = min(tok0 + k, static_cast<int64_t>(a.n) - 1);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[k][e] = p[k][e] = 0.f;
    if (turned && a.halves) partner8<T, PART>(a, tok, col + s.dim, d - s.Da, p[k]);
    if (own) prep_ld8<T, PART>(a, tok, col, d, s.dim, f[k]);
    else if (turned) prep_ld8<T, PART>(a, tok, col + s.dim, d - s.Da, s.rot, f[k]);
    pos[k] = turned ? a.positions[tok] : 0;
  }
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    if (tok0 + k >= a.n) return;
    if (turned) {
      const float *cs = pos[k] >= 0 && pos[k] < a.max_pos ? a.cos_sin + pos[k] * s.rot : nullptr;
      if (a.halves) turn8_halves(a, cs, d - s.Da, p[k], f[k]);
      else turn8(a, cs, d - s.Da, f[k]);
    }
    Elem<T>::st8(static_cast<T *>(a.q_out) + ((tok0 + k) * s.H + h) * s.Dq + d, f[k]);
  }
}

// ---------------------------------------------------------------------------------------------------------------
// y[row, h, n] = sum_k W[h, n, k] x[row, h, k].  Rows n < n_main have weights in k < k_main only.
struct HeadGemmArgs {
  const void *x, *w;
  void *y;
  int32_t rows, H, N, K, n_main, k_main;
};

// bf16: a workgroup takes one head, 64 rows and 64 outputs; weights and inputs straight from L2 into MFMA operands
__global__ __launch_bounds__(256) void head_gemm_kernel(const HeadGemmArgs a) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = lane & 15, g = lane >> 4;
  const int h = blockIdx.x, row0 = blockIdx.y * 64, n0 = (blockIdx.z * 4 + wave) * 16;
  if (n0 >= a.N) return;
  const int kend = n0 + 16 <= a.n_main ? a.k_main : a.K;
  const unsigned short *wp = static_cast<const unsigned short *>(a.w) + (static_cast<int64_t>(h) * a.N + n0 + n) * a.K + g * 8;
  const unsigned short *xp[4];
#pragma unroll
  for (int j = 0; j < 4; ++j)
    xp[j] = static_cast<const unsigned short *>(a.x) + (static_cast<int64_t>(min(row0 + j * 16 + n, a.rows - 1)) * a.H + h) * a.K + g * 8;
  floatx4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = floatx4{0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < kend; k += 32) {
    Pack16 wf, xf[4];
    wf.u = *reinterpret_cast<const uint4 *>(wp + k);
#pragma unroll
    for (int j = 0; j < 4; ++j) xf[j].u = *reinterpret_cast<const uint4 *>(xp[j] + k);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf.v, xf[j].v, acc[j], 0, 0, 0);
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int row = row0 + j * 16 + n;
    if (row < a.rows)
      *reinterpret_cast<uint2 *>(static_cast<unsigned short *>(a.y) + (static_cast<int64_t>(row) * a.H + h) * a.N + n0 + g * 4) =
          make_uint2(pack_bf16x2(acc[j][0], acc[j][1]), pack_bf16x2(acc[j][2], acc[j][3]));
  }
}

__global__ __launch_bounds__(256) void head_gemm_f32_kernel(const HeadGemmArgs a) {
  const int64_t at = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (at >= static_cast<int64_t>(a.rows) * a.H * a.N) return;
  const int64_t rh = at / a.N;
  const int nn = static_cast<int>(at - rh * a.N), h = static_cast<int>(rh % a.H);
  const float *x = static_cast<const float *>(a.x) + rh * a.K;
  const float *w = static_cast<const float *>(a.w) + (static_cast<int64_t>(h) * a.N + nn) * a.K;
  float s = 0.f;
  for (int k = 0; k < a.K; ++k) s = fmaf(x[k], w[k], s);
  static_cast<float *>(a.y)[at] = s;
}

// ---------------------------------------------------------------------------------------------------------------
struct LatentRowsArgs {
  LatentShape s;
  LatentCache c;
  const void *q;             // [rows, H, Lp]
  const int64_t *positions;
  const int32_t *slots;      // negative: padding row
  const int32_t *row_seq;    // [rows] or NULL: row r belongs to sequence r
  float *part;               // [rows, H, Rp] mixed latents (not divided)
  float *ml;                 // [rows, H, 2] maximum (log2 units) and denominator
  int32_t window;
  float scale_log2;
};

// E = values of a cache row per lane
template <typename T, int E>
__global__ __launch_bounds__(256) void latent_rows_kernel(const LatentRowsArgs a) {
  __shared__ float sm[4], sl[4], so[4][E * 64];
  const LatentShape &s = a.s;
  const int row = blockIdx.y, h = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int64_t rh = static_cast<int64_t>(row) * s.H + h;
  const int i = static_cast<int>(a.positions[row]);
  const bool live = a.slots[row] >= 0 && i >= 0;
  float q[E], o[E], m = -INFINITY, l = 0.f;
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int d = e * 64 + lane;
    q[e] = d < s.Lp ? Elem<T>::ld(static_cast<const T *>(a.q) + rh * s.Lp + d) * a.scale_log2 : 0.f;
    o[e] = 0.f;
  }
  if (live) {
    const int32_t *bt = a.c.bt + (a.row_seq ? a.row_seq[row] : row) * a.c.bt_stride;
    for (int j = max(0, i - a.window + 1) + wave; j <= i; j += 4) {
      const T *kr = static_cast<const T *>(a.c.rows) + latent_row(a.c, bt, j) * s.Lp;
      float k[E], dot = 0.f;
#pragma unroll
      for (int e = 0; e < E; ++e) {
        const int d = e * 64 + lane;
        k[e] = d < s.Lp ? Elem<T>::ld(kr + d) : 0.f;
        dot = fmaf(q[e], k[e], dot);
      }
      dot = wave_sum(dot);
      const float mn = fmaxf(m, dot), back = exp2f(m - mn), p = exp2f(dot - mn);
      l = fmaf(l, back, p);
#pragma unroll
      for (int e = 0; e < E; ++e) o[e] = fmaf(o[e], back, p * k[e]);
      m = mn;
    }
  }
  if (lane == 0) { sm[wave] = m; sl[wave] = l; }
#pragma unroll
  for (int e = 0; e < E; ++e) so[wave][e * 64 + lane] = o[e];
  __syncthreads();
  const float mx = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
  float f[4], den = 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    f[w] = sl[w] > 0.f ? exp2f(sm[w] - mx) : 0.f;
    den = fmaf(sl[w], f[w], den);
  }
  for (int d = threadIdx.x; d < s.Rp; d += 256)
    a.part[rh * s.Rp + d] = d < s.Ra ? so[0][d] * f[0] + so[1][d] * f[1] + so[2][d] * f[2] + so[3][d] * f[3] : 0.f;
  if (threadIdx.x == 0) { a.ml[rh * 2] = mx; a.ml[rh * 2 + 1] = den; }
}

// ---------------------------------------------------------------------------------------------------------------
struct LatentValuesArgs {
  LatentShape s;
  const float *part, *ml;   // pieces of Rp values, and their maximum and denominator
  const int32_t *plan;      // of the tile kernel, NULL: one piece per (row, head), in that order
  LatentJobs jb;
  const int32_t *row_seq;   // [rows] with jb.cu_q: sequence of a row
  const void *uv;           // [H, Vp, Rp], Vp = vdim rounded up to 16
  const float *gate;        // [rows, H] or NULL
  void *out;                // [rows, ldo]
  int64_t ldo;
  int32_t rows, Vp, wgs;
};

// The pieces of (row, head): units first, first + step, ...
struct Pieces {
  int64_t first;
  int32_t step, count;
};
__device__ __forceinline__ Pieces latent_pieces(const LatentValuesArgs &a, int row, int h) {
  if (!a.plan) return Pieces{static_cast<int64_t>(row) * a.s.H + h, 0, 1};
  const LatentJobs &j = a.jb;
  int seq = row, r = 0;
  if (j.cu_q) {
    seq = a.row_seq[row];
    r = row + j.first_row - j.cu_q[seq];
    seq -= j.first_seq;
  }
  const int pass = h / j.hpp, job = (seq * j.xtiles + r / j.bq) * j.passes + pass;
  const int32_t *rec = a.plan + latent_plan_jobs(a.wgs, j.jobs) + 2 * job;
  const bool ok = rec[0] >= 0 && rec[1] >= 0 && rec[1] <= kLatentMaxPieces && rec[0] + rec[1] <= latent_max_pieces(a.wgs, j.jobs);
  return Pieces{static_cast<int64_t>(rec[0]) * j.units + r % j.bq * j.hpp + h - pass * j.hpp, j.units, ok ? rec[1] : 0};
}
// Maximum and inverse denominator over the pieces (inverse 0: no keys).
__device__ __forceinline__ void pieces_total(const LatentValuesArgs &a, const Pieces &p, float &mx, float &inv) {
  mx = -INFINITY;
  for (int k = 0; k < p.count; ++k) {
    const float2 v = *reinterpret_cast<const float2 *>(a.ml + (p.first + static_cast<int64_t>(k) * p.step) * 2);
    if (v.y > 0.f) mx = fmaxf(mx, v.x);
  }
  float den = 0.f;
  for (int k = 0; k < p.count; ++k) {
    const float2 v = *reinterpret_cast<const float2 *>(a.ml + (p.first + static_cast<int64_t>(k) * p.step) * 2);
    if (v.y > 0.f) den = fmaf(v.y, exp2f(v.x - mx), den);
  }
  inv = den > 0.f ? 1.0f / den : 0.f;
}
__device__ __forceinline__ float piece_weight(const LatentValuesArgs &a, const Pieces &p, int k, float mx, float inv) {
  const float2 v = *reinterpret_cast<const float2 *>(a.ml + (p.first + static_cast<int64_t>(k) * p.step) * 2);
  return v.y > 0.f ? exp2f(v.x - mx) * inv : 0.f;
}

// bf16: a workgroup takes one head, 16 rows and 64 outputs; the mixed latents of the rows go through LDS once
__global__ __launch_bounds__(256) void latent_values_kernel(const LatentValuesArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned short lat[];   // [16][Rp + 8]
  __shared__ float wt[16][kLatentMaxPieces + 1];
  __shared__ Pieces pcs[16];
  const LatentShape &s = a.s;
  const int h = blockIdx.x, row0 = blockIdx.y * 16, tid = threadIdx.x;
  const int stride = s.Rp + 8;
  {
    // 16 lanes per row, a piece each at a time
    const int r = tid >> 4, j = tid & 15;
    const Pieces p = row0 + r < a.rows ? latent_pieces(a, row0 + r, h) : Pieces{0, 0, 0};
    if (j == 0) pcs[r] = p;
    float mx = -INFINITY, den = 0.f;
    for (int k0 = 0; k0 < p.count; k0 += 16) {
      float2 v = make_float2(-INFINITY, 0.f);
      if (k0 + j < p.count) v = *reinterpret_cast<const float2 *>(a.ml + (p.first + static_cast<int64_t>(k0 + j) * p.step) * 2);
      const float m1 = v.y > 0.f ? v.x : -INFINITY;
      float mn = m1;
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) mn = fmaxf(mn, __shfl_xor(mn, o, 64));
      mn = fmaxf(mn, mx);
      den = den * (mx == mn ? 1.f : exp2f(mx - mn)) + group_sum<16>(v.y > 0.f ? v.y * exp2f(m1 - mn) : 0.f);
      mx = mn;
      if (k0 + j < p.count) wt[r][k0 + j] = m1;
    }
    const float inv = den > 0.f ? 1.0f / den : 0.f;
    for (int k = j; k < p.count; k += 16) wt[r][k] = wt[r][k] == -INFINITY ? 0.f : exp2f(wt[r][k] - mx) * inv;
  }
  __syncthreads();
  const int nch = s.Rp / 8;
  for (int item = tid; item < 16 * nch; item += 256) {
    const int r = item / nch, d = (item - r * nch) * 8;
    const Pieces p = pcs[r];
    float o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    const float *src = a.part + p.first * s.Rp + d;
    const int64_t step = static_cast<int64_t>(p.step) * s.Rp;
    for (int k0 = 0; k0 < p.count; k0 += 4) {
      float f[4][8];
#pragma unroll
      for (int k = 0; k < 4; ++k) Elem<float>::ld8(src + min(k0 + k, p.count - 1) * step, f[k]);
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float w = k0 + k < p.count ? wt[r][k0 + k] : 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = fmaf(w, f[k][e], o[e]);
      }
    }
    *reinterpret_cast<uint4 *>(lat + r * stride + d) = pack8(o);
  }
  __syncthreads();
  const int lane = tid & 63, wave = tid >> 6, n = lane & 15, g = lane >> 4;
  const int v0 = (blockIdx.z * 4 + wave) * 16;
  if (v0 >= a.Vp) return;
  const unsigned short *wp = static_cast<const unsigned short *>(a.uv) + (static_cast<int64_t>(h) * a.Vp + v0 + n) * s.Rp + g * 8;
  floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = 0; k < s.Rp; k += 32) {
    Pack16 wf, xf;
    wf.u = *reinterpret_cast<const uint4 *>(wp + k);
    xf.u = *reinterpret_cast<const uint4 *>(lat + n * stride + k + g * 8);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf.v, xf.v, acc, 0, 0, 0);
  }
  const int row = row0 + n;
  if (row >= a.rows) return;
  if (a.gate) acc *= a.gate[static_cast<int64_t>(row) * s.H + h];
  unsigned short *o = static_cast<unsigned short *>(a.out) + row * a.ldo + static_cast<int64_t>(h) * s.vdim + v0 + g * 4;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (v0 + g * 4 + e < s.vdim) o[e] = float_to_bf16_bits(acc[e]);
}

template <typename T>
__global__ __launch_bounds__(256) void latent_values_rows_kernel(const LatentValuesArgs a) {
  extern __shared__ __attribute__((aligned(16))) float mixed[];   // [Rp]
  const LatentShape &s = a.s;
  const int h = blockIdx.x, row = blockIdx.y;
  const Pieces p = latent_pieces(a, row, h);
  float mx, inv;
  pieces_total(a, p, mx, inv);
  for (int d = threadIdx.x; d < s.Rp; d += 256) {
    float o = 0.f;
    for (int k = 0; k < p.count; ++k) {
      const float w = piece_weight(a, p, k, mx, inv);
      if (w > 0.f) o = fmaf(w, a.part[(p.first + static_cast<int64_t>(k) * p.step) * s.Rp + d], o);
    }
    mixed[d] = Elem<T>::rnd(o);
  }
  __syncthreads();
  for (int v = threadIdx.x; v < s.vdim; v += 256) {
    const T *w = static_cast<const T *>(a.uv) + (static_cast<int64_t>(h) * a.Vp + v) * s.Rp;
    float o = 0.f;
    for (int r = 0; r < s.rank; ++r) o = fmaf(mixed[r], Elem<T>::ld(w + r), o);
    if (a.gate) o *= a.gate[static_cast<int64_t>(row) * s.H + h];
    Elem<T>::st(static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(h) * s.vdim + v, o);
  }
}

// ---------------------------------------------------------------------------------------------------------------
// Keys of portion s: positions max(0, start - window + 1) .. start + tokens - 1, at dense rows kv_off[s] ..
__global__ __launch_bounds__(256) void latent_gather_kernel(const LatentCache c, const int32_t *cu_q, const int32_t *starts,
                                                            const int32_t *kv_off, int32_t first_seq, int32_t window,
                                                            int32_t Lp, unsigned short *out) {
  const int seq = first_seq + blockIdx.y;
  const int at = kv_off[blockIdx.y], count = kv_off[blockIdx.y + 1] - at;
  const int k0 = max(0, starts[seq] - window + 1);
  const int nch = Lp / 8;
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  const int r = static_cast<int>(item / nch), ch = static_cast<int>(item - static_cast<int64_t>(r) * nch);
  if (r >= count) return;
  const int64_t row = latent_row(c, c.bt + seq * c.bt_stride, k0 + r);
  *reinterpret_cast<uint4 *>(out + static_cast<int64_t>(at + r) * Lp + ch * 8) =
      *reinterpret_cast<const uint4 *>(static_cast<const unsigned short *>(c.rows) + row * Lp + ch * 8);
}

}  // namespace tlf

extern "C" int tlf_latent_prep(const void *proj, int64_t proj_stride, const float *partials, int32_t splits,
                               const float *scale, int32_t latent_col, const void *norm_weight, const int64_t *positions,
                               const float *cos_sin, int32_t max_pos, int32_t halves, const int32_t *slot_mapping,
                               int64_t num_slots, void *q_out, void *cache, int32_t cq_col, int32_t cq_rank, const void *cq_norm,
                               void *cq_out, int32_t cq_stride, int32_t gate_col, float *gate_out, int32_t n, int32_t heads,
                               int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim, float eps, int32_t dtype, void *stream) {
  using namespace tlf;
  LatentPrepArgs a{};
  if (n < 0 || !latent_shape(a.s, heads, dim, rot_dim, rank, vdim)) return TLF_E_SHAPE;
  if (!q_out && !cache) return TLF_E_NULL;
  if (q_out && proj_stride < heads * (dim + rot_dim)) return TLF_E_SHAPE;
  if (cache && (latent_col < (q_out ? heads * (dim + rot_dim) : 0) || proj_stride < latent_col + rank + rot_dim)) return TLF_E_SHAPE;
  if (cq_norm && (cq_rank <= 0 || cq_col < 0 || proj_stride < cq_col + cq_rank || cq_stride < cq_rank || cq_stride % 8)) return TLF_E_SHAPE;
  if (gate_out && (!cache || gate_col < 0 || proj_stride < gate_col + heads)) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (n == 0) return TLF_OK;
  if (int rc = partials_check(partials, scale, splits, dtype)) return rc;
  if ((!proj && splits <= 1) || !positions || (rot_dim && !cos_sin) || (cache && (!slot_mapping || !norm_weight)) || (cq_norm && !cq_out)) return TLF_E_NULL;
  if (!aligned16(q_out) || !aligned16(cache) || !aligned16(cq_out)) return TLF_E_ALIGN;
  a.proj = proj; a.ld = proj_stride; a.off = latent_col; a.norm = norm_weight; a.positions = positions; a.cos_sin = cos_sin;
  a.part = Partials{partials, scale, n * proj_stride, static_cast<int32_t>(proj_stride), splits};
  a.max_pos = max_pos; a.slots = slot_mapping; a.num_slots = num_slots; a.q_out = q_out; a.cache = cache; a.n = n; a.eps = eps;
  a.halves = halves; a.latents = cache ? 1 : 0;
  a.cq_norm = cq_norm; a.cq_out = cq_out; a.cq_col = cq_col; a.cq_rank = cq_rank; a.cq_ld = cq_stride;
  a.gate_col = gate_col; a.gate_out = gate_out;
  a.vec = dim % 8 == 0 && rot_dim % 8 == 0 && proj_stride % 8 == 0 && (splits > 1 || aligned16(proj)) &&
          (!cache || (rank % 8 == 0 && latent_col % 8 == 0)) && (!cq_norm || (cq_rank % 8 == 0 && cq_col % 8 == 0));
  const int tok = splits <= 1 && n > 1024 ? 4 : 1;
  const dim3 grid((n + tok - 1) / tok, a.latents + (cq_norm ? 1 : 0) + (q_out ? (heads * (a.s.Dq / 8) + 255) / 256 : 0));
  hipStream_t s = static_cast<hipStream_t>(stream);
#define TLF_PREP(T, PART)                                                                        \
  do {                                                                                           \
    if (tok == 4) TLF_LAUNCH((latent_prep_kernel<T, PART, 4>), grid, dim3(256), 0, s, a);        \
    else TLF_LAUNCH((latent_prep_kernel<T, PART, 1>), grid, dim3(256), 0, s, a);                 \
  } while (0)
  if (splits > 1) TLF_PREP(unsigned short, true);
  else if (dtype == TLF_DT_BF16) TLF_PREP(unsigned short, false);
  else TLF_PREP(float, false);
#undef TLF_PREP
  return launch_status();
}

extern "C" int tlf_head_gemm(const void *x, const void *w, void *y, int32_t rows, int32_t heads, int32_t N, int32_t K,
                             int32_t n_main, int32_t k_main, int32_t dtype, void *stream) {
  using namespace tlf;
  if (rows < 0 || heads <= 0 || N <= 0 || K <= 0 || N % 16 || K % 32 || n_main < 0 || k_main < 0 || k_main > K || k_main % 32) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (rows == 0) return TLF_OK;
  if (!x || !w || !y) return TLF_E_NULL;
  if (!aligned16(x) || !aligned16(w) || !aligned16(y)) return TLF_E_ALIGN;
  const HeadGemmArgs a{x, w, y, rows, heads, N, K, n_main, k_main};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == TLF_DT_BF16) {
    if ((rows + 63) / 64 > 65535) return TLF_E_SHAPE;
    TLF_LAUNCH(head_gemm_kernel, dim3(heads, (rows + 63) / 64, (N + 63) / 64), dim3(256), 0, s, a);
  } else {
    const int64_t total = static_cast<int64_t>(rows) * heads * N;
    if ((total + 255) / 256 > 0x7fffffff) return TLF_E_SHAPE;
    TLF_LAUNCH(head_gemm_f32_kernel, dim3(static_cast<unsigned>((total + 255) / 256)), dim3(256), 0, s, a);
  }
  return launch_status();
}

extern "C" int tlf_latent_rows(const void *q, const void *cache, const int32_t *block_tables, int64_t bt_stride,
                               const int64_t *positions, const int32_t *slot_mapping, const int32_t *row_seq, float *part,
                               float *ml, int32_t rows, int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank,
                               int32_t vdim, int32_t block_size, int32_t window, int64_t num_pages, float scale,
                               int32_t dtype, void *stream) {
  using namespace tlf;
  LatentRowsArgs a{};
  if (rows < 0 || rows > 65535 || window <= 0 || !latent_shape(a.s, heads, dim, rot_dim, rank, vdim)) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (rows == 0) return TLF_OK;
  a.c = LatentCache{cache, block_tables, bt_stride, num_pages, block_size, -1};
  if (int rc = latent_cache_check(a.c)) return rc;
  if (!q || !positions || !slot_mapping || !part || !ml) return TLF_E_NULL;
  a.q = q; a.positions = positions; a.slots = slot_mapping; a.row_seq = row_seq; a.part = part; a.ml = ml; a.window = window;
  a.scale_log2 = scale * 1.4426950408889634f;
  const dim3 grid(heads, rows);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define TLF_LROWS(T)                                                                                  \
  do {                                                                                                \
    if (a.s.Lp <= 128) TLF_LAUNCH((latent_rows_kernel<T, 2>), grid, dim3(256), 0, s, a);              \
    else if (a.s.Lp <= 256) TLF_LAUNCH((latent_rows_kernel<T, 4>), grid, dim3(256), 0, s, a);         \
    else if (a.s.Lp <= 640) TLF_LAUNCH((latent_rows_kernel<T, 10>), grid, dim3(256), 0, s, a);        \
    else TLF_LAUNCH((latent_rows_kernel<T, 32>), grid, dim3(256), 0, s, a);                           \
  } while (0)
  if (dtype == TLF_DT_BF16) TLF_LROWS(unsigned short);
  else TLF_LROWS(float);
#undef TLF_LROWS
  return launch_status();
}

extern "C" int tlf_latent_values(const float *part, const float *ml, const int32_t *plan, const int32_t *cu_seqlens_q,
                                 const int32_t *row_seq, int32_t first_seq, int32_t first_row, int32_t num_seqs,
                                 int32_t max_tokens, const void *uv, const float *gate, void *out, int64_t out_stride, int32_t rows, int32_t heads,
                                 int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim, int32_t dtype, void *stream) {
  using namespace tlf;
  LatentValuesArgs a{};
  if (rows < 0 || !latent_shape(a.s, heads, dim, rot_dim, rank, vdim)) return TLF_E_SHAPE;
  if (out_stride < static_cast<int64_t>(heads) * vdim) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (rows == 0) return TLF_OK;
  if (!part || !ml || !uv || !out || (plan && cu_seqlens_q && !row_seq)) return TLF_E_NULL;
  if (!aligned16(part) || !aligned16(uv)) return TLF_E_ALIGN;
  a.part = part; a.ml = ml; a.uv = uv; a.gate = gate; a.out = out; a.ldo = out_stride; a.rows = rows;
  a.Vp = round_up_to(vdim, 16);
  if (plan) {
    if (num_seqs <= 0 || max_tokens <= 0 || first_seq < 0 || (!cu_seqlens_q && rows > num_seqs)) return TLF_E_SHAPE;
    a.plan = plan; a.row_seq = row_seq;
    a.jb = LatentJobs{nullptr, nullptr, cu_seqlens_q, nullptr, first_seq, first_row, 1};
    if (!latent_jobs(a.jb, num_seqs, max_tokens, heads)) return TLF_E_TOO_LARGE;
    a.wgs = latent_workgroups(a.s.Lp, a.jb.units);
  }
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == TLF_DT_BF16) {
    if ((rows + 15) / 16 > 65535) return TLF_E_SHAPE;
    TLF_LAUNCH(latent_values_kernel, dim3(heads, (rows + 15) / 16, (a.Vp + 63) / 64), dim3(256), 16 * (a.s.Rp + 8) * 2, s, a);
  } else {
    if (rows > 65535) return TLF_E_SHAPE;
    TLF_LAUNCH((latent_values_rows_kernel<float>), dim3(heads, rows), dim3(256), a.s.Rp * 4, s, a);
  }
  return launch_status();
}

extern "C" int tlf_latent_gather(const void *cache, const int32_t *block_tables, int64_t bt_stride, const int32_t *cu_seqlens_q,
                                 const int32_t *seq_starts, const int32_t *kv_offsets, int32_t first_seq, int32_t num_seqs,
                                 int32_t max_rows, void *out, int32_t row_size, int32_t block_size, int32_t window,
                                 int64_t num_pages, void *stream) {
  using namespace tlf;
  if (num_seqs < 0 || num_seqs > 65535 || max_rows < 0 || first_seq < 0 || row_size <= 0 || row_size % 64 || window <= 0) return TLF_E_SHAPE;
  if (num_seqs == 0 || max_rows == 0) return TLF_OK;
  LatentCache c{cache, block_tables, bt_stride, num_pages, block_size, -1};
  if (int rc = latent_cache_check(c)) return rc;
  if (!cu_seqlens_q || !seq_starts || !kv_offsets || !out) return TLF_E_NULL;
  if (!aligned16(out)) return TLF_E_ALIGN;
  const int64_t items = static_cast<int64_t>(max_rows) * (row_size / 8);
  TLF_LAUNCH(latent_gather_kernel, dim3(static_cast<unsigned>((items + 255) / 256), num_seqs), dim3(256), 0,
             static_cast<hipStream_t>(stream), c, cu_seqlens_q, seq_starts, kv_offsets, first_seq, window, row_size,
             static_cast<unsigned short *>(out));
  return launch_status();
}
