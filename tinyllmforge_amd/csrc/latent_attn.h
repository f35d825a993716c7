// Geometry shared by the kernels of latent attention (latent_attn.hip, latent_decode.hip, latent_prefill.hip).
//
// Each token leaves one row in the paged cache for all heads: the normed latent c (`rank` values) and a rotated key part
// (`rot` values).  Head h scores it with  q_own . (Uk_h c) + q_rot . k_rot  and takes the value Uv_h c.  Two ways to run:
//   absorbed   q' = Uk_h^T q_own once per query; score = [q' | q_rot] . [c | k_rot]; the output is a mix of latents, and
//              Uv_h is applied to it once per query.  Every head reads the same cache row.
//   expanded   keys and values of every head are formed once per key by one matrix product (long prompt portions).
// All parts are padded with zeros so that each begins at a multiple of 8 elements:
//   cache row  [c: Ra | k_rot: Ta | 0]  Lp (a multiple of 64)      query row  [q_own: Da | q_rot: Ta | 0]  Dq (of 32)
#pragma once
#include "elem.h"

namespace tlf {

struct LatentShape {
  int32_t H, dim, rot, rank, vdim;
  int32_t Da, Ta, Ra, Va;   // own query / key part, rotated part, latent, value: rounded up to 8
  int32_t Dq, Lp, Rp;       // query row, cache row, row of mixed latents (a multiple of 32)
};
inline int round_up_to(int v, int m) { return (v + m - 1) / m * m; }
inline bool latent_shape(LatentShape &s, int H, int dim, int rot, int rank, int vdim) {
  if (H <= 0 || dim <= 0 || rot < 0 || rot % 2 || rank <= 0 || vdim <= 0) return false;
  if (H > 4096 || dim > 1024 || rot > 1024 || rank > 1536 || vdim > 1024) return false;
  s = LatentShape{H, dim, rot, rank, vdim, round_up_to(dim, 8), round_up_to(rot, 8), round_up_to(rank, 8), round_up_to(vdim, 8)};
  s.Dq = round_up_to(s.Da + s.Ta, 32);
  s.Lp = round_up_to(s.Ra + s.Ta, 64);
  s.Rp = round_up_to(s.Ra, 32);
  return s.Lp <= 2048;
}

struct LatentCache {
  const void *rows;         // [pages, bs, Lp]
  const int32_t *bt;        // block tables, one row per sequence
  int64_t bt_stride;
  int64_t pages;
  int32_t bs, bs_shift;     // log2 of bs, -1 if it is no power of two
};
inline int latent_cache_check(LatentCache &c) {
  if (c.bs <= 0 || c.bs % 64 || c.pages <= 0) return TLF_E_SHAPE;
  if (!c.rows || !c.bt) return TLF_E_NULL;
  c.bs_shift = (c.bs & (c.bs - 1)) == 0 ? __builtin_ctz(c.bs) : -1;
  return aligned16(c.rows) ? TLF_OK : TLF_E_ALIGN;
}
// Cache row of token j; an unmapped page reads row 0 (never visible).
__device__ __forceinline__ int64_t latent_row(const LatentCache &c, const int32_t *bt, int j) {
  const int pg = c.bs_shift >= 0 ? j >> c.bs_shift : j / c.bs;
  const int64_t page = bt[pg];
  return page >= 0 && page < c.pages ? page * c.bs + (j - pg * c.bs) : 0;
}

}  // namespace tlf
