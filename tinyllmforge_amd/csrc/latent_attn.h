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

// ---- jobs of the absorbed kernels: 16 or 32 units (row, head) of one sequence and the key tiles their window covers
constexpr int kLatentTile = 64;          // keys per tile
constexpr int kLatentMaxPieces = 128;    // pieces of a job, at most
// Plan: a head (tiles per piece, pieces), a record per piece (its tiles, job, first tile of it, start of the job's sequence:
// what a workgroup needs before its first copy) and per job (first piece, pieces).
constexpr int kLatentPlanHead = 4, kLatentRecord = 4;
// Pieces there may be: about one per workgroup the chip holds, and one more per job.
__host__ __device__ __forceinline__ int latent_max_pieces(int wgs, int jobs) { return wgs + jobs; }
__host__ __device__ __forceinline__ int64_t latent_plan_jobs(int wgs, int jobs) {
  return kLatentPlanHead + static_cast<int64_t>(kLatentRecord) * latent_max_pieces(wgs, jobs);
}

struct LatentJobs {
  const int64_t *positions;              // sequence s is the single row s at positions[s] (slots[s] < 0: no keys) ...
  const int32_t *slots;
  const int32_t *cu_q, *starts;          // ... or, with cu_q, rows cu_q[s] - first_row .. after starts[s] cached tokens
  int32_t first_seq, first_row, window;
  int32_t H, units, hpp, passes, bq, xtiles, jobs;   // heads, units of a job, heads per pass, passes, rows per job
};
inline bool latent_jobs(LatentJobs &j, int num_seqs, int max_tokens, int heads) {
  j.H = heads;
  j.units = static_cast<int64_t>(max_tokens) * heads > 16 ? 32 : 16;
  j.hpp = heads < j.units ? heads : j.units;
  j.passes = (heads + j.hpp - 1) / j.hpp;
  j.bq = j.units / j.hpp;
  j.xtiles = (max_tokens + j.bq - 1) / j.bq;
  const int64_t jobs = static_cast<int64_t>(num_seqs) * j.xtiles * j.passes;
  j.jobs = static_cast<int32_t>(jobs);
  return jobs <= (1 << 24);
}
// Workgroups of the tile kernel: as many as the chip holds at once.
inline int latent_workgroups(int lp, int units) { return 256 * (lp <= 128 ? 2 : 1); }

// Loads through the scalar path: the vector path's counter belongs to the copies in flight.
template <typename T>
__device__ __forceinline__ T uniform_load(const T *p) {
  return *(const T __attribute__((address_space(4))) *)(reinterpret_cast<uintptr_t>(p));
}

struct LatentJob {
  int seq, q0, start, row0, last_row, head0, heads, w0, tiles;
};
// UNIFORM: `job` is the same in all lanes.  known_start: the start of a single row's sequence if the caller has it (-1: a
// padding row)
template <bool UNIFORM>
__device__ __forceinline__ LatentJob latent_job(const LatentJobs &a, int job, int known_start = -2) {
  auto ld = [](auto *p) __attribute__((always_inline)) { return UNIFORM ? uniform_load(p) : *p; };
  LatentJob j;
  const int pass = job % a.passes, rest = job / a.passes, xt = rest % a.xtiles;
  j.seq = a.first_seq + rest / a.xtiles;
  int lq = 1;
  if (a.cu_q) {
    const int lo = ld(a.cu_q + j.seq);
    j.q0 = lo - a.first_row;
    lq = ld(a.cu_q + j.seq + 1) - lo;
    j.start = ld(a.starts + j.seq);
  } else {
    j.q0 = j.seq;
    j.start = known_start != -2 ? known_start : ld(a.slots + j.seq) >= 0 ? static_cast<int>(ld(a.positions + j.seq)) : -1;
  }
  j.row0 = xt * a.bq;
  j.last_row = min(j.row0 + a.bq, lq) - 1;
  j.head0 = pass * a.hpp;
  j.heads = min(a.hpp, a.H - j.head0);
  j.w0 = max(0, j.start + j.row0 - a.window + 1) / kLatentTile * kLatentTile;
  j.tiles = j.start >= 0 && j.row0 < lq ? (j.start + j.last_row - j.w0) / kLatentTile + 1 : 0;
  return j;
}

}  // namespace tlf
