// Absorbed latent attention on the matrix cores, bf16: decoded tokens and short portions (geometry in latent_attn.h).
//
// The (row, head) pairs of a sequence are flattened into units; 16 CT units make a job, whose work is the 64-key tiles that
// its window covers.  Jobs are cut into pieces of about equal length, one per workgroup, by a plan made once per step and
// window: as short as the workgroups that the chip holds at once allow, so that sequences of unequal length keep all CUs busy
// alike.
//
// All units share the cache rows, so a tile in LDS serves as keys and as values; 4 CT waves split the work by keys in the
// first product and by latent dimensions in the second, and each row is read from LDS once per product:
//   S^T[key, unit] = C . Q^T      wave (kt, ct): 16 keys, 16 units       v_mfma_f32_16x16x32_bf16
//   softmax weights               running maximum per unit, shared between the waves through LDS; weights as bf16 hi + lo
//   O^T[dim, unit] += C^T . P^T   wave w: dimension tiles w, w + 4 CT, ...; C^T by LDS transpose reads
// Tiles travel global -> LDS directly into a ring of stages.  64 rows from a multiple of 64 on are contiguous in a page, so
// a copy instruction moves 1 KiB; LDS rows are unpadded and their 16-byte pieces are swizzled against bank conflicts (the
// lane that fills a position picks the matching global piece).  A workgroup writes its unnormalised mix of latents with
// the maximum and the denominator; latent_values_kernel (latent_attn.hip) joins the pieces.
#include <algorithm>

#include "gemm_shared.h"
#include "latent_attn.h"

namespace tlf {

__device__ __forceinline__ shortx4 latent_read_tr16(const unsigned short *p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p));
}

// One workgroup: the length of a piece, the pieces' records, which pieces a job has.
__global__ __launch_bounds__(1024) void latent_plan_kernel(const LatentJobs jb, int32_t *plan, int32_t wgs) {
  constexpr int kKept = 4096;                 // jobs whose tile counts are kept
  __shared__ int tiles[kKept], part[16], most[16], busy[16], per_shared;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  int sum = 0, mx = 0, some = 0;
  for (int j = tid; j < jb.jobs; j += 1024) {
    const int t = latent_job<false>(jb, j).tiles;
    if (j < kKept) tiles[j] = t;
    sum += t;
    mx = max(mx, t);
    some += t > 0;
  }
  for (int o = 32; o > 0; o >>= 1) {
    sum += __shfl_xor(sum, o, 64);
    some += __shfl_xor(some, o, 64);
    mx = max(mx, __shfl_xor(mx, o, 64));
  }
  if (lane == 0) { part[wave] = sum; most[wave] = mx; busy[wave] = some; }
  __syncthreads();
  int total = 0, longest = 0, live = 0;
  for (int w = 0; w < 16; ++w) { total += part[w]; longest = max(longest, most[w]); live += busy[w]; }
  // not shorter than `least`: more pieces than workgroups, or than a job may have; `safe` needs no look at the jobs
  const int least = max(1, max((total + wgs - 1) / wgs, (longest + kLatentMaxPieces - 1) / kLatentMaxPieces));
  const int safe = live < wgs ? max(least, (total + wgs - live - 1) / (wgs - live)) : least;
  if (tid == 0) per_shared = safe;
  __syncthreads();
  if (safe > least && jb.jobs <= kKept) {
    // 16 lengths between the two, a wave each: the shortest whose pieces fit the workgroups
    const int per = least + (safe - least) * wave / 16;
    int pieces = 0;
    for (int j = lane; j < jb.jobs; j += 64) pieces += (tiles[j] + per - 1) / per;
    for (int o = 32; o > 0; o >>= 1) pieces += __shfl_xor(pieces, o, 64);
    if (lane == 0 && pieces <= wgs) atomicMin(&per_shared, per);
    __syncthreads();
  }
  const int per = per_shared;
  int before = 0;
  for (int j0 = 0; j0 < jb.jobs; j0 += 1024) {
    const int j = j0 + tid;
    LatentJob job;
    job.tiles = 0;
    if (j < jb.jobs) job = latent_job<false>(jb, j);
    const int n = (job.tiles + per - 1) / per;
    int x = n;
    for (int o = 1; o < 64; o <<= 1) {
      const int y = __shfl_up(x, o, 64);
      if (lane >= o) x += y;
    }
    __syncthreads();
    if (lane == 63) part[wave] = x;
    __syncthreads();
    int a = before + x - n;
    for (int w = 0; w < 16; ++w) {
      if (w < wave) a += part[w];
      before += part[w];
    }
    if (j < jb.jobs) {
      int32_t *rec = plan + latent_plan_jobs(wgs, jb.jobs) + 2 * j;
      rec[0] = a;
      rec[1] = n;
      for (int k = 0; k < n; ++k)
        *reinterpret_cast<int4 *>(plan + kLatentPlanHead + kLatentRecord * (a + k)) =
            make_int4(min(per, job.tiles - k * per), j, k * per, job.start);
    }
  }
  if (tid == 0) { plan[0] = per; plan[1] = before; }
  for (int w = before + tid; w < latent_max_pieces(wgs, jb.jobs); w += 1024) plan[kLatentPlanHead + kLatentRecord * w] = 0;
}

struct LatentTileArgs {
  LatentShape s;
  LatentJobs jb;
  const unsigned short *rows;  // [pages, bs, Lp]
  const int32_t *bt;
  int64_t bt_stride, pages;
  int32_t bs, bs_shift;
  const unsigned short *q;     // [rows, H, Lp]
  const int32_t *plan;
  float *part, *ml;            // [pieces, 16 CT, Rp], [.., 2]
  float scale_log2;
};

// NC = Lp / 64, NS = LDS stages
template <int NC, int CT, int NS>
__global__ __launch_bounds__(256 * CT) void latent_tile_kernel(const LatentTileArgs a) {
  constexpr int LP = NC * 64, KS = NC * 2, W = 4 * CT, U = 16 * CT;
  constexpr int NL = NC * 8 / W;                         // copies of 1 KiB per wave and tile
  constexpr int MT = (NC * 4 + W - 1) / W;               // dimension tiles per wave
  constexpr int PIECES = LP / 8, SWZ = NC % 2 ? 7 : 15;  // 16-byte pieces per row, swizzled bits
  __shared__ __attribute__((aligned(1024))) unsigned short pool[NS][kLatentTile * LP];
  __shared__ __attribute__((aligned(16))) unsigned short Ph[U][kLatentTile + 8], Pl[U][kLatentTile + 8];
  __shared__ float mpart[CT][4][16];
  const LatentShape &s = a.s;
  const int tid = threadIdx.x, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), kt = wave & 3, ct = wave >> 2;
  const int w = blockIdx.x;
  const int32_t *rec = a.plan + kLatentPlanHead + kLatentRecord * w;
  const int count = uniform_load(rec), job = uniform_load(rec + 1), tile0 = uniform_load(rec + 2), start = uniform_load(rec + 3);
  if (count <= 0 || job < 0 || job >= a.jb.jobs) return;
  const LatentJob J = latent_job<true>(a.jb, job, start);
  if (tile0 < 0 || count > J.tiles - tile0) return;      // not a plan
  // row R: an odd row begins 32 banks in if NC is odd, so 8 positions and the parity tell 16 rows apart, otherwise 16 positions
  auto swz = [](int row) __attribute__((always_inline)) { return NC % 2 ? (row >> 1) & 7 : row & 15; };

  unsigned int voff[NL];
#pragma unroll
  for (int i = 0; i < NL; ++i) {
    const int slot = (i * W + wave) * 64 + lane, row = slot / PIECES, pos = slot % PIECES;
    voff[i] = static_cast<unsigned int>((row * PIECES + (pos ^ (swz(row) & SWZ))) * 16);
  }
  const unsigned int lds0 = TLF_DL_LDSADDR(&pool[0][0]) + wave * 1024;

  // copy side: NS - 1 tiles ahead; the page of the tile to come is looked up one tile early
  const int32_t *bt = a.bt + J.seq * a.bt_stride;
  auto page_at = [&](int tile) __attribute__((always_inline)) {
    const int at = J.w0 + (tile0 + min(tile, count - 1)) * kLatentTile;
    return uniform_load(bt + (a.bs_shift >= 0 ? at >> a.bs_shift : at / a.bs));
  };
  int page = page_at(0);
  auto issue = [&](int tile, int stage) __attribute__((always_inline)) {
    const int at = J.w0 + (tile0 + tile) * kLatentTile;
    const int within = a.bs_shift >= 0 ? at & (a.bs - 1) : at % a.bs;
    const int64_t row = page >= 0 && page < a.pages ? static_cast<int64_t>(page) * a.bs + within : 0;
    const unsigned char *base = reinterpret_cast<const unsigned char *>(a.rows + row * LP);
    const unsigned int lds = lds0 + stage * (kLatentTile * LP * 2);
#pragma unroll
    for (int i = 0; i < NL; ++i) TLF_DL_COPY(voff[i], base, lds + i * (W * 1024));
    page = page_at(tile + 1);
  };
#pragma unroll
  for (int i = 0; i < NS - 1; ++i)
    if (i < count) issue(i, i);

  int upos[CT];
  bf16x8 qf[KS];
  floatx4 acc[MT][CT];
  float m[CT], l;      // l: this wave's keys, this lane's unit of column tile ct
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const int u = k * 16 + n, r = J.row0 + u / a.jb.hpp;
    const bool ok = u < a.jb.bq * a.jb.hpp && r <= J.last_row && u % a.jb.hpp < J.heads;
    upos[k] = J.start + (ok ? r : J.row0);
    m[k] = -INFINITY;
    if (k == ct || CT == 1) {
      const unsigned short *qp = a.q + (static_cast<int64_t>(J.q0 + (ok ? r : J.row0)) * s.H + J.head0 + (ok ? u % a.jb.hpp : 0)) * LP + g * 8;
#pragma unroll
      for (int i = 0; i < KS; ++i) {
        Pack16 x;
        x.u = *reinterpret_cast<const uint4 *>(qp + i * 32);
        qf[i] = x.v;
      }
    }
  }
  // the loads end here: a wait inside the loop would be one for the copies, too
#pragma unroll
  for (int i = 0; i < KS; ++i) asm volatile("" : "+v"(qf[i]));
  l = 0.f;
#pragma unroll
  for (int d = 0; d < MT; ++d)
#pragma unroll
    for (int k = 0; k < CT; ++k) acc[d][k] = floatx4{0.f, 0.f, 0.f, 0.f};

  int cur = 0;
  for (int i = 0; i < count; ++i) {
    // the tile is there, for all waves, and nobody reads the stage before it any more
    if (i + NS - 1 < count) {
      TLF_DL_BARRIER((NS - 2) * NL);
      issue(i + NS - 1, cur == 0 ? NS - 1 : cur - 1);
    } else {
      TLF_DL_BARRIER(0);
    }
    const unsigned short *C = pool[cur];
    cur = cur + 1 == NS ? 0 : cur + 1;
    floatx4 sc = floatx4{0.f, 0.f, 0.f, 0.f};
    {
      const int row = kt * 16 + n, f = swz(row) & SWZ;
      const unsigned short *cr = C + row * LP;
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        Pack16 c;
        c.u = *reinterpret_cast<const uint4 *>(cr + ((k * 4 + g) ^ f) * 8);
        sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c.v, qf[k], sc, 0, 0, 0);
      }
    }
    // lane (n, g): keys key .. key + 3 of unit n
    const int key = J.w0 + (tile0 + i) * kLatentTile + kt * 16 + g * 4;
    const int my_pos = ct == 0 ? upos[0] : upos[CT - 1];
    float p[4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      p[j] = key + j <= my_pos && key + j > my_pos - a.jb.window ? sc[j] * a.scale_log2 : -INFINITY;
    const float mloc = max_lanes_16_32_48(fmaxf(fmaxf(p[0], p[1]), fmaxf(p[2], p[3])));
    if (g == 0) mpart[ct][kt][n] = mloc;
    lds_barrier();
    float back[CT];
#pragma unroll
    for (int k = 0; k < CT; ++k) {
      const float mn = fmaxf(fmaxf(fmaxf(mpart[k][0][n], mpart[k][1][n]), fmaxf(mpart[k][2][n], mpart[k][3][n])), m[k]);
      back[k] = mn == m[k] ? 1.f : __builtin_amdgcn_exp2f(m[k] - mn);
      m[k] = mn;
    }
    const float mc = ct == 0 ? m[0] : m[CT - 1];
    float sum = 0.f;
    unsigned int h[2], lo[2];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      p[j] = p[j] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(p[j] - mc);
      sum += p[j];
    }
    l = fmaf(l, ct == 0 ? back[0] : back[CT - 1], sum);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      h[j] = pack_bf16x2(p[2 * j], p[2 * j + 1]);
      lo[j] = pack_bf16x2(p[2 * j] - __uint_as_float(h[j] << 16), p[2 * j + 1] - __uint_as_float(h[j] & 0xffff0000u));
    }
    *reinterpret_cast<uint2 *>(&Ph[ct * 16 + n][kt * 16 + g * 4]) = make_uint2(h[0], h[1]);
    *reinterpret_cast<uint2 *>(&Pl[ct * 16 + n][kt * 16 + g * 4]) = make_uint2(lo[0], lo[1]);
#pragma unroll
    for (int d = 0; d < MT; ++d)
#pragma unroll
      for (int k = 0; k < CT; ++k) acc[d][k] *= back[k];
    lds_barrier();
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      bf16x8 ph[CT], pl[CT];
#pragma unroll
      for (int k = 0; k < CT; ++k) {
        Pack16 x, y;
        x.u = *reinterpret_cast<const uint4 *>(&Ph[k * 16 + n][hf * 32 + g * 8]);
        y.u = *reinterpret_cast<const uint4 *>(&Pl[k * 16 + n][hf * 32 + g * 8]);
        ph[k] = x.v;
        pl[k] = y.v;
      }
      const int v0 = hf * 32 + g * 8 + (n >> 2), v1 = v0 + 4;
      const int f0 = swz(v0) & SWZ, f1 = swz(v1) & SWZ, sub = (n & 3) >> 1, byte = (n & 1) * 4;
#pragma unroll
      for (int d = 0; d < MT; ++d) {
        const int dt = d * W + wave;
        if ((d + 1) * W <= NC * 4 || dt < NC * 4) {   // wave uniform; only the last may be false
          const uint2 a0 = __builtin_bit_cast(uint2, latent_read_tr16(C + v0 * LP + ((dt * 2 + sub) ^ f0) * 8 + byte));
          const uint2 a1 = __builtin_bit_cast(uint2, latent_read_tr16(C + v1 * LP + ((dt * 2 + sub) ^ f1) * 8 + byte));
          const bf16x8 cv = __builtin_bit_cast(bf16x8, make_uint4(a0.x, a0.y, a1.x, a1.y));
#pragma unroll
          for (int k = 0; k < CT; ++k) {
            acc[d][k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cv, ph[k], acc[d][k], 0, 0, 0);
            acc[d][k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cv, pl[k], acc[d][k], 0, 0, 0);
          }
        }
      }
    }
  }
  l = sum_lanes_16_32_48(l);
  if (g == 0) mpart[ct][kt][n] = l;                      // read last before the barrier in front of the second product
  lds_barrier();
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const int64_t at = static_cast<int64_t>(w) * U + k * 16 + n;
    if (wave == 0 && g == 0) {
      a.ml[at * 2] = m[k];
      a.ml[at * 2 + 1] = mpart[k][0][n] + mpart[k][1][n] + mpart[k][2][n] + mpart[k][3][n];
    }
#pragma unroll
    for (int d = 0; d < MT; ++d) {
      const int col = (d * W + wave) * 16 + g * 4;
      if (col < s.Rp)
        *reinterpret_cast<float4 *>(a.part + at * s.Rp + col) =
            col < s.Ra ? make_float4(acc[d][k][0], acc[d][k][1], acc[d][k][2], acc[d][k][3]) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
  }
}

}  // namespace tlf

extern "C" int tlf_latent_attn_supported(int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim) {
  tlf::LatentShape s;
  return tlf::latent_shape(s, heads, dim, rot_dim, rank, vdim) && s.Lp <= 576;   // two tiles of longer rows do not fit LDS
}

extern "C" int tlf_latent_attn_layout(int32_t num_seqs, int32_t max_tokens, int32_t heads, int32_t row_size, int32_t *layout) {
  using namespace tlf;
  if (num_seqs < 0 || max_tokens <= 0 || heads <= 0 || row_size <= 0 || row_size % 64) return TLF_E_SHAPE;
  if (!layout) return TLF_E_NULL;
  LatentJobs jb{};
  if (!latent_jobs(jb, num_seqs, max_tokens, heads)) return TLF_E_TOO_LARGE;
  const int wgs = latent_workgroups(row_size, jb.units);
  layout[0] = static_cast<int32_t>(latent_plan_jobs(wgs, jb.jobs)) + 2 * jb.jobs;   // plan, in int32
  layout[1] = latent_max_pieces(wgs, jb.jobs);         // pieces
  layout[2] = jb.units;                                // units of a piece
  return TLF_OK;
}

extern "C" int tlf_latent_attn_plan(const int64_t *positions, const int32_t *slot_mapping, const int32_t *cu_seqlens_q,
                                    const int32_t *seq_starts, int32_t first_seq, int32_t first_row, int32_t num_seqs,
                                    int32_t max_tokens, int32_t heads, int32_t row_size, int32_t window, int32_t *plan,
                                    void *stream) {
  using namespace tlf;
  if (num_seqs < 0 || max_tokens <= 0 || heads <= 0 || first_seq < 0 || window <= 0 || row_size <= 0 || row_size % 64) return TLF_E_SHAPE;
  if (num_seqs == 0) return TLF_OK;
  if (!plan || (cu_seqlens_q ? !seq_starts : (!positions || !slot_mapping))) return TLF_E_NULL;
  if (!aligned16(plan)) return TLF_E_ALIGN;
  if (!cu_seqlens_q && max_tokens != 1) return TLF_E_SHAPE;
  LatentJobs jb{positions, slot_mapping, cu_seqlens_q, seq_starts, first_seq, first_row, window};
  if (!latent_jobs(jb, num_seqs, max_tokens, heads)) return TLF_E_TOO_LARGE;
  TLF_LAUNCH(latent_plan_kernel, dim3(1), dim3(1024), 0, static_cast<hipStream_t>(stream), jb, plan, latent_workgroups(row_size, jb.units));
  return launch_status();
}

extern "C" int tlf_latent_attn(const void *q, const void *cache, const int32_t *block_tables, int64_t bt_stride,
                               const int64_t *positions, const int32_t *slot_mapping, const int32_t *cu_seqlens_q,
                               const int32_t *seq_starts, int32_t first_seq, int32_t first_row, int32_t num_seqs,
                               int32_t max_tokens, const int32_t *plan, float *part, float *ml, int32_t heads, int32_t dim,
                               int32_t rot_dim, int32_t rank, int32_t vdim, int32_t block_size, int32_t window,
                               int64_t num_pages, float scale, void *stream) {
  using namespace tlf;
  LatentTileArgs a{};
  if (num_seqs < 0 || max_tokens <= 0 || first_seq < 0 || window <= 0) return TLF_E_SHAPE;
  if (!latent_shape(a.s, heads, dim, rot_dim, rank, vdim)) return TLF_E_SHAPE;
  if (a.s.Lp > 576) return TLF_E_UNSUPPORTED;
  if (num_seqs == 0) return TLF_OK;
  LatentCache c{cache, block_tables, bt_stride, num_pages, block_size, -1};
  if (int rc = latent_cache_check(c)) return rc;
  if (!q || !part || !ml || !plan || (cu_seqlens_q ? !seq_starts : (!positions || !slot_mapping))) return TLF_E_NULL;
  if (!cu_seqlens_q && max_tokens != 1) return TLF_E_SHAPE;
  if (!aligned16(q) || !aligned16(part)) return TLF_E_ALIGN;
  a.jb = LatentJobs{positions, slot_mapping, cu_seqlens_q, seq_starts, first_seq, first_row, window};
  if (!latent_jobs(a.jb, num_seqs, max_tokens, heads)) return TLF_E_TOO_LARGE;
  a.rows = static_cast<const unsigned short *>(cache); a.bt = block_tables; a.bt_stride = bt_stride; a.pages = num_pages;
  a.bs = c.bs; a.bs_shift = c.bs_shift; a.q = static_cast<const unsigned short *>(q); a.plan = plan; a.part = part; a.ml = ml;
  a.scale_log2 = scale * 1.4426950408889634f;
  const dim3 grid(latent_max_pieces(latent_workgroups(a.s.Lp, a.jb.units), a.jb.jobs));
  hipStream_t st = static_cast<hipStream_t>(stream);
#define TLF_LT(NC, NS)                                                                                              \
  case NC:                                                                                                          \
    if (a.jb.units == 16) TLF_LAUNCH((latent_tile_kernel<NC, 1, NS>), grid, dim3(256), 0, st, a);                   \
    else TLF_LAUNCH((latent_tile_kernel<NC, 2, NS>), grid, dim3(512), 0, st, a);                                    \
    break;
  switch (a.s.Lp / 64) {
    TLF_LT(1, 4) TLF_LT(2, 4) TLF_LT(3, 3) TLF_LT(4, 4) TLF_LT(5, 3) TLF_LT(6, 3) TLF_LT(7, 2) TLF_LT(8, 2) TLF_LT(9, 2)
#undef TLF_LT
    default: return TLF_E_UNSUPPORTED;
  }
  return launch_status();
}
