// Absorbed latent attention on the matrix cores, bf16: decoded tokens and short portions (geometry in latent_attn.h).
//
// The (row, head) pairs of a sequence are flattened into units; a workgroup owns 16 CT units and a range of the key tiles
// their window covers.  All units share the cache rows, so 64 of them are staged in LDS once and serve as keys and as
// values; 4 CT waves split the work by keys in the first product and by latent dimensions in the second, and each row is
// read from LDS once per product:
//   S^T[key, unit] = C . Q^T      wave (kt, ct): 16 keys, 16 units       v_mfma_f32_16x16x32_bf16
//   softmax weights               running maximum per unit, shared between the waves through LDS; weights as bf16 hi + lo
//   O^T[dim, unit] += C^T . P^T   wave w: dimension tiles w, w + 4 CT, ...; C^T by LDS transpose reads
// Rows travel global -> registers -> LDS one tile ahead, two LDS tiles.  A workgroup writes its unnormalised mix of latents
// with the maximum and the denominator; latent_values_kernel joins the splits.
#include <algorithm>

#include "latent_attn.h"

namespace tlf {

constexpr int kLK = 64;   // keys per tile

struct LatentTileArgs {
  LatentShape s;
  LatentCache c;
  const unsigned short *q;     // [rows, H, Lp]
  const int64_t *positions;    // one row per sequence (cu_q NULL): its position
  const int32_t *slots;        // likewise; negative: padding row
  const int32_t *cu_q, *starts;
  float *part, *ml;
  int32_t rows;                // rows of part / ml in all
  int32_t hpp, passes, bq;     // heads per workgroup, passes over the heads, rows per workgroup
  int32_t xtiles, splits, first_seq, first_row, window;
  float scale_log2;
};

__device__ __forceinline__ shortx4 latent_read_tr16(const unsigned short *p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p));
}

// NC = Lp / 64
template <int NC, int CT>
__global__ __launch_bounds__(256 * CT) void latent_tile_kernel(const LatentTileArgs a) {
  constexpr int LP = NC * 64, KS = NC * 2, W = 4 * CT, T = 256 * CT;
  constexpr int NL = kLK * (LP / 8) / T;                 // 16-byte pieces a thread copies per tile
  constexpr int MT = (LP / 16 + W - 1) / W;              // dimension tiles per wave, at most
  __shared__ __attribute__((aligned(16))) unsigned short Cs[2][kLK][LP + 8];
  __shared__ __attribute__((aligned(16))) unsigned short Ph[CT * 16][kLK + 8], Pl[CT * 16][kLK + 8];
  __shared__ float mpart[CT][4][16];
  const LatentShape &s = a.s;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int kt = wave & 3, ct = wave >> 2;
  const int split = blockIdx.x, pass = blockIdx.y % a.passes, xt = blockIdx.y / a.passes, sq = blockIdx.z;
  const int seq = a.first_seq + sq;
  int q0, lq, start;
  if (a.cu_q) {
    q0 = a.cu_q[seq] - a.first_row;
    lq = a.cu_q[seq + 1] - a.cu_q[seq];
    start = a.starts[seq];
  } else {
    q0 = seq;
    lq = 1;
    start = a.slots[seq] >= 0 ? static_cast<int>(a.positions[seq]) : -1;
  }
  const int row0 = xt * a.bq;
  if (row0 >= lq) return;
  const bool live = start >= 0;
  const int nh = min(a.hpp, s.H - pass * a.hpp), last_row = min(row0 + a.bq, lq) - 1;
  const int i_first = start + row0, i_last = start + last_row;

  // this lane's unit of every column tile
  int upos[CT];
  int64_t urh[CT];
  bool uok[CT];
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const int u = k * 16 + n, r = row0 + u / a.hpp, hh = u % a.hpp;
    uok[k] = u < a.bq * a.hpp && r <= last_row && hh < nh;
    const int row = uok[k] ? r : row0;
    upos[k] = start + row;
    urh[k] = static_cast<int64_t>(q0 + row) * s.H + pass * a.hpp + (uok[k] ? hh : 0);
  }
  bf16x8 qf[KS];
  {
    const unsigned short *qp = a.q + (CT == 1 || ct == 0 ? urh[0] : urh[CT - 1]) * LP + g * 8;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      Pack16 t;
      t.u = *reinterpret_cast<const uint4 *>(qp + k * 32);
      qf[k] = t.v;
    }
  }
  const int my_pos = ct == 0 ? upos[0] : upos[CT - 1];

  const int w0 = max(0, i_first - a.window + 1) / kLK * kLK;
  const int tiles_all = live ? (i_last - w0) / kLK + 1 : 0;
  const int per = (tiles_all + a.splits - 1) / a.splits;
  const int t0 = split * per, t1 = min(tiles_all, t0 + per);
  const int32_t *bt = a.c.bt + seq * a.c.bt_stride;
  const unsigned short *rows = static_cast<const unsigned short *>(a.c.rows);

  uint4 reg[NL];
  auto tile_base = [&](int t) __attribute__((always_inline)) { return latent_row(a.c, bt, w0 + min(t, t1 - 1) * kLK) * LP; };
  auto load_tile = [&](int64_t base) __attribute__((always_inline)) {   // 64 tokens from a multiple of 64 on lie in one page
#pragma unroll
    for (int i = 0; i < NL; ++i) reg[i] = *reinterpret_cast<const uint4 *>(rows + base + (tid + i * T) * 8);
  };
  auto store_tile = [&](int b) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int item = tid + i * T, r = item / (LP / 8), ch = item % (LP / 8);
      *reinterpret_cast<uint4 *>(&Cs[b][r][ch * 8]) = reg[i];
    }
  };

  floatx4 acc[MT][CT];
#pragma unroll
  for (int d = 0; d < MT; ++d)
#pragma unroll
    for (int k = 0; k < CT; ++k) acc[d][k] = floatx4{0.f, 0.f, 0.f, 0.f};
  float m[CT], l = 0.f;   // l: this wave's keys, this lane's unit of column tile ct
#pragma unroll
  for (int k = 0; k < CT; ++k) m[k] = -INFINITY;
  const int dtiles = (s.Ra + 15) / 16;

  if (t0 < t1) {
    load_tile(tile_base(t0));
    store_tile(0);
    load_tile(tile_base(t0 + 1));
    int64_t next = tile_base(t0 + 2);
    lds_barrier();
    for (int t = t0; t < t1; ++t) {
      const int b = (t - t0) & 1;
      const unsigned short(*C)[LP + 8] = Cs[b];
      floatx4 sc = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        Pack16 c;
        c.u = *reinterpret_cast<const uint4 *>(&C[kt * 16 + n][k * 32 + g * 8]);
        sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c.v, qf[k], sc, 0, 0, 0);
      }
      // lane (n, g): keys key .. key + 3 of unit n
      const int key = w0 + t * kLK + kt * 16 + g * 4;
      float p[4];
#pragma unroll
      for (int j = 0; j < 4; ++j)
        p[j] = key + j <= my_pos && key + j > my_pos - a.window ? sc[j] * a.scale_log2 : -INFINITY;
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
      store_tile(b ^ 1);            // read last before the previous barrier
      load_tile(next);
      next = tile_base(t + 3);
      lds_barrier();
#pragma unroll
      for (int d = 0; d < MT; ++d)
#pragma unroll
        for (int k = 0; k < CT; ++k) acc[d][k] *= back[k];
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
        const int vt = hf * 32 + g * 8 + (n >> 2);
#pragma unroll
        for (int d = 0; d < MT; ++d) {
          const int dt = d * W + wave;
          if (dt < dtiles) {   // wave uniform
            const shortx4 v0 = latent_read_tr16(&C[vt][dt * 16 + (n & 3) * 4]);
            const shortx4 v1 = latent_read_tr16(&C[vt + 4][dt * 16 + (n & 3) * 4]);
            const uint2 a0 = __builtin_bit_cast(uint2, v0), a1 = __builtin_bit_cast(uint2, v1);
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
  }

  l = sum_lanes_16_32_48(l);
  lds_barrier();
  if (g == 0) mpart[ct][kt][n] = l;
  lds_barrier();
  const int64_t plane = static_cast<int64_t>(a.rows) * s.H;
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    if (!uok[k]) continue;
    const int64_t at = split * plane + urh[k];
    if (wave == 0 && g == 0) {
      a.ml[at * 2] = m[k];
      a.ml[at * 2 + 1] = mpart[k][0][n] + mpart[k][1][n] + mpart[k][2][n] + mpart[k][3][n];
    }
    if (t0 < t1) {
#pragma unroll
      for (int d = 0; d < MT; ++d) {
        const int col = (d * W + wave) * 16 + g * 4;
        if (col < s.Rp)
          *reinterpret_cast<float4 *>(a.part + at * s.Rp + col) =
              col < s.Ra ? make_float4(acc[d][k][0], acc[d][k][1], acc[d][k][2], acc[d][k][3]) : make_float4(0.f, 0.f, 0.f, 0.f);
      }
    }
  }
}

// Splits of the keys: about one workgroup per CU, at least two tiles each.
inline int latent_splits(int64_t groups, int64_t max_keys) {
  const int64_t tiles = (max_keys + kLK - 1) / kLK + 1;
  const int64_t want = (256 + groups / 2) / groups;
  return static_cast<int>(std::max<int64_t>(1, std::min<int64_t>({want, (tiles + 1) / 2, 32})));
}
inline int latent_ct(int units) { return units > 16 ? 2 : 1; }

}  // namespace tlf

extern "C" int tlf_latent_attn_splits(int32_t num_seqs, int32_t max_tokens, int32_t heads, int32_t window, int32_t max_len) {
  using namespace tlf;
  if (num_seqs <= 0 || max_tokens <= 0 || heads <= 0 || window <= 0 || max_len <= 0) return 1;
  const int64_t units = static_cast<int64_t>(max_tokens) * heads;
  const int u = 16 * latent_ct(static_cast<int>(std::min<int64_t>(units, 64)));
  return latent_splits(num_seqs * ((units + u - 1) / u), std::min<int64_t>(static_cast<int64_t>(window) + max_tokens, max_len));
}

extern "C" int tlf_latent_attn_supported(int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim) {
  tlf::LatentShape s;
  return tlf::latent_shape(s, heads, dim, rot_dim, rank, vdim) && s.Lp <= 576;
}

extern "C" int tlf_latent_attn(const void *q, const void *cache, const int32_t *block_tables, int64_t bt_stride,
                               const int64_t *positions, const int32_t *slot_mapping, const int32_t *cu_seqlens_q,
                               const int32_t *seq_starts, int32_t first_seq, int32_t first_row, int32_t num_seqs,
                               int32_t max_tokens, float *part, float *ml, int32_t splits, int32_t rows, int32_t heads, int32_t dim,
                               int32_t rot_dim, int32_t rank, int32_t vdim, int32_t block_size, int32_t window,
                               int64_t num_pages, float scale, void *stream) {
  using namespace tlf;
  LatentTileArgs a{};
  if (num_seqs < 0 || num_seqs > 65535 || max_tokens < 0 || first_seq < 0 || rows < 0 || window <= 0 || splits <= 0 || splits > 32) return TLF_E_SHAPE;
  if (!latent_shape(a.s, heads, dim, rot_dim, rank, vdim)) return TLF_E_SHAPE;
  if (a.s.Lp > 576) return TLF_E_UNSUPPORTED;   // two tiles of longer rows do not fit LDS
  if (num_seqs == 0 || max_tokens == 0) return TLF_OK;
  a.c = LatentCache{cache, block_tables, bt_stride, num_pages, block_size, -1};
  if (int rc = latent_cache_check(a.c)) return rc;
  if (!q || !part || !ml || (cu_seqlens_q ? !seq_starts : (!positions || !slot_mapping))) return TLF_E_NULL;
  if (!cu_seqlens_q && max_tokens != 1) return TLF_E_SHAPE;
  if (!aligned16(q) || !aligned16(part)) return TLF_E_ALIGN;
  a.q = static_cast<const unsigned short *>(q); a.positions = positions; a.slots = slot_mapping; a.cu_q = cu_seqlens_q;
  a.starts = seq_starts; a.part = part; a.ml = ml; a.rows = rows; a.splits = splits; a.first_seq = first_seq; a.first_row = first_row;
  a.window = window; a.scale_log2 = scale * 1.4426950408889634f;
  const int64_t units = static_cast<int64_t>(max_tokens) * heads;
  const int ct = latent_ct(static_cast<int>(std::min<int64_t>(units, 64))), u = 16 * ct;
  a.hpp = std::min(heads, u);
  a.passes = (heads + a.hpp - 1) / a.hpp;
  a.bq = u / a.hpp;
  a.xtiles = (max_tokens + a.bq - 1) / a.bq;
  if (static_cast<int64_t>(a.passes) * a.xtiles > 65535) return TLF_E_SHAPE;
  const dim3 grid(splits, a.passes * a.xtiles, num_seqs);
  hipStream_t st = static_cast<hipStream_t>(stream);
#define TLF_LT(NC)                                                                                  \
  case NC:                                                                                          \
    if (ct == 1) TLF_LAUNCH((latent_tile_kernel<NC, 1>), grid, dim3(256), 0, st, a);                \
    else TLF_LAUNCH((latent_tile_kernel<NC, 2>), grid, dim3(512), 0, st, a);                        \
    break;
  switch (a.s.Lp / 64) {
    TLF_LT(1) TLF_LT(2) TLF_LT(3) TLF_LT(4) TLF_LT(5) TLF_LT(6) TLF_LT(7) TLF_LT(8) TLF_LT(9)
#undef TLF_LT
    default: return TLF_E_UNSUPPORTED;
  }
  return launch_status();
}
