// Attention of talk_attn.h for prompt portions, bf16, on the matrix cores, from the paged cache.  Mixing needs every head's
// weights, and weights need their denominators, so there are two kernels:
//
//   talk_stats_kernel    log2 of every (row, head)'s sum of exponentials: m + log2 l.  A workgroup owns one KV head and 64 CT units
//                        (row, head) of it and walks the keys 64 at a time through LDS; S^T[key, unit] = K . Q^T.
//   talk_prefill_kernel  a workgroup owns 16 RT query rows with all their heads, a wave 16 rows of four heads, or 32 rows of two, or 64
//                        of one (those that share a KV head), and walks the keys 32 at a time:
//     S^T[key, row] = K . Q^T per head, K straight from the caches in operand order, half a tile ahead;
//     W = 2^(S - m - log2 l), complete weights, as a bf16 hi + lo pair (16 significant bits) into LDS, [row][key][head];
//     per row (dealt to the waves) M^T[key, head] = W^T . talk^T, back into the row's place in LDS as a pair, [row][head][key];
//     O^T[dim, row] += V^T . M^T per head, V^T by LDS transpose reads of a tile that all waves share.
//
// Nothing is rescaled.  The rows of two 16-key tiles are picked so that their accumulators are eight consecutive keys.  V travels
// from the cache into LDS directly, behind the weights and the mix; rows are unpadded and pairs of their 16-byte pieces swizzled
// against bank conflicts (the lane that fills a position picks the matching piece).
#include "gemm_shared.h"
#include "talk_attn.h"

namespace tlf {

constexpr int kTK = 32;             // keys per tile
constexpr int kTM = kTK + 8;        // keys of a head's mixed weights, padded

struct TalkPrefillArgs {
  SinkCache c;
  const unsigned short *q;          // [rows, H, Dp]
  const unsigned short *talk;       // [H, H]
  float *stats;                     // [rows, H]
  const int32_t *cu_q, *starts;
  unsigned short *out;
  int64_t ldo;
  int32_t H, group;
  int32_t hpp, passes, bq;          // stats: query heads per pass, passes, rows per workgroup
  int32_t xtiles, total, first_seq, per_xcd, table_cols;
};

template <typename T>
__device__ __forceinline__ T talk_uniform(const T *p) {              // through the scalar path
  return *(const T __attribute__((address_space(4))) *)(reinterpret_cast<uintptr_t>(p));
}

constexpr int kTS = 64;             // keys per tile of the first kernel
__device__ __forceinline__ int talk_tile_row(int t) { return (t & 32) | ((t & 4) << 2) | ((t & 24) >> 1) | (t & 3); }

template <int DC, int CT>
__global__ __launch_bounds__(256) void talk_stats_kernel(const TalkPrefillArgs p) {
  constexpr int DP = DC * 32, KCH = DC * 4;
  __shared__ __attribute__((aligned(16))) unsigned short Ks[2][kTS][DP + 8];
  const int id = (blockIdx.x & 7) * p.per_xcd + (blockIdx.x >> 3);   // row tiles of one KV head share keys: the same XCD
  if (id >= p.total) return;
  const SinkCache &c = p.c;
  const int xt = p.xtiles - 1 - id % p.xtiles, rest = id / p.xtiles, planes = c.G * p.passes;    // the longest first
  const int plane = rest % planes, seq = p.first_seq + rest / planes, kvh = plane / p.passes, pass = plane % p.passes;
  const int q0 = p.cu_q[seq], lq = p.cu_q[seq + 1] - q0, start = p.starts[seq];
  const int row0 = xt * p.bq;
  if (row0 >= lq || start + lq > static_cast<int64_t>(p.table_cols) * c.bs) return;
  const int32_t *bt = c.bt + seq * c.bt_stride;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int nh = min(p.hpp, p.group - pass * p.hpp);
  const int last_row = min(row0 + p.bq, lq) - 1, i_last = start + last_row;
  const int wave_first = start + min(row0 + wave * CT * 16 / p.hpp, last_row);
  const int wave_last = min(start + row0 + ((wave + 1) * CT * 16 - 1) / p.hpp, i_last);

  int upos[CT];
  int64_t uat[CT];
  bool uok[CT];
  bf16x8 qf[CT][DC];
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const int u = wave * CT * 16 + k * 16 + n, r = row0 + u / p.hpp, hh = u % p.hpp;
    uok[k] = u < p.bq * p.hpp && r <= last_row && hh < nh;
    const int row = min(r, last_row), h = kvh * p.group + pass * p.hpp + (hh < nh ? hh : 0);
    upos[k] = start + row;
    uat[k] = static_cast<int64_t>(q0 + row) * p.H + h;
#pragma unroll
    for (int kc = 0; kc < DC; ++kc) {
      Pack16 t;
      t.u = *reinterpret_cast<const uint4 *>(p.q + uat[k] * DP + g * 8 + kc * 32);
      qf[k][kc] = t.v;
    }
  }
  uint4 kreg[DC];
#pragma unroll
  for (int i = 0; i < DC; ++i) kreg[i] = make_uint4(0, 0, 0, 0);
  auto load_tile = [&](int j0) __attribute__((always_inline)) {
    const int pg = sink_page_of(c, j0);
    const unsigned short *kp = static_cast<const unsigned short *>(c.k) + sink_row(c, bt[pg], pg, kvh, j0) * DP;
#pragma unroll
    for (int i = 0; i < DC; ++i) kreg[i] = *reinterpret_cast<const uint4 *>(kp + (tid + i * 256) * 8);
  };
  auto store_tile = [&](int stage) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < DC; ++i) {
      const int item = tid + i * 256;
      *reinterpret_cast<uint4 *>(&Ks[stage][talk_tile_row(item / KCH)][item % KCH * 8]) = kreg[i];
    }
  };
  float m[CT], l[CT];
#pragma unroll
  for (int k = 0; k < CT; ++k) { m[k] = -INFINITY; l[k] = 0.f; }
  const int tiles = i_last / kTS + 1;
  load_tile(0);
  store_tile(0);
  lds_barrier();
  for (int t = 0; t < tiles; ++t) {
    const int k0 = t * kTS, stage = t & 1;
    if (t + 1 < tiles) load_tile(k0 + kTS);
    if (k0 <= wave_last) {                                           // wave uniform: some unit sees some key
      float w[CT][2][8];
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        floatx4 s0[CT], s1[CT];
#pragma unroll
        for (int k = 0; k < CT; ++k) s0[k] = s1[k] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kc = 0; kc < DC; ++kc) {
          Pack16 a0, a1;
          a0.u = *reinterpret_cast<const uint4 *>(&Ks[stage][hf * 32 + n][kc * 32 + g * 8]);
          a1.u = *reinterpret_cast<const uint4 *>(&Ks[stage][hf * 32 + n + 16][kc * 32 + g * 8]);
#pragma unroll
          for (int k = 0; k < CT; ++k) {
            s0[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0.v, qf[k][kc], s0[k], 0, 0, 0);
            s1[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1.v, qf[k][kc], s1[k], 0, 0, 0);
          }
        }
#pragma unroll
        for (int k = 0; k < CT; ++k)
#pragma unroll
          for (int j = 0; j < 8; ++j) w[k][hf][j] = j < 4 ? s0[k][j & 3] : s1[k][j & 3];
      }
      if (k0 + kTS - 1 > wave_first)                                 // the diagonal cuts the tile
#pragma unroll
        for (int k = 0; k < CT; ++k)
#pragma unroll
          for (int j = 0; j < 16; ++j) w[k][j >> 3][j & 7] = k0 + (j >> 3) * 32 + g * 8 + (j & 7) <= upos[k] ? w[k][j >> 3][j & 7] : -INFINITY;
#pragma unroll
      for (int k = 0; k < CT; ++k) {                                 // a lane's own maximum
        float x = w[k][0][0];
#pragma unroll
        for (int j = 1; j < 16; ++j) x = fmaxf(x, w[k][j >> 3][j & 7]);
        const float mn = fmaxf(m[k], x), ms = mn == -INFINITY ? 0.f : mn;
        l[k] *= __builtin_amdgcn_exp2f(m[k] - ms);
        m[k] = mn;
#pragma unroll
        for (int j = 0; j < 16; ++j) l[k] += __builtin_amdgcn_exp2f(w[k][j >> 3][j & 7] - ms);
      }
    }
    if (t + 1 < tiles) store_tile(stage ^ 1);
    lds_barrier();
  }
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const float top = max_lanes_16_32_48(m[k]);                      // a row sees itself: finite
    const float sum = sum_lanes_16_32_48(l[k] * __builtin_amdgcn_exp2f(m[k] - top));
    if (g == 0 && uok[k]) p.stats[uat[k]] = top + __builtin_amdgcn_logf(sum);
  }
}

// A row's place in LDS for heads of WV waves: W [key][head], later M [head][key]; hi and lo apart; rows begin in different banks.
__host__ __device__ constexpr int talk_heads_held(int wv) { return wv == 1 ? 8 : wv * 4; }
__host__ __device__ constexpr int talk_row_size(int wv) {
  return (talk_heads_held(wv) * kTM > kTK * talk_heads_held(wv) ? talk_heads_held(wv) * kTM : kTK * talk_heads_held(wv)) + 8;
}

__device__ __forceinline__ shortx4 talk_read_tr16_at(unsigned int lds) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16(reinterpret_cast<shortx4 __attribute__((address_space(3))) *>(lds));
}

// LDS by byte address: one register and constants instead of a pointer per place
typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));
template <typename T>
__device__ __forceinline__ T talk_ld(unsigned int at) {
  return *reinterpret_cast<const T __attribute__((address_space(3))) *>(at);
}
template <typename T>
__device__ __forceinline__ void talk_st(unsigned int at, const T &v) {
  *reinterpret_cast<T __attribute__((address_space(3))) *>(at) = v;
}

// WV: quads of heads, RT: tiles of 16 rows; DC: key dimensions in units of 32, VC: of values, rounded up to 2 or 4; GS: heads of a
// quad that share a KV head (1, 2 or 4).  A wave has RW row tiles of HW heads of KV KV heads, HK each: item e = (KV head, row tile, head).
template <int WV, int RT, int DC, int VC, int GS>
__global__ __launch_bounds__(WV * RT * 64) void talk_prefill_kernel(const TalkPrefillArgs p) {
  constexpr int HP = talk_heads_held(WV), HT = (HP + 15) / 16, KH = (HP + 31) / 32, ROW = talk_row_size(WV), TQ = RT * 16, NW = WV * RT;
  constexpr int VP = VC * 32, PIECES = VP / 8, RW = RT < 4 / GS ? RT : 4 / GS, HW = 4 / RW, KV = HW > GS ? HW / GS : 1, HK = HW / KV;
  constexpr int PER = 4 / KV;                                        // items of a KV head
  constexpr int TS = KH * 32 + 8;                                    // heads of a talk row in LDS
  constexpr int kAtOnce = HT == 1 ? 4 : 1;                           // rows of the mix, as registers allow
  extern __shared__ __attribute__((aligned(1024))) unsigned short lds[];
  unsigned short *Vs = lds, *Wh = lds + p.c.G * kTK * VP, *Wl = Wh + TQ * ROW, *Ts = Wl + TQ * ROW;    // Vs [G][32][VP], Ts [16 HT][TS]
  const int id = (blockIdx.x & 7) * p.per_xcd + (blockIdx.x >> 3);   // neighbours in rows share keys: the same XCD
  if (id >= p.total) return;
  const SinkCache &c = p.c;
  const int xt = p.xtiles - 1 - id % p.xtiles, seq = p.first_seq + id / p.xtiles;       // the longest first
  const int q0 = p.cu_q[seq], lq = p.cu_q[seq + 1] - q0, start = p.starts[seq];
  const int row0 = xt * TQ;
  if (row0 >= lq || start + lq > static_cast<int64_t>(p.table_cols) * c.bs) return;
  const int32_t *bt = c.bt + seq * c.bt_stride;
  const int G = c.G;
  const int tid = threadIdx.x, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), h0 = wave % (WV * 4 / HW) * HW, rt = wave / (WV * 4 / HW) * RW * 16;
  const int last_row = min(row0 + TQ, lq) - 1, i_last = start + last_row;
  const int wave_first = start + min(row0 + rt, last_row);           // keys behind it are masked for some row of the wave
  auto head_of = [](int e) { return e / PER * HK + e % HK; };        // of the wave's heads; and the row tile
  auto tile_of = [](int e) { return e % PER / HK; };
  const int tiles = i_last / kTK + 1;
  // where a tile lies: its page (an unmapped one reads page 0) and its first row there, stepped tile by tile
  struct Place {
    int index, page, row;
  };
  auto page_at = [&](int index) __attribute__((always_inline)) {
    const int page = talk_uniform(bt + index);
    return page >= 0 && page < c.pages ? page : 0;
  };
  auto after = [&](const Place &at, bool more) __attribute__((always_inline)) {       // the next tile's, if there is one
    const bool turn = at.row + kTK == c.bs;
    Place b{at.index + (turn && more ? 1 : 0), at.page, turn ? 0 : at.row + kTK};
    if (turn && more) b.page = page_at(b.index);
    return more ? b : at;
  };
  auto row_of = [&](const Place &at, int kv) __attribute__((always_inline)) { return (static_cast<int64_t>(at.page) * G + kv) * c.bs + at.row; };

  // heads that no wave has, and keys that a first tile does not, are read by the mix (times zero)
  for (int i = tid; i < 2 * TQ * ROW / 8; i += NW * 64) reinterpret_cast<uint4 *>(Wh)[i] = make_uint4(0, 0, 0, 0);
  for (int i = tid; i < HT * 16 * TS; i += NW * 64) {
    const int h = i / TS, k = i % TS;
    Ts[i] = h < p.H && k < p.H ? p.talk[h * p.H + k] : 0;
  }
  bf16x8 qf[4][DC];
  int kvh[KV];
  float m[4];
#pragma unroll
  for (int i = 0; i < KV; ++i) kvh[i] = min(h0 + i * HK, p.H - 1) / p.group;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int h = min(h0 + head_of(e), p.H - 1), row = q0 + min(row0 + rt + tile_of(e) * 16 + n, last_row);
    m[e] = p.stats[static_cast<int64_t>(row) * p.H + h];
    const unsigned short *qp = p.q + (static_cast<int64_t>(row) * p.H + h) * c.Dp + g * 8;
#pragma unroll
    for (int kc = 0; kc < DC; ++kc) {
      Pack16 t;
      t.u = *reinterpret_cast<const uint4 *>(qp + kc * 32);
      qf[e][kc] = t.v;
    }
  }
  const int krow = (n >> 2) * 8 + (n & 3);
  const unsigned int koff = (krow * DC * 32 + g * 8) * 2;
  auto load_k = [&](bf16x8 (&kf)[DC], const Place &at, int kv, int s) __attribute__((always_inline)) {    // half s of a tile's rows
    const char *kp = static_cast<const char *>(c.k) + row_of(at, kv) * (DC * 64);    // uniform
#pragma unroll
    for (int kc = 0; kc < DC; ++kc) {
      Pack16 t;
      t.u = *reinterpret_cast<const uint4 *>(kp + koff + (s * 4 * DC * 64 + kc * 64));
      kf[kc] = t.v;
    }
  };
  floatx4 acc[4][2 * VC];
#pragma unroll
  for (int e = 0; e < 4; ++e)
#pragma unroll
    for (int d = 0; d < 2 * VC; ++d) acc[e][d] = floatx4{0.f, 0.f, 0.f, 0.f};
  const unsigned int vlds = TLF_DL_LDSADDR(Vs);
  // V's 16-byte pieces in LDS: pairs of them are permuted within a row, so that a transpose read (rows 8 g + 0 .. 3, or four on)
  // meets every bank twice.  Byte address of this lane's part of the first pair; pair d is d * 32 away by exclusive or.
  auto pair_of = [](int row) __attribute__((always_inline)) { return VC >= 4 ? (row & 3) | (row >> 1 & 4) : (row >> 1 & 1) | (row >> 2 & 2); };
  const int vrow = g * 8 + (n >> 2);
  unsigned int vat = vlds + (vrow * VP + pair_of(vrow) * 16 + (n & 3) * 4) * 2;
  constexpr unsigned int LO = TQ * ROW * 2;                          // from a pair's high half to its low one
  const unsigned int w0 = TLF_DL_LDSADDR(Wh);
  unsigned int tat = TLF_DL_LDSADDR(Ts) + (n * TS + g * 8) * 2;
  unsigned int wat = w0 + ((rt + n) * ROW + g * 8 * HP + h0) * 2;    // where this lane puts weights
  unsigned int mat = w0 + ((rt + n) * ROW + h0 * kTM + g * 8) * 2;   // where it finds mixed ones
  unsigned int rat = w0 + (wave * ROW + krow * HP + g * 8) * 2;      // a row's weights as the mix's operand
  unsigned int pat = w0 + (wave * ROW + n * kTM + g * 8) * 2;        // and its result

  bf16x8 kb[DC];
  Place at{0, page_at(0), 0};
  load_k(kb, at, kvh[0], 0);
  lds_barrier();
  for (int t = 0; t < tiles; ++t) {
    const int j0 = t * kTK;
    const Place next = after(at, t + 1 < tiles);
    auto copy_v = [&]() __attribute__((always_inline)) {
      const int pieces = c.Vp / 8;
      for (int i = wave; i < G * (VP / 16); i += NW) {
        const int kv = i / (VP / 16), slot = i % (VP / 16) * 64 + lane, row = slot / PIECES, piece = (slot % PIECES) ^ (pair_of(row) * 2);
        const unsigned char *base = reinterpret_cast<const unsigned char *>(static_cast<const unsigned short *>(c.v) + row_of(at, kv) * c.Vp);
        TLF_DL_COPY(static_cast<unsigned int>((row * pieces + (piece < pieces ? piece : 0)) * 16), base, vlds + i * 1024);
      }
    };
#pragma unroll
    for (int u = 0; u < 2 * KV; ++u) {                               // (KV head, half a tile)
      const int e0 = u / 2 * PER, s = u % 2;
      floatx4 w[PER];
#pragma unroll
      for (int e = 0; e < PER; ++e) w[e] = floatx4{0.f, 0.f, 0.f, 0.f};
      // lane (n, g): keys j0 + g * 8 + s * 4 + 0 .. 3 of row n
#pragma unroll
      for (int kc = 0; kc < DC; ++kc)
#pragma unroll
        for (int e = 0; e < PER; ++e) w[e] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kb[kc], qf[e0 + e][kc], w[e], 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
      if (u == 2 * KV - 1) copy_v();                                 // this tile's K is there: V's copies follow it
      if (u + 1 < 2 * KV) load_k(kb, at, kvh[(u + 1) / 2], (u + 1) % 2);
      else if (t + 1 < tiles) load_k(kb, next, kvh[0], 0);
      if (j0 + kTK - 1 > wave_first)                                 // the diagonal cuts the tile
#pragma unroll
        for (int e = 0; e < PER; ++e) {
          const int pos = start + min(row0 + rt + tile_of(e0 + e) * 16 + n, last_row) - j0 - g * 8 - s * 4;
#pragma unroll
          for (int r = 0; r < 4; ++r) w[e][r] = r <= pos ? w[e][r] : -INFINITY;
        }
#pragma unroll
      for (int x = 0; x < PER / HK; ++x)                             // row tiles
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const unsigned int to = wat + (x * 16 * ROW + (s * 4 + r) * HP + u / 2 * HK) * 2;
          const int e1 = x * HK;
          if constexpr (HK == 1) {
            const float a = __builtin_amdgcn_exp2f(w[e1][r] - m[e0 + e1]);
            const unsigned short hi = float_to_bf16_bits(a);
            talk_st<unsigned short>(to, hi);
            talk_st<unsigned short>(to + LO, float_to_bf16_bits(a - bf16_bits_to_float(hi)));
          } else {
            unsigned int hi[HK / 2], lo[HK / 2];
#pragma unroll
            for (int e = 0; e < HK; e += 2) {
              const float a = __builtin_amdgcn_exp2f(w[e1 + e][r] - m[e0 + e1 + e]), b = __builtin_amdgcn_exp2f(w[e1 + e + 1][r] - m[e0 + e1 + e + 1]);
              hi[e / 2] = pack_bf16x2(a, b);
              lo[e / 2] = pack_bf16x2(a - __uint_as_float(hi[e / 2] << 16), b - __uint_as_float(hi[e / 2] & 0xffff0000u));
            }
            if constexpr (HK == 4) {
              talk_st<u32x2>(to, u32x2{hi[0], hi[1]});
              talk_st<u32x2>(to + LO, u32x2{lo[0], lo[1]});
            } else {
              talk_st<unsigned int>(to, hi[0]);
              talk_st<unsigned int>(to + LO, lo[0]);
            }
          }
        }
    }
    lds_barrier();
    // talk^T as the mix's B operand: lane (n, g) of tile t holds talk[16 t + n][32 k + 8 g ..]
    bf16x8 tf[HT][KH];
    asm volatile("" : "+v"(tat), "+v"(rat), "+v"(pat));              // read here, not kept in registers
#pragma unroll
    for (int ht = 0; ht < HT; ++ht)
#pragma unroll
      for (int k = 0; k < KH; ++k) tf[ht][k] = talk_ld<bf16x8>(tat + (ht * 16 * TS + k * 32) * 2);
#pragma unroll kAtOnce
    for (int i = 0; i < TQ / NW; ++i) {                              // a row's W is read and its M written by the same wave
      const unsigned int row_at = i * (NW * ROW * 2);
      floatx4 mx[HT][2];
#pragma unroll
      for (int ht = 0; ht < HT; ++ht) mx[ht][0] = mx[ht][1] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KH; ++k) {
        bf16x8 hi[2], lo[2];
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          hi[s] = lo[s] = __builtin_bit_cast(bf16x8, make_uint4(0, 0, 0, 0));
          if (k * 32 + g * 8 < HP) {                                 // heads there are room for
            hi[s] = talk_ld<bf16x8>(rat + row_at + (s * 4 * HP + k * 32) * 2);
            lo[s] = talk_ld<bf16x8>(rat + row_at + (s * 4 * HP + k * 32) * 2 + LO);
          }
        }
#pragma unroll
        for (int ht = 0; ht < HT; ++ht)
#pragma unroll
          for (int s = 0; s < 2; ++s) mx[ht][s] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[s], tf[ht][k], mx[ht][s], 0, 0, 0);
#pragma unroll
        for (int ht = 0; ht < HT; ++ht)
#pragma unroll
          for (int s = 0; s < 2; ++s) mx[ht][s] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[s], tf[ht][k], mx[ht][s], 0, 0, 0);
      }
      wave_lds_fence();
#pragma unroll
      for (int ht = 0; ht < HT; ++ht) {                              // lane (n, g): head 16 ht + n, keys 8 g ..
        const float x[8] = {mx[ht][0][0], mx[ht][0][1], mx[ht][0][2], mx[ht][0][3], mx[ht][1][0], mx[ht][1][1], mx[ht][1][2], mx[ht][1][3]};
        bf16x8 hi, lo;
        talk_pair(x, hi, lo);
        if (HP >= 16 || n < HP) {
          talk_st<bf16x8>(pat + row_at + ht * 16 * kTM * 2, hi);
          talk_st<bf16x8>(pat + row_at + ht * 16 * kTM * 2 + LO, lo);
        }
      }
    }
    // this wave's copies are there when at most the loads of the next K, issued after them, are on their way
    if (t + 1 < tiles) TLF_DL_BARRIER(DC);
    else TLF_DL_BARRIER(0);
    asm volatile("" : "+v"(vat), "+v"(mat), "+v"(wat));                                    // addresses are made here, not kept in registers
#pragma unroll
    for (int e0 = 0; e0 < 4; e0 += 2) {
      bf16x8 mh[2], ml[2];
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const unsigned int from = mat + (tile_of(e0 + e) * 16 * ROW + head_of(e0 + e) * kTM) * 2;
        mh[e] = talk_ld<bf16x8>(from);
        ml[e] = talk_ld<bf16x8>(from + LO);
      }
#pragma unroll
      for (int d = 0; d < 2 * VC; ++d) {
        bf16x8 vb[2];
#pragma unroll
        for (int e = 0; e < 2; ++e)
          if (e == 0 || PER == 1) {
            const unsigned int at = (vat + kvh[(e0 + e) / PER] * (kTK * VP * 2)) ^ (d * 32);
            const uint2 v0 = __builtin_bit_cast(uint2, talk_read_tr16_at(at)), v1 = __builtin_bit_cast(uint2, talk_read_tr16_at(at + 8 * VP));
            vb[e] = __builtin_bit_cast(bf16x8, make_uint4(v0.x, v0.y, v1.x, v1.y));
          } else {
            vb[e] = vb[0];
          }
#pragma unroll
        for (int e = 0; e < 2; ++e) acc[e0 + e][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb[e], mh[e], acc[e0 + e][d], 0, 0, 0);
#pragma unroll
        for (int e = 0; e < 2; ++e) acc[e0 + e][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb[e], ml[e], acc[e0 + e][d], 0, 0, 0);
      }
    }
    lds_barrier();                                                   // V and M have been read by all
    at = next;
  }

  const bool vec = (c.Dv & 3) == 0 && (p.ldo & 3) == 0 && (reinterpret_cast<uintptr_t>(p.out) & 7) == 0;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int row = row0 + rt + tile_of(e) * 16 + n, h = h0 + head_of(e);
    if (row > last_row || h >= p.H) continue;
    unsigned short *o = p.out + static_cast<int64_t>(q0 + row) * p.ldo + static_cast<int64_t>(h) * c.Dv;
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

// Quads of heads as instantiated, 0: too many.
inline int talk_quads(int heads) { return heads <= 4 ? 1 : heads <= 8 ? 2 : heads <= 16 ? 4 : heads <= 32 ? 8 : 0; }
constexpr int kTalkLds = 160 * 1024;
inline int talk_units(int padded) { return padded <= 64 ? 2 : 4; }     // of 32, as instantiated
int talk_prefill_lds(int quads, int rt, int G, int Vp) {
  return 2 * (2 * rt * 16 * talk_row_size(quads) + G * kTK * talk_units(Vp) * 32 + (quads > 4 ? 32 : 16) * 40);
}
// Row tiles per workgroup: up to eight waves, with 16 heads fewer where LDS does not hold them; 0: no room.
int talk_row_tiles(int quads, int G, int Vp) {
  const int most = 8 / quads < 4 ? 8 / quads : 4;
  return talk_prefill_lds(quads, most, G, Vp) <= kTalkLds ? most : quads == 4 && talk_prefill_lds(quads, 1, G, Vp) <= kTalkLds ? 1 : 0;
}

template <int DC>
int launch_talk_stats(TalkPrefillArgs &a, int num_seqs, int max_tokens, hipStream_t s) {
  constexpr int CT = 2, kUnits = 64 * CT;
  a.hpp = a.group < kUnits ? a.group : kUnits;
  a.passes = (a.group + a.hpp - 1) / a.hpp;
  a.bq = kUnits / a.hpp;
  a.xtiles = (max_tokens + a.bq - 1) / a.bq;
  const int64_t total = static_cast<int64_t>(a.xtiles) * a.c.G * a.passes * num_seqs;
  if (total > (1 << 28)) return TLF_E_SHAPE;
  a.total = static_cast<int32_t>(total);
  a.per_xcd = (a.total + 7) / 8;
  TLF_LAUNCH((talk_stats_kernel<DC, CT>), dim3(a.per_xcd * 8), dim3(256), 0, s, a);
  return launch_status();
}

template <int WV, int RT, int DC, int VC, int GS>
int launch_talk_prefill(TalkPrefillArgs &a, int num_seqs, int max_tokens, hipStream_t s) {
  static const hipError_t allowed = hipFuncSetAttribute(reinterpret_cast<const void *>(&talk_prefill_kernel<WV, RT, DC, VC, GS>),
                                                        hipFuncAttributeMaxDynamicSharedMemorySize, kTalkLds);
  if (allowed != hipSuccess) return static_cast<int>(allowed);
  a.xtiles = (max_tokens + RT * 16 - 1) / (RT * 16);
  const int64_t total = static_cast<int64_t>(a.xtiles) * num_seqs;
  if (total > (1 << 28)) return TLF_E_SHAPE;
  a.total = static_cast<int32_t>(total);
  a.per_xcd = (a.total + 7) / 8;
  TLF_LAUNCH((talk_prefill_kernel<WV, RT, DC, VC, GS>), dim3(a.per_xcd * 8), dim3(WV * RT * 64), talk_prefill_lds(WV, RT, a.c.G, a.c.Vp), s, a);
  return launch_status();
}
template <int WV, int RT>
int launch_talk_prefill_dims(TalkPrefillArgs &a, int num_seqs, int max_tokens, hipStream_t s) {
#define TLF_TP(DC, VC)                                                                                                    \
  do {                                                                                                                    \
    if (a.group % 4 == 0) return launch_talk_prefill<WV, RT, DC, VC, 4>(a, num_seqs, max_tokens, s);                      \
    if (a.group % 2 == 0) return launch_talk_prefill<WV, RT, DC, VC, 2>(a, num_seqs, max_tokens, s);                      \
    return launch_talk_prefill<WV, RT, DC, VC, 1>(a, num_seqs, max_tokens, s);                                            \
  } while (0)
#define TLF_TP_V(DC)                            \
  case DC:                                      \
    if (talk_units(a.c.Vp) == 2) TLF_TP(DC, 2); \
    TLF_TP(DC, 4);
  switch (a.c.Dp / 32) {
    TLF_TP_V(1) TLF_TP_V(2) TLF_TP_V(3) TLF_TP_V(4)
    default: return TLF_E_UNSUPPORTED;
  }
#undef TLF_TP_V
#undef TLF_TP
}

}  // namespace tlf

extern "C" int tlf_talk_attn_prefill_supported(int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim) {
  return heads > 0 && kv_heads > 0 && dim > 0 && vdim > 0 && heads <= 32 && dim <= 128 && vdim <= 128 &&
         tlf::talk_row_tiles(tlf::talk_quads(heads), kv_heads, (vdim + 31) / 32 * 32) > 0;
}

extern "C" int tlf_talk_attn_prefill(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables,
                                     int64_t bt_stride, const int32_t *cu_seqlens_q, const int32_t *seq_starts, int32_t first_seq,
                                     int32_t num_seqs, int32_t max_tokens, const void *talk, float *stats, void *out, int64_t out_stride,
                                     int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size,
                                     int64_t num_pages, void *stream) {
  using namespace tlf;
  if (num_seqs < 0 || max_tokens < 0 || first_seq < 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads) return TLF_E_SHAPE;
  if (out_stride < static_cast<int64_t>(heads) * vdim || bt_stride <= 0) return TLF_E_SHAPE;
  if (num_seqs == 0 || max_tokens == 0) return TLF_OK;
  TalkPrefillArgs a{};
  if (int rc = sink_cache_make(a.c, k_cache, v_cache, block_tables, bt_stride, block_size, kv_heads, dim, vdim, num_pages)) return rc;
  if (!tlf_talk_attn_prefill_supported(heads, kv_heads, dim, vdim)) return TLF_E_UNSUPPORTED;
  if (!q || !block_tables || !cu_seqlens_q || !seq_starts || !talk || !stats || !out) return TLF_E_NULL;
  if (!aligned16(q)) return TLF_E_ALIGN;
  a.stats = stats; a.q = static_cast<const unsigned short *>(q); a.talk = static_cast<const unsigned short *>(talk); a.cu_q = cu_seqlens_q;
  a.starts = seq_starts; a.out = static_cast<unsigned short *>(out); a.ldo = out_stride; a.H = heads; a.group = heads / kv_heads;
  a.first_seq = first_seq; a.table_cols = static_cast<int32_t>(bt_stride);
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int quads = talk_quads(heads);
  int rc;
  switch (a.c.Dp / 32) {
    case 1: rc = launch_talk_stats<1>(a, num_seqs, max_tokens, s); break;
    case 2: rc = launch_talk_stats<2>(a, num_seqs, max_tokens, s); break;
    case 3: rc = launch_talk_stats<3>(a, num_seqs, max_tokens, s); break;
    default: rc = launch_talk_stats<4>(a, num_seqs, max_tokens, s); break;
  }
  if (rc != TLF_OK) return rc;
#define TLF_TP(WV, RT) \
  case (WV) * 8 + (RT): return launch_talk_prefill_dims<WV, RT>(a, num_seqs, max_tokens, s);
  switch (quads * 8 + talk_row_tiles(quads, kv_heads, a.c.Vp)) {
    TLF_TP(1, 4) TLF_TP(2, 4) TLF_TP(4, 1) TLF_TP(4, 2) TLF_TP(8, 1)
    default: return TLF_E_UNSUPPORTED;
  }
#undef TLF_TP
}
