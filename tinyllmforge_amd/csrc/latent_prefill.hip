// Latent attention of long prompt portions, bf16, on the matrix cores, from keys and values expanded per head (geometry in
// latent_attn.h): row r of `expanded` holds the keys' own parts of all heads and then the values, the rotated key part
// shared by the heads is read from the gathered cache rows.
//
// A workgroup owns one portion, one head and 128 query rows, 32 per wave, and walks the keys its window covers 64 at a time
// (global -> registers one tile ahead -> LDS):
//   S^T[key, row] = K . Q^T       v_mfma_f32_16x16x32_bf16
//   P = 2^(S * scale - m)         fp32; m follows a row's maximum only when that has grown by more than 8 (a factor of 256,
//                                 which the fp32 sums and the bf16 pair hold), so the accumulators are rarely rescaled
//   O^T[dim, row] += V^T . P^T    V^T by LDS transpose reads; P as a bf16 hi + lo pair (16 significant bits)
// K rows are permuted inside a tile so that the accumulators of two 16-key sub-tiles are the 32-key B operand of the second
// product.
#include "latent_attn.h"

namespace tlf {

constexpr int kPK = 64, kPQ = 128;   // keys per tile, query rows per workgroup

struct LatentPrefillArgs {
  LatentShape s;
  const unsigned short *q;          // [rows, H, Dq]
  const unsigned short *expanded;   // [kv rows, lde]: H * Da, then H * Va
  const unsigned short *latents;    // [kv rows, Lp]
  const int32_t *cu_q, *starts, *kv_off;
  const float *gate;                // [rows, H] or NULL
  unsigned short *out;              // [rows, ldo]
  int64_t lde, ldo;
  int32_t first_seq, window, xtiles, total, per_xcd;
  float scale_log2;
};

__device__ __forceinline__ int prefill_tile_row(int t) { return (t & 32) | ((t & 4) << 2) | ((t & 24) >> 1) | (t & 3); }
__device__ __forceinline__ shortx4 prefill_read_tr16(const unsigned short *p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p));
}

// DC, VC: query / key and value dimensions in units of 32 (rounded up to what is instantiated)
template <int DC, int VC>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2, 2))) void latent_prefill_kernel(const LatentPrefillArgs p) {
  constexpr int CT = 2, DP = DC * 32, VP = VC * 32;
  __shared__ __attribute__((aligned(16))) unsigned short Ks[kPK][DP + 8], Vs[kPK][VP + 16];
  // consecutive row tiles of one head share keys: they go to the same XCD (workgroup w runs on XCD w % 8)
  const int id = (blockIdx.x & 7) * p.per_xcd + (blockIdx.x >> 3);
  if (id >= p.total) return;
  const LatentShape &s = p.s;
  const int xt = id % p.xtiles, rest = id / p.xtiles;
  const int h = rest % s.H, sq = rest / s.H, seq = p.first_seq + sq;
  const int q0 = p.cu_q[seq], lq = p.cu_q[seq + 1] - q0, start = p.starts[seq];
  const int row0 = xt * kPQ;
  if (row0 >= lq) return;
  const int kv0 = p.kv_off[sq], kv_n = p.kv_off[sq + 1] - kv0;
  const int kbase = max(0, start - p.window + 1);            // position of the portion's first dense row
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int last_row = min(row0 + kPQ, lq) - 1;
  const int i_first = start + row0, i_last = start + last_row;
  const int wave_first = i_first + wave * 32, wave_last = min(wave_first + 31, i_last);

  int upos[CT];
  bool uok[CT];
  bf16x8 qf[CT][DC];
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const int r = row0 + wave * 32 + k * 16 + n;
    uok[k] = r <= last_row;
    const int row = uok[k] ? r : last_row;
    upos[k] = start + row;
    const unsigned short *qp = p.q + (static_cast<int64_t>(q0 + row) * s.H + h) * s.Dq + g * 8;
#pragma unroll
    for (int kc = 0; kc < DC; ++kc) {
      Pack16 t;
      t.u = kc * 32 < s.Dq ? *reinterpret_cast<const uint4 *>(qp + kc * 32) : make_uint4(0, 0, 0, 0);
      qf[k][kc] = t.v;
    }
  }

  // four threads copy a row of a tile, every fourth piece of 8 each: own part, rotated part or zeros; then the value
  const int tr = tid >> 2, td = (tid & 3) * 8;
  uint4 kreg[DC], vreg[VC];
  auto load_tile = [&](int k0) __attribute__((always_inline)) {
    const int64_t row = kv0 + min(k0 - kbase + tr, kv_n - 1);
    const unsigned short *er = p.expanded + row * p.lde, *kr = er + h * s.Da, *vr = er + s.H * s.Da + h * s.Va;
    const unsigned short *lr = p.latents + row * s.Lp + s.Ra - s.Da;
#pragma unroll
    for (int i = 0; i < DC; ++i) {
      const int d = td + i * 32;
      kreg[i] = make_uint4(0, 0, 0, 0);
      if (d < s.Da + s.Ta) kreg[i] = *reinterpret_cast<const uint4 *>((d < s.Da ? kr : lr) + d);
    }
#pragma unroll
    for (int i = 0; i < VC; ++i) {
      const int d = td + i * 32;
      vreg[i] = make_uint4(0, 0, 0, 0);
      if (d < s.Va) vreg[i] = *reinterpret_cast<const uint4 *>(vr + d);
    }
  };
  const int kw = prefill_tile_row(tr);
  auto store_tile = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < DC; ++i) *reinterpret_cast<uint4 *>(&Ks[kw][td + i * 32]) = kreg[i];
#pragma unroll
    for (int i = 0; i < VC; ++i) *reinterpret_cast<uint4 *>(&Vs[tr][td + i * 32]) = vreg[i];
  };

  floatx4 acc[CT][2 * VC];
  float m[CT], l[CT];
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    m[k] = -INFINITY;
    l[k] = 0.f;
#pragma unroll
    for (int d = 0; d < 2 * VC; ++d) acc[k][d] = floatx4{0.f, 0.f, 0.f, 0.f};
  }

  const int w0 = max(0, i_first - p.window + 1);             // >= kbase
  const int tiles = (i_last - w0) / kPK + 1;
  load_tile(w0);
  store_tile();
  lds_barrier();
  for (int t = 0; t < tiles; ++t) {
    const bool more = t + 1 < tiles;
    const int k0 = w0 + t * kPK;
    if (more) load_tile(k0 + kPK);
    if (k0 <= wave_last && k0 + kPK - 1 > wave_first - p.window) {   // wave uniform: some row sees some key
      const bool need_mask = k0 + kPK - 1 > wave_first || k0 <= wave_last - p.window;
      float w[CT][2][8];
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        floatx4 s0[CT], s1[CT];
#pragma unroll
        for (int k = 0; k < CT; ++k) s0[k] = s1[k] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kc = 0; kc < DC; ++kc) {
          Pack16 a0, a1;
          a0.u = *reinterpret_cast<const uint4 *>(&Ks[hf * 32 + n][kc * 32 + g * 8]);
          a1.u = *reinterpret_cast<const uint4 *>(&Ks[hf * 32 + n + 16][kc * 32 + g * 8]);
#pragma unroll
          for (int k = 0; k < CT; ++k) {
            s0[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0.v, qf[k][kc], s0[k], 0, 0, 0);
            s1[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1.v, qf[k][kc], s1[k], 0, 0, 0);
          }
        }
        // lane (n, g) of column tile k holds keys k0 + hf * 32 + g * 8 + j
#pragma unroll
        for (int k = 0; k < CT; ++k) {
#pragma unroll
          for (int j = 0; j < 8; ++j) w[k][hf][j] = (j < 4 ? s0[k][j & 3] : s1[k][j & 3]) * p.scale_log2;
          if (need_mask) {
            const int key = k0 + hf * 32 + g * 8;
#pragma unroll
            for (int j = 0; j < 8; ++j) w[k][hf][j] = key + j <= upos[k] && key + j > upos[k] - p.window ? w[k][hf][j] : -INFINITY;
          }
        }
      }
      float mt[CT];
      bool grown = false;
#pragma unroll
      for (int k = 0; k < CT; ++k) {
        float x = w[k][0][0];
#pragma unroll
        for (int j = 1; j < 16; ++j) x = fmaxf(x, w[k][j >> 3][j & 7]);
        mt[k] = max_lanes_16_32_48(x);
        grown = grown || mt[k] > m[k] + 8.f;
      }
      if (__any(grown)) {
#pragma unroll
        for (int k = 0; k < CT; ++k) {
          const float mn = fmaxf(m[k], mt[k]);
          const float back = mn == m[k] ? 1.f : __builtin_amdgcn_exp2f(m[k] - mn);
          m[k] = mn;
          l[k] *= back;
#pragma unroll
          for (int d = 0; d < 2 * VC; ++d) acc[k][d] *= back;
        }
      }
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        uint4 ph[CT], pl[CT];
#pragma unroll
        for (int k = 0; k < CT; ++k) {
          const float ms = m[k] == -INFINITY ? 0.f : m[k];
          float e[8];
#pragma unroll
          for (int j = 0; j < 8; ++j) e[j] = __builtin_amdgcn_exp2f(w[k][hf][j] - ms);
          l[k] += ((e[0] + e[1]) + (e[2] + e[3])) + ((e[4] + e[5]) + (e[6] + e[7]));
          unsigned int hi[4], lo[4];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            hi[j] = pack_bf16x2(e[2 * j], e[2 * j + 1]);
            lo[j] = pack_bf16x2(e[2 * j] - __uint_as_float(hi[j] << 16), e[2 * j + 1] - __uint_as_float(hi[j] & 0xffff0000u));
          }
          ph[k] = make_uint4(hi[0], hi[1], hi[2], hi[3]);
          pl[k] = make_uint4(lo[0], lo[1], lo[2], lo[3]);
        }
        const int vt = hf * 32 + g * 8 + (n >> 2);
#pragma unroll
        for (int d = 0; d < 2 * VC; ++d) {
          const uint2 v0 = __builtin_bit_cast(uint2, prefill_read_tr16(&Vs[vt][d * 16 + (n & 3) * 4]));
          const uint2 v1 = __builtin_bit_cast(uint2, prefill_read_tr16(&Vs[vt + 4][d * 16 + (n & 3) * 4]));
          const bf16x8 vb = __builtin_bit_cast(bf16x8, make_uint4(v0.x, v0.y, v1.x, v1.y));
#pragma unroll
          for (int k = 0; k < CT; ++k) {
            acc[k][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, __builtin_bit_cast(bf16x8, ph[k]), acc[k][d], 0, 0, 0);
            acc[k][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, __builtin_bit_cast(bf16x8, pl[k]), acc[k][d], 0, 0, 0);
          }
        }
      }
    }
    lds_barrier();
    if (more) {
      store_tile();
      lds_barrier();
    }
  }

  const bool vec = (s.vdim & 3) == 0 && (p.ldo & 3) == 0 && (reinterpret_cast<uintptr_t>(p.out) & 7) == 0;
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const float den = sum_lanes_16_32_48(l[k]);
    if (!uok[k]) continue;
    float inv = 1.0f / den;                                  // a row sees itself: den > 0
    if (p.gate) inv *= p.gate[static_cast<int64_t>(q0 + upos[k] - start) * s.H + h];
    unsigned short *o = p.out + static_cast<int64_t>(q0 + upos[k] - start) * p.ldo + static_cast<int64_t>(h) * s.vdim;
#pragma unroll
    for (int d = 0; d < 2 * VC; ++d) {
      const int col = d * 16 + g * 4;
      const uint2 v = make_uint2(pack_bf16x2(acc[k][d][0] * inv, acc[k][d][1] * inv), pack_bf16x2(acc[k][d][2] * inv, acc[k][d][3] * inv));
      if (vec) {
        if (col < s.vdim) *reinterpret_cast<uint2 *>(o + col) = v;
      } else {
        const unsigned int e[2] = {v.x, v.y};
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (col + r < s.vdim) o[col + r] = static_cast<unsigned short>(e[r / 2] >> (16 * (r & 1)));
      }
    }
  }
}

inline int fit_units(int units) { return units <= 4 ? units : units <= 6 ? 6 : 8; }   // of 32, as instantiated

}  // namespace tlf

extern "C" int tlf_latent_prefill_supported(int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim) {
  tlf::LatentShape s;
  return tlf::latent_shape(s, heads, dim, rot_dim, rank, vdim) && s.Dq <= 256 && vdim <= 128;
}

extern "C" int tlf_latent_prefill(const void *q, const void *expanded, int64_t expanded_stride, const void *latents,
                                  const int32_t *cu_seqlens_q, const int32_t *seq_starts, const int32_t *kv_offsets,
                                  int32_t first_seq, int32_t num_seqs, int32_t max_tokens, const float *gate, void *out, int64_t out_stride,
                                  int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim, int32_t window,
                                  float scale, void *stream) {
  using namespace tlf;
  LatentPrefillArgs a{};
  if (num_seqs < 0 || max_tokens < 0 || first_seq < 0 || window <= 0 || !latent_shape(a.s, heads, dim, rot_dim, rank, vdim)) return TLF_E_SHAPE;
  if (a.s.Dq > 256 || vdim > 128) return TLF_E_UNSUPPORTED;
  if (expanded_stride < static_cast<int64_t>(heads) * (a.s.Da + a.s.Va) || expanded_stride % 8 || out_stride < static_cast<int64_t>(heads) * vdim) return TLF_E_SHAPE;
  if (num_seqs == 0 || max_tokens == 0) return TLF_OK;
  if (!q || !expanded || !latents || !cu_seqlens_q || !seq_starts || !kv_offsets || !out) return TLF_E_NULL;
  if (!aligned16(q) || !aligned16(expanded) || !aligned16(latents)) return TLF_E_ALIGN;
  a.q = static_cast<const unsigned short *>(q); a.expanded = static_cast<const unsigned short *>(expanded);
  a.latents = static_cast<const unsigned short *>(latents); a.cu_q = cu_seqlens_q; a.starts = seq_starts; a.kv_off = kv_offsets;
  a.out = static_cast<unsigned short *>(out); a.lde = expanded_stride; a.ldo = out_stride; a.first_seq = first_seq;
  a.gate = gate; a.window = window; a.scale_log2 = scale * 1.4426950408889634f;
  a.xtiles = (max_tokens + kPQ - 1) / kPQ;
  const int64_t total = static_cast<int64_t>(a.xtiles) * heads * num_seqs;
  if (total > (1 << 30)) return TLF_E_SHAPE;
  a.total = static_cast<int32_t>(total);
  a.per_xcd = (a.total + 7) / 8;
  const dim3 grid(a.per_xcd * 8);
  hipStream_t st = static_cast<hipStream_t>(stream);
  const int dc = fit_units(a.s.Dq / 32), vc = (vdim + 31) / 32;
#define TLF_LP(DC, VC) TLF_LAUNCH((latent_prefill_kernel<DC, VC>), grid, dim3(256), 0, st, a)
#define TLF_LP_V(DC)              \
  case DC:                        \
    if (vc == 1) TLF_LP(DC, 1);   \
    else if (vc == 2) TLF_LP(DC, 2); \
    else TLF_LP(DC, 4);           \
    break;
  switch (dc) {
    TLF_LP_V(1) TLF_LP_V(2) TLF_LP_V(3) TLF_LP_V(4) TLF_LP_V(6) TLF_LP_V(8)
    default: return TLF_E_UNSUPPORTED;
  }
#undef TLF_LP_V
#undef TLF_LP
  return launch_status();
}
