// Attention of sink_attn.h for prompt portions, bf16, on the matrix cores, from the paged cache.
//
// A workgroup owns one portion, one KV head and a tile of query rows; the (row, head) pairs of the KV head's query heads are
// flattened into 64 CT units, 16 CT per wave.  It walks the keys up to its last row 64 at a time (a tile of 64 keys is one
// contiguous piece of a page; global -> registers one tile ahead -> LDS):
//   S^T[key, unit] = K . Q^T      v_mfma_f32_16x16x32_bf16
//   P = 2^(score - m)             fp32; m follows a unit's maximum only when that has grown by more than 8 (a factor of 256,
//                                 which the fp32 sums and the bf16 pair hold), so the accumulators are rarely rescaled
//   O^T[dim, unit] += V^T . P^T   V^T by LDS transpose reads; P as a bf16 hi + lo pair (16 significant bits)
// K rows are permuted inside a tile so that the accumulators of two 16-key sub-tiles are the 32-key B operand of the second
// product.  Only tiles that the diagonal cuts are masked.  The sink and the gate are applied at the end.
#include "sink_attn.h"

namespace tlf {

constexpr int kSK = 64;   // keys per tile

struct SinkPrefillArgs {
  SinkCache c;
  float cap_log2;                   // cap * log2(e), 0: none
  const unsigned short *q;          // [rows, H, Dp]
  const unsigned short *sink;       // [H] or NULL
  const unsigned short *gate;       // [rows, ldg] or NULL
  const int32_t *cu_q, *starts;
  unsigned short *out;
  int64_t ldo, ldg;
  int32_t H, group, hpp, passes;    // query heads, per KV head, per pass
  int32_t bq, xtiles, total, first_seq, per_xcd, table_cols;
};

__device__ __forceinline__ int sink_tile_row(int t) { return (t & 32) | ((t & 4) << 2) | ((t & 24) >> 1) | (t & 3); }
__device__ __forceinline__ shortx4 sinkp_read_tr16(const unsigned short *p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p));
}

// MODE 0: no cap, 1: a cap, 2: a cap small enough to take the largest score it allows as everyone's maximum
template <int DC, int VC, int CT, int MODE>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2, 2))) void sink_prefill_kernel(const SinkPrefillArgs p) {
  constexpr int DP = DC * 32, VP = VC * 32, KCH = DC * 4, VCH = VC * 4;
  __shared__ __attribute__((aligned(16))) unsigned short Ks[kSK][DP + 8], Vs[kSK][VP + 16];
  // consecutive row tiles of one KV head share keys: they go to the same XCD (workgroup w runs on XCD w % 8); the last row
  // tiles, which see the most keys, come first
  const int id = (blockIdx.x & 7) * p.per_xcd + (blockIdx.x >> 3);
  if (id >= p.total) return;
  const SinkCache &c = p.c;
  const int xt = p.xtiles - 1 - id % p.xtiles, rest = id / p.xtiles;
  const int planes = c.G * p.passes;
  const int plane = rest % planes, seq = p.first_seq + rest / planes;
  const int kvh = plane / p.passes, pass = plane % p.passes;
  const int q0 = p.cu_q[seq], lq = p.cu_q[seq + 1] - q0, start = p.starts[seq];
  const int row0 = xt * p.bq;
  if (row0 >= lq || start + lq > static_cast<int64_t>(p.table_cols) * c.bs) return;
  const int32_t *bt = c.bt + seq * c.bt_stride;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int nh = min(p.hpp, p.group - pass * p.hpp);         // heads of this pass
  const int last_row = min(row0 + p.bq, lq) - 1;
  const int i_last = start + last_row;
  const int wave_first = start + row0 + wave * CT * 16 / p.hpp;
  const int wave_last = min(start + row0 + ((wave + 1) * CT * 16 - 1) / p.hpp, i_last);

  int upos[CT], urow[CT], uhead[CT];
  bool uok[CT];
  bf16x8 qf[CT][DC];
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const int u = wave * CT * 16 + k * 16 + n;
    const int r = row0 + u / p.hpp, hh = u % p.hpp;
    uok[k] = u < p.bq * p.hpp && r <= last_row && hh < nh;
    uhead[k] = kvh * p.group + pass * p.hpp + (hh < nh ? hh : 0);
    const int row = min(r, last_row);
    upos[k] = start + row;
    urow[k] = q0 + row;
    const unsigned short *qp = p.q + (static_cast<int64_t>(urow[k]) * p.H + uhead[k]) * c.Dp + g * 8;
#pragma unroll
    for (int kc = 0; kc < DC; ++kc) {
      Pack16 t;
      t.u = kc * 32 < c.Dp ? *reinterpret_cast<const uint4 *>(qp + kc * 32) : make_uint4(0, 0, 0, 0);
      qf[k][kc] = t.v;
    }
  }

  uint4 kreg[DC], vreg[VC];
#pragma unroll
  for (int i = 0; i < DC; ++i) kreg[i] = make_uint4(0, 0, 0, 0);
#pragma unroll
  for (int i = 0; i < VC; ++i) vreg[i] = make_uint4(0, 0, 0, 0);
  auto load_tile = [&](int j0, int page) __attribute__((always_inline)) {
    const int64_t r0 = sink_row(c, page, sink_page_of(c, j0), kvh, j0);     // rows past the last query are masked
    const unsigned short *kp = static_cast<const unsigned short *>(c.k) + r0 * c.Dp;
    const unsigned short *vp = static_cast<const unsigned short *>(c.v) + r0 * c.Vp;
#pragma unroll
    for (int i = 0; i < DC; ++i) {
      const int item = tid + i * 256, r = item / KCH, ch = item % KCH;
      if (ch * 8 < c.Dp) kreg[i] = *reinterpret_cast<const uint4 *>(kp + r * c.Dp + ch * 8);
    }
#pragma unroll
    for (int i = 0; i < VC; ++i) {
      const int item = tid + i * 256, r = item / VCH, ch = item % VCH;
      if (ch * 8 < c.Vp) vreg[i] = *reinterpret_cast<const uint4 *>(vp + r * c.Vp + ch * 8);
    }
  };
  auto store_tile = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < DC; ++i) {
      const int item = tid + i * 256, r = item / KCH, ch = item % KCH;
      *reinterpret_cast<uint4 *>(&Ks[sink_tile_row(r)][ch * 8]) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < VC; ++i) {
      const int item = tid + i * 256, r = item / VCH, ch = item % VCH;
      *reinterpret_cast<uint4 *>(&Vs[r][ch * 8]) = vreg[i];
    }
  };

  floatx4 acc[CT][2 * VC];
  float m[CT], l[CT];
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    m[k] = MODE == 2 ? p.cap_log2 : -INFINITY;
    l[k] = 0.f;
#pragma unroll
    for (int d = 0; d < 2 * VC; ++d) acc[k][d] = floatx4{0.f, 0.f, 0.f, 0.f};
  }

  const int tiles = i_last / kSK + 1;
  int next_page = bt[sink_page_of(c, min(kSK, i_last))];
  load_tile(0, bt[0]);
  store_tile();
  lds_barrier();
  for (int t = 0; t < tiles; ++t) {
    const bool more = t + 1 < tiles;
    const int k0 = t * kSK;
    if (more) {
      load_tile(k0 + kSK, next_page);
      next_page = bt[sink_page_of(c, min(k0 + 2 * kSK, i_last))];
    }
    if (k0 <= wave_last) {                                   // wave uniform: some unit sees some key
      const bool need_mask = k0 + kSK - 1 > wave_first;
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
          for (int j = 0; j < 8; ++j) {
            const float dot = j < 4 ? s0[k][j & 3] : s1[k][j & 3];
            if (MODE == 2) w[k][hf][j] = -2.f * p.cap_log2 * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(dot));
            else w[k][hf][j] = sink_score_log2<MODE == 1>(dot, p.cap_log2);
          }
          if (need_mask) {
            const int key = k0 + hf * 32 + g * 8;
#pragma unroll
            for (int j = 0; j < 8; ++j) w[k][hf][j] = key + j <= upos[k] ? w[k][hf][j] : -INFINITY;
          }
        }
      }
      if constexpr (MODE == 2) {
        // nothing to rescale; without this the compiler moves the accumulators back and forth on every tile
#pragma unroll
        for (int k = 0; k < CT; ++k)
#pragma unroll
          for (int d = 0; d < 2 * VC; ++d) asm volatile("" : "+v"(acc[k][d]));
      } else {
#pragma unroll
        for (int k = 0; k < CT; ++k) {
          float x = w[k][0][0];
#pragma unroll
          for (int j = 1; j < 16; ++j) x = fmaxf(x, w[k][j >> 3][j & 7]);
          x = max_lanes_16_32_48(x);
          const bool grown = x > m[k] + 8.f;
          const float back = grown ? __builtin_amdgcn_exp2f(m[k] - x) : 1.f;
          m[k] = grown ? x : m[k];
          l[k] *= back;
#pragma unroll
          for (int d = 0; d < VC; ++d) sink_rescale(acc[k][2 * d], acc[k][2 * d + 1], back);
        }
      }
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        uint4 ph[CT], pl[CT];
#pragma unroll
        for (int k = 0; k < CT; ++k) {
          const float ms = MODE == 2 || m[k] == -INFINITY ? 0.f : m[k];
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
          const uint2 v0 = __builtin_bit_cast(uint2, sinkp_read_tr16(&Vs[vt][d * 16 + (n & 3) * 4]));
          const uint2 v1 = __builtin_bit_cast(uint2, sinkp_read_tr16(&Vs[vt + 4][d * 16 + (n & 3) * 4]));
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

  const bool vec = (c.Dv & 3) == 0 && (p.ldo & 3) == 0 && (p.ldg & 3) == 0 && (reinterpret_cast<uintptr_t>(p.out) & 7) == 0 &&
                   (reinterpret_cast<uintptr_t>(p.gate) & 7) == 0;
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const float den = sum_lanes_16_32_48(l[k]);
    if (!uok[k]) continue;
    const float sk = p.sink ? bf16_bits_to_float(p.sink[uhead[k]]) * kSinkLog2e : -INFINITY;
    const float top = fmaxf(m[k], sk), f = __builtin_amdgcn_exp2f(m[k] - top);
    const float inv = f / (den * f + __builtin_amdgcn_exp2f(sk - top));
    unsigned short *o = p.out + static_cast<int64_t>(urow[k]) * p.ldo + static_cast<int64_t>(uhead[k]) * c.Dv;
    const unsigned short *gp = p.gate + static_cast<int64_t>(urow[k]) * p.ldg + static_cast<int64_t>(uhead[k]) * c.Dv;
#pragma unroll
    for (int d = 0; d < 2 * VC; ++d) {
      const int col = d * 16 + g * 4;
      float gt[4] = {1.f, 1.f, 1.f, 1.f};
      if (p.gate) {
        if (vec && col < c.Dv) {
          const uint2 b = *reinterpret_cast<const uint2 *>(gp + col);
          gt[0] = __uint_as_float(b.x << 16); gt[1] = __uint_as_float(b.x & 0xffff0000u);
          gt[2] = __uint_as_float(b.y << 16); gt[3] = __uint_as_float(b.y & 0xffff0000u);
        } else if (!vec) {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (col + r < c.Dv) gt[r] = bf16_bits_to_float(gp[col + r]);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) gt[r] = sigmoid_f32(gt[r]);
      }
      const uint2 v = make_uint2(pack_bf16x2(acc[k][d][0] * inv * gt[0], acc[k][d][1] * inv * gt[1]),
                                 pack_bf16x2(acc[k][d][2] * inv * gt[2], acc[k][d][3] * inv * gt[3]));
      if (vec) {
        if (col < c.Dv) *reinterpret_cast<uint2 *>(o + col) = v;
      } else {
        const unsigned int e[2] = {v.x, v.y};
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (col + r < c.Dv) o[col + r] = static_cast<unsigned short>(e[r / 2] >> (16 * (r & 1)));
      }
    }
  }
}

}  // namespace tlf

extern "C" int tlf_sink_attn_prefill_supported(int32_t dim, int32_t vdim) { return dim > 0 && vdim > 0 && dim <= 256 && vdim <= 256; }

extern "C" int tlf_sink_attn_prefill(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables,
                                     int64_t bt_stride, const int32_t *cu_seqlens_q, const int32_t *seq_starts, int32_t first_seq,
                                     int32_t num_seqs, int32_t max_tokens, const void *sink, const void *gate, int64_t gate_stride,
                                     void *out, int64_t out_stride, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim,
                                     int32_t block_size, int64_t num_pages, float cap, void *stream) {
  using namespace tlf;
  if (num_seqs < 0 || max_tokens < 0 || first_seq < 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || cap < 0.f) return TLF_E_SHAPE;
  const int64_t cols = static_cast<int64_t>(heads) * vdim;
  if (out_stride < cols || (gate && gate_stride < cols) || bt_stride <= 0) return TLF_E_SHAPE;
  if (num_seqs == 0 || max_tokens == 0) return TLF_OK;
  SinkPrefillArgs a{};
  if (int rc = sink_cache_make(a.c, k_cache, v_cache, block_tables, bt_stride, block_size, kv_heads, dim, vdim, num_pages)) return rc;
  if (!tlf_sink_attn_prefill_supported(dim, vdim)) return TLF_E_UNSUPPORTED;
  if (!q || !block_tables || !cu_seqlens_q || !seq_starts || !out) return TLF_E_NULL;
  if (!aligned16(q)) return TLF_E_ALIGN;
  const int dc = a.c.Dp / 32, vc = a.c.Vp / 32, ct = dc <= 4 && vc <= 4 ? 2 : 1, units = 64 * ct;
  a.cap_log2 = cap * kSinkLog2e;
  a.q = static_cast<const unsigned short *>(q); a.sink = static_cast<const unsigned short *>(sink);
  a.gate = static_cast<const unsigned short *>(gate); a.cu_q = cu_seqlens_q; a.starts = seq_starts;
  a.out = static_cast<unsigned short *>(out); a.ldo = out_stride; a.ldg = gate ? gate_stride : 0;
  a.H = heads; a.group = heads / kv_heads; a.hpp = a.group < units ? a.group : units;
  a.passes = (a.group + a.hpp - 1) / a.hpp;
  a.bq = units / a.hpp;
  a.xtiles = (max_tokens + a.bq - 1) / a.bq;
  a.first_seq = first_seq; a.table_cols = static_cast<int32_t>(bt_stride);
  const int64_t total = static_cast<int64_t>(a.xtiles) * kv_heads * a.passes * num_seqs;
  if (total > (1 << 30)) return TLF_E_SHAPE;
  a.total = static_cast<int32_t>(total);
  a.per_xcd = (a.total + 7) / 8;
  const dim3 grid(a.per_xcd * 8);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define TLF_SP(DC, VC)                                                                                                        \
  do {                                                                                                                        \
    constexpr int kCT = (DC) <= 4 && (VC) <= 4 ? 2 : 1;                                                                       \
    if (cap <= 0.f) TLF_LAUNCH((sink_prefill_kernel<DC, VC, kCT, 0>), grid, dim3(256), 0, s, a);                              \
    else if (cap <= 32.f) TLF_LAUNCH((sink_prefill_kernel<DC, VC, kCT, 2>), grid, dim3(256), 0, s, a);                        \
    else TLF_LAUNCH((sink_prefill_kernel<DC, VC, kCT, 1>), grid, dim3(256), 0, s, a);                                         \
  } while (0)
#define TLF_SP_V(DC)                \
  do {                              \
    if (vc <= 1) TLF_SP(DC, 1);     \
    else if (vc <= 2) TLF_SP(DC, 2); \
    else if (vc <= 4) TLF_SP(DC, 4); \
    else TLF_SP(DC, 8);             \
  } while (0)
  if (dc <= 1) TLF_SP_V(1);
  else if (dc <= 2) TLF_SP_V(2);
  else if (dc <= 4) TLF_SP_V(4);
  else if (dc <= 6) TLF_SP_V(6);
  else TLF_SP_V(8);
#undef TLF_SP_V
#undef TLF_SP
  return launch_status();
}
