// Sigmoid attention over a window plus pooled blocks for prompt portions, bf16, on the matrix cores (geometry in
// pooled_attn.h).
//
// A workgroup owns one sequence, one KV head and a tile of query rows; the (row, head) pairs of the KV head's query
// heads are flattened into 64 CT units, 16 CT per wave.  It walks the pooled rows its last query sees and then the
// tokens from its first query's window on, 64 keys at a time (global -> registers one tile ahead -> LDS):
//   S^T[key, unit] = K . Q^T       v_mfma_f32_16x16x32_bf16
//   P = sigmoid(S * scale + bias)  fp32, masked on the tiles that a window's or the diagonal's edge cuts
//   O^T[dim, unit] += V^T . P^T    the V^T operand by LDS transpose reads; P as a bf16 hi + lo pair (16 significant bits)
// The weights are not normalised: no running maximum, no rescaling, no second pass.  K rows are permuted inside a
// tile so that the accumulators of two 16-key sub-tiles are the 32-key B operand of the second product.
#include "pooled_attn.h"

namespace tlf {

constexpr int kTK = 64;   // keys per tile

struct PooledPrefillArgs {
  PooledCache c;
  const unsigned short *q;     // [rows, H, Dp]
  const unsigned short *bias;  // [H]
  const float *gate;           // [rows, H]
  const int32_t *cu_q, *starts;
  unsigned short *out;
  int64_t ldo;
  int32_t H, group, hpp, passes;   // query heads, per KV head, per pass
  int32_t bq, xtiles, total;       // query rows per workgroup, row tiles, workgroups
  int32_t first_seq, per_xcd;
  float scale_log2;
};

__device__ __forceinline__ int pooled_tile_row(int t) {
  return (t & 32) | ((t & 4) << 2) | ((t & 24) >> 1) | (t & 3);
}
__device__ __forceinline__ shortx4 pooled_read_tr16(const unsigned short *p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p));
}

template <int DC, int CT>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2, 2))) void pooled_prefill_kernel(const PooledPrefillArgs p) {
  constexpr int DP = DC * 32, NCH = DC * 4;
  __shared__ __attribute__((aligned(16))) unsigned short Ks[kTK][DP + 8], Vs[kTK][DP + 16];
  // consecutive row tiles of one KV head share keys: they go to the same XCD (workgroup w runs on XCD w % 8)
  const int id = (blockIdx.x & 7) * p.per_xcd + (blockIdx.x >> 3);
  if (id >= p.total) return;
  const PooledCache &c = p.c;
  const int xt = id % p.xtiles, rest = id / p.xtiles;
  const int planes = c.G * p.passes;
  const int plane = rest % planes, seq = p.first_seq + rest / planes;
  const int kvh = plane / p.passes, pass = plane % p.passes;
  const int q0 = p.cu_q[seq], lq = p.cu_q[seq + 1] - q0, start = p.starts[seq];
  const int row0 = xt * p.bq;
  if (row0 >= lq) return;
  const int32_t *bt = c.bt + seq * c.bt_stride;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int nh = min(p.hpp, p.group - pass * p.hpp);         // heads of this pass
  const int last_row = min(row0 + p.bq, lq) - 1;
  const int i_first = start + row0, i_last = start + last_row;

  int upos[CT], unb[CT], uoff[CT];
  bool uok[CT];
  float pb[CT];
  bf16x8 qf[CT][DC];
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    const int u = wave * CT * 16 + k * 16 + n;
    const int r = row0 + u / p.hpp, hh = u % p.hpp;
    uok[k] = u < p.bq * p.hpp && r <= last_row && hh < nh;
    const int head = kvh * p.group + pass * p.hpp + (hh < nh ? hh : 0);
    const int row = uok[k] ? r : row0;
    upos[k] = start + row;
    unb[k] = pooled_visible(upos[k], c.size, c.pool);
    uoff[k] = (q0 + row) * p.H + head;
    pb[k] = -kLog2e * bf16_bits_to_float(p.bias[head]);
    const unsigned short *qp = p.q + static_cast<int64_t>(uoff[k]) * DP + g * 8;
#pragma unroll
    for (int kc = 0; kc < DC; ++kc) {
      Pack16 t;
      t.u = *reinterpret_cast<const uint4 *>(qp + kc * 32);
      qf[k][kc] = t.v;
    }
  }
  const float nscale = -p.scale_log2;

  const int nb = pooled_visible(i_last, c.size, c.pool), nb_first = pooled_visible(i_first, c.size, c.pool);
  const int ptiles = (nb + kTK - 1) / kTK;
  const int w0 = max(0, i_first - c.size + 1) / kTK * kTK;
  const int tiles = ptiles + (i_last - w0) / kTK + 1;
  const int64_t rs = static_cast<int64_t>(c.G) * DP;
  const unsigned short *kc_ = static_cast<const unsigned short *>(c.k) + kvh * DP;
  const unsigned short *vc_ = static_cast<const unsigned short *>(c.v) + kvh * DP;
  const unsigned short *pk_ = static_cast<const unsigned short *>(c.pk) + kvh * DP;
  const unsigned short *pv_ = static_cast<const unsigned short *>(c.pv) + kvh * DP;

  uint4 kreg[DC], vreg[DC];
  auto load_tile = [&](int t) __attribute__((always_inline)) {
    if (t < ptiles) {
#pragma unroll
      for (int i = 0; i < DC; ++i) {
        const int item = tid + i * 256, r = item / NCH, ch = item % NCH;
        const int64_t o = block_row(c, bt, min(t * kTK + r, nb - 1)) * rs + ch * 8;
        kreg[i] = *reinterpret_cast<const uint4 *>(pk_ + o);
        vreg[i] = *reinterpret_cast<const uint4 *>(pv_ + o);
      }
    } else {
      // 64 tokens from a multiple of 64 on lie in one page; rows past the last query are masked
      const int j0 = w0 + (t - ptiles) * kTK;
      const int64_t base = token_row(c, bt, j0) * rs;
#pragma unroll
      for (int i = 0; i < DC; ++i) {
        const int item = tid + i * 256, r = item / NCH, ch = item % NCH;
        const int64_t o = base + r * rs + ch * 8;
        kreg[i] = *reinterpret_cast<const uint4 *>(kc_ + o);
        vreg[i] = *reinterpret_cast<const uint4 *>(vc_ + o);
      }
    }
  };
  auto store_tile = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < DC; ++i) {
      const int item = tid + i * 256, r = item / NCH, ch = item % NCH;
      *reinterpret_cast<uint4 *>(&Ks[pooled_tile_row(r)][ch * 8]) = kreg[i];
      *reinterpret_cast<uint4 *>(&Vs[r][ch * 8]) = vreg[i];
    }
  };

  floatx4 acc[CT][2 * DC];
#pragma unroll
  for (int k = 0; k < CT; ++k)
#pragma unroll
    for (int d = 0; d < 2 * DC; ++d) acc[k][d] = floatx4{0.f, 0.f, 0.f, 0.f};

  load_tile(0);
  store_tile();
  lds_barrier();
  for (int t = 0; t < tiles; ++t) {
    const bool more = t + 1 < tiles;
    if (more) load_tile(t + 1);
    const bool pooled = t < ptiles;
    const int k0 = pooled ? t * kTK : w0 + (t - ptiles) * kTK;
    const bool need_mask = pooled ? k0 + kTK > nb_first : (k0 + kTK - 1 > i_first || k0 <= i_last - c.size);
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
      uint4 ph[CT], pl[CT];
#pragma unroll
      for (int k = 0; k < CT; ++k) {
        float w[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) w[j] = sigmoid_neg_log2(fmaf(j < 4 ? s0[k][j & 3] : s1[k][j & 3], nscale, pb[k]));
        if (need_mask) {  // workgroup uniform
          const int key = k0 + hf * 32 + g * 8;
          const int lo = pooled ? 0 : upos[k] - c.size + 1, hi = pooled ? unb[k] : upos[k] + 1;
#pragma unroll
          for (int j = 0; j < 8; ++j) w[j] = key + j >= lo && key + j < hi ? w[j] : 0.f;
        }
        unsigned int h[4], l[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          h[j] = pack_bf16x2(w[2 * j], w[2 * j + 1]);
          l[j] = pack_bf16x2(w[2 * j] - __uint_as_float(h[j] << 16), w[2 * j + 1] - __uint_as_float(h[j] & 0xffff0000u));
        }
        ph[k] = make_uint4(h[0], h[1], h[2], h[3]);
        pl[k] = make_uint4(l[0], l[1], l[2], l[3]);
      }
      const int vt = hf * 32 + g * 8 + (n >> 2);
#pragma unroll
      for (int d = 0; d < 2 * DC; ++d) {
        const shortx4 v0 = pooled_read_tr16(&Vs[vt][d * 16 + (n & 3) * 4]);
        const shortx4 v1 = pooled_read_tr16(&Vs[vt + 4][d * 16 + (n & 3) * 4]);
        const bf16x8 vb = __builtin_bit_cast(bf16x8, make_uint4(__builtin_bit_cast(uint2, v0).x, __builtin_bit_cast(uint2, v0).y,
                                                               __builtin_bit_cast(uint2, v1).x, __builtin_bit_cast(uint2, v1).y));
#pragma unroll
        for (int k = 0; k < CT; ++k) {
          acc[k][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, __builtin_bit_cast(bf16x8, ph[k]), acc[k][d], 0, 0, 0);
          acc[k][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, __builtin_bit_cast(bf16x8, pl[k]), acc[k][d], 0, 0, 0);
        }
      }
    }
    lds_barrier();
    if (more) {
      store_tile();
      lds_barrier();
    }
  }

  const bool vec = (c.D & 3) == 0 && (p.ldo & 3) == 0 && (reinterpret_cast<uintptr_t>(p.out) & 7) == 0;
#pragma unroll
  for (int k = 0; k < CT; ++k) {
    if (!uok[k]) continue;
    const float gt = p.gate[uoff[k]];
    const int row = uoff[k] / p.H, head = uoff[k] - row * p.H;
    unsigned short *o = p.out + static_cast<int64_t>(row) * p.ldo + static_cast<int64_t>(head) * c.D;
#pragma unroll
    for (int d = 0; d < 2 * DC; ++d) {
      const int col = d * 16 + g * 4;
      const uint2 v = make_uint2(pack_bf16x2(acc[k][d][0] * gt, acc[k][d][1] * gt), pack_bf16x2(acc[k][d][2] * gt, acc[k][d][3] * gt));
      if (vec) {
        if (col < c.D) *reinterpret_cast<uint2 *>(o + col) = v;
      } else {
        const unsigned int e[2] = {v.x, v.y};
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (col + r < c.D) o[col + r] = static_cast<unsigned short>(e[r / 2] >> (16 * (r & 1)));
      }
    }
  }
}

}  // namespace tlf

extern "C" int tlf_pooled_attn_prefill(const void *q, const void *score_bias, const float *gate, const void *k_cache,
                                       const void *v_cache, const void *pk_cache, const void *pv_cache,
                                       const int32_t *block_tables, int64_t bt_stride, const int32_t *cu_seqlens_q,
                                       const int32_t *seq_starts, int32_t first_seq, int32_t num_seqs,
                                       int32_t max_tokens, void *out, int64_t out_stride, int32_t num_q_heads,
                                       int32_t num_kv_heads, int32_t head_dim, int32_t block_size, int32_t pool,
                                       int32_t window, int64_t num_pages, float scale, void *stream) {
  using namespace tlf;
  if (num_seqs < 0 || max_tokens < 0 || first_seq < 0 || num_q_heads <= 0 || num_kv_heads <= 0 || num_q_heads % num_kv_heads)
    return TLF_E_SHAPE;
  if (out_stride < static_cast<int64_t>(num_q_heads) * head_dim) return TLF_E_SHAPE;
  if (num_seqs == 0 || max_tokens == 0) return TLF_OK;
  PooledCache c{k_cache, v_cache, pk_cache, pv_cache, block_tables, bt_stride, block_size, pool, 0, window,
                num_kv_heads, head_dim, (head_dim + 31) / 32 * 32, num_pages, -1};
  if (int rc = pooled_cache_check(c, TLF_DT_BF16)) return rc;
  if (!q || !score_bias || !gate || !cu_seqlens_q || !seq_starts || !out) return TLF_E_NULL;
  if (!aligned16(q)) return TLF_E_ALIGN;
  pooled_cache_finish(c);
  const int dc = c.Dp / 32, ct = dc <= 4 ? 2 : 1, units = 64 * ct;
  PooledPrefillArgs a{c, static_cast<const unsigned short *>(q), static_cast<const unsigned short *>(score_bias), gate,
                      cu_seqlens_q, seq_starts, static_cast<unsigned short *>(out), out_stride, num_q_heads,
                      num_q_heads / num_kv_heads, 0, 0, 0, 0, 0, first_seq, 0, scale * kLog2e};
  a.hpp = a.group < units ? a.group : units;
  a.passes = (a.group + a.hpp - 1) / a.hpp;
  a.bq = units / a.hpp;
  a.xtiles = (max_tokens + a.bq - 1) / a.bq;
  const int64_t total = static_cast<int64_t>(a.xtiles) * num_kv_heads * a.passes * num_seqs;
  if (total > (1 << 30)) return TLF_E_SHAPE;
  a.total = static_cast<int32_t>(total);
  a.per_xcd = (a.total + 7) / 8;
  const dim3 grid(a.per_xcd * 8);
  hipStream_t s = static_cast<hipStream_t>(stream);
  switch (dc) {
    case 1: TLF_LAUNCH((pooled_prefill_kernel<1, 2>), grid, dim3(256), 0, s, a); break;
    case 2: TLF_LAUNCH((pooled_prefill_kernel<2, 2>), grid, dim3(256), 0, s, a); break;
    case 3: TLF_LAUNCH((pooled_prefill_kernel<3, 2>), grid, dim3(256), 0, s, a); break;
    case 4: TLF_LAUNCH((pooled_prefill_kernel<4, 2>), grid, dim3(256), 0, s, a); break;
    case 5: TLF_LAUNCH((pooled_prefill_kernel<5, 1>), grid, dim3(256), 0, s, a); break;
    case 6: TLF_LAUNCH((pooled_prefill_kernel<6, 1>), grid, dim3(256), 0, s, a); break;
    case 7: TLF_LAUNCH((pooled_prefill_kernel<7, 1>), grid, dim3(256), 0, s, a); break;
    default: TLF_LAUNCH((pooled_prefill_kernel<8, 1>), grid, dim3(256), 0, s, a); break;
  }
  return launch_status();
}
