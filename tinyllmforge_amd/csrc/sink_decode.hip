// Attention of sink_attn.h for single rows: decoded tokens, the rows of short portions, and every row in 32-bit mode.
//
// A workgroup owns one row, one KV head (up to 16 of its query heads at a time) and a split of the keys; the splits' partial
// results are joined by sink_merge_kernel, which also adds the sink and applies the gate.  HBM bound: a cache row is read once
// for all query heads that share it.
//
//   sink_tile_kernel   bf16, matrix cores.  A wave walks 32-key tiles with an online softmax of its own:
//     S^T[key, head] = K . Q^T      v_mfma_f32_16x16x32_bf16, K straight from memory in operand order: the rows of the two
//                                   16-key halves are picked so that their accumulators are the next product's operand
//     O^T[dim, head] += V^T . P^T   V through LDS rows of the wave's own and transpose reads; P as a bf16 hi + lo pair
//     The next tile's loads are issued as soon as the registers are free.  The four waves meet once, at the end.
//   sink_rows_kernel   any size and dtype on the vector ALU, 16 bytes (bf16) of a row per lane.
#include <algorithm>

#include "sink_attn.h"

namespace tlf {

struct SinkRowsArgs {
  SinkCache c;
  float cap_log2;            // cap * log2(e), 0: none
  const void *q;             // [rows, H, Dp]
  const void *sink;          // [H] or NULL
  const void *gate;          // [rows, ldg] or NULL: H * Dv columns
  const int64_t *positions;  // [rows]
  const int32_t *slots;      // [rows], negative: padding row
  const int32_t *row_seq;    // [rows] or NULL: row r belongs to sequence r
  void *out;                 // [rows, ldo]
  int64_t ldo, ldg;
  float *part_o;             // [splits, rows, H, Vp]
  float *part_ml;            // [splits, rows, H, 2]: maximum (log 2 units), sum
  int32_t rows, H, group, per_pass, passes, splits, least, max_len;
};

__device__ __forceinline__ shortx4 sink_read_tr16(const unsigned short *p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p));
}

// A row's keys are cut into pieces of equal length, a multiple of 64 and at least `least`, so short rows use few of the splits.
// Split `split` has keys [lo, hi); returns how many splits the row uses, 0 for a padding row.
__device__ __forceinline__ int sink_split(const SinkRowsArgs &a, int64_t row, int split, int &lo, int &hi) {
  const int64_t i = a.positions[row];
  lo = hi = 0;
  if (a.slots[row] < 0 || i < 0 || i >= a.max_len) return 0;
  const int total = static_cast<int>(i) + 1, per = max(((total + a.splits - 1) / a.splits + 63) & ~63, a.least);
  lo = min(total, split * per);
  hi = min(total, lo + per);
  return (total + per - 1) / per;
}
// Row r's output element: mix / denominator, the sink in the denominator, the gate on top.
template <typename T>
__device__ __forceinline__ float sink_finish(const SinkRowsArgs &a, int64_t row, int head, int d, float o, float m, float l) {
  const float sk = a.sink ? Elem<T>::ld(static_cast<const T *>(a.sink) + head) * kSinkLog2e : -INFINITY;
  const float top = fmaxf(m, sk);
  const float f = __builtin_amdgcn_exp2f(m - top);
  const float g = a.gate ? sigmoid_f32(Elem<T>::ld(static_cast<const T *>(a.gate) + row * a.ldg + static_cast<int64_t>(head) * a.c.Dv + d)) : 1.f;
  return o * f / (l * f + __builtin_amdgcn_exp2f(sk - top)) * g;
}

// Four waves' (m, l, O) in LDS -> one; written as the row's result or as a partial one.  O[wave][head][dim], rows of `ldw`.
template <typename T>
__device__ __forceinline__ void sink_join_waves(const SinkRowsArgs &a, const float *ow, int ldw, int heads_w, const float (*ml)[16][2],
                                                int64_t row, int split, int h0, int nh, int used) {
  const int Vp = a.c.Vp;
  for (int t = threadIdx.x; t < nh * Vp; t += 256) {
    const int g = t / Vp, d = t - g * Vp;
    const int head = h0 + g;
    float m = -INFINITY, l = 0.f, o = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) m = fmaxf(m, ml[w][g][0]);
    if (m > -INFINITY) {
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        const float f = __builtin_amdgcn_exp2f(ml[w][g][0] - m);
        l += f * ml[w][g][1];
        if (f > 0.f) o += f * ow[(w * heads_w + g) * ldw + d];
      }
    }
    if (used > 1) {
      const int64_t at = (static_cast<int64_t>(split) * a.rows + row) * a.H + head;
      if (l > 0.f) a.part_o[at * Vp + d] = o;
      if (d == 0) a.part_ml[at * 2] = m, a.part_ml[at * 2 + 1] = l;
    } else if (d < a.c.Dv) {
      Elem<T>::st(static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(head) * a.c.Dv + d,
                  used ? sink_finish<T>(a, row, head, d, o, m, l) : 0.f);
    }
  }
}

// DC, VC: key and value dimensions in units of 32, rounded up to what is instantiated
template <int DC, int VC, bool CAP>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2))) void sink_tile_kernel(const SinkRowsArgs a) {
  constexpr int VP = VC * 32, LV = VP + 16, LO = VP + 4;
  constexpr int kBytes = 4 * 32 * LV * 2 > 4 * 16 * LO * 4 ? 4 * 32 * LV * 2 : 4 * 16 * LO * 4;
  __shared__ __attribute__((aligned(16))) unsigned char lds[kBytes];
  __shared__ float ml[4][16][2];
  const SinkCache &c = a.c;
  const int64_t row = blockIdx.y;
  const int split = blockIdx.z, kvh = blockIdx.x / a.passes, pass = blockIdx.x % a.passes;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int seq = a.row_seq ? a.row_seq[row] : static_cast<int>(row);
  int lo, hi;
  const int used = sink_split(a, row, split, lo, hi);
  if (split >= max(used, 1)) return;                    // workgroup uniform; split 0 of a padding row writes its zeros
  const int h0 = kvh * a.group + pass * a.per_pass, nh = min(a.per_pass, a.group - pass * a.per_pass);
  unsigned short(*Vs)[LV] = reinterpret_cast<unsigned short(*)[LV]>(lds) + wave * 32;

  bf16x8 qf[DC];
  const unsigned short *qp = static_cast<const unsigned short *>(a.q) + (row * a.H + h0 + min(n, nh - 1)) * c.Dp + g * 8;
#pragma unroll
  for (int kc = 0; kc < DC; ++kc) {
    Pack16 t;
    t.u = kc * 32 < c.Dp && n < nh ? *reinterpret_cast<const uint4 *>(qp + kc * 32) : make_uint4(0, 0, 0, 0);
    qf[kc] = t.v;
  }
  floatx4 acc[2 * VC];
#pragma unroll
  for (int d = 0; d < 2 * VC; ++d) acc[d] = floatx4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;

  if (lo + wave * 32 < hi) {
    const int32_t *bt = c.bt + seq * c.bt_stride;
    uint4 kreg[2][DC], vreg[2 * VC];
    const int krow = (n >> 2) * 8 + (n & 3);
    // V: 4 VC pieces of 16 bytes per row
    auto tile_row = [&](int j0, int page) __attribute__((always_inline)) { return sink_row(c, page, sink_page_of(c, j0), kvh, j0); };
    auto load_k = [&](int64_t r0) __attribute__((always_inline)) {
      const unsigned short *kp = static_cast<const unsigned short *>(c.k) + (r0 + krow) * c.Dp + g * 8;
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int kc = 0; kc < DC; ++kc)
          if (kc * 32 < c.Dp) kreg[s][kc] = load_nt_u4(kp + s * 4 * c.Dp + kc * 32);
    };
    auto load_v = [&](int64_t r0) __attribute__((always_inline)) {
      const unsigned short *vp = static_cast<const unsigned short *>(c.v) + r0 * c.Vp;
#pragma unroll
      for (int p = 0; p < 2 * VC; ++p) {
        const int item = lane + p * 64, r = item / (4 * VC), ch = item % (4 * VC);
        if (ch * 8 < c.Vp) vreg[p] = load_nt_u4(vp + r * c.Vp + ch * 8);
      }
    };
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int kc = 0; kc < DC; ++kc) kreg[s][kc] = make_uint4(0, 0, 0, 0);
#pragma unroll
    for (int p = 0; p < 2 * VC; ++p) vreg[p] = make_uint4(0, 0, 0, 0);
    int j0 = lo + wave * 32;
    const int64_t first = tile_row(j0, bt[sink_page_of(c, j0)]);
    int next_page = bt[sink_page_of(c, min(j0 + 128, hi - 1))];
    load_k(first);
    load_v(first);
    for (; j0 < hi; j0 += 128) {
      floatx4 s0 = floatx4{0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
      for (int kc = 0; kc < DC; ++kc) {
        Pack16 k0, k1;
        k0.u = kreg[0][kc];
        k1.u = kreg[1][kc];
        s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0.v, qf[kc], s0, 0, 0, 0);
        s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1.v, qf[kc], s1, 0, 0, 0);
      }
      wave_lds_fence();
#pragma unroll
      for (int p = 0; p < 2 * VC; ++p) {
        const int item = lane + p * 64, r = item / (4 * VC), ch = item % (4 * VC);
        *reinterpret_cast<uint4 *>(&Vs[r][ch * 8]) = vreg[p];
      }
      wave_lds_fence();
      if (j0 + 128 < hi) {                              // wave uniform
        const int64_t r0 = tile_row(j0 + 128, next_page);
        next_page = bt[sink_page_of(c, min(j0 + 256, hi - 1))];
        load_k(r0);
        load_v(r0);
      }
      // lane (n, g) holds head n, keys j0 + g * 8 + e
      float w[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) w[e] = sink_score_log2<CAP>(e < 4 ? s0[e & 3] : s1[e & 3], a.cap_log2);
      if (j0 + 32 > hi) {
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = j0 + g * 8 + e < hi ? w[e] : -INFINITY;
      }
      float mt = w[0];
#pragma unroll
      for (int e = 1; e < 8; ++e) mt = fmaxf(mt, w[e]);
      mt = max_lanes_16_32_48(mt);
      // the maximum is moved only when it has grown by a factor of 256
      const bool grown = mt > m + 8.f;
      const float back = grown ? __builtin_amdgcn_exp2f(m - mt) : 1.f;
      m = grown ? mt : m;
      l *= back;
#pragma unroll
      for (int d = 0; d < VC; ++d) sink_rescale(acc[2 * d], acc[2 * d + 1], back);
      unsigned int ph[4], pl[4];
#pragma unroll
      for (int e = 0; e < 8; ++e) w[e] = __builtin_amdgcn_exp2f(w[e] - m);
      l += ((w[0] + w[1]) + (w[2] + w[3])) + ((w[4] + w[5]) + (w[6] + w[7]));
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        ph[e] = pack_bf16x2(w[2 * e], w[2 * e + 1]);
        pl[e] = pack_bf16x2(w[2 * e] - __uint_as_float(ph[e] << 16), w[2 * e + 1] - __uint_as_float(ph[e] & 0xffff0000u));
      }
      const bf16x8 hi8 = __builtin_bit_cast(bf16x8, make_uint4(ph[0], ph[1], ph[2], ph[3]));
      const bf16x8 lo8 = __builtin_bit_cast(bf16x8, make_uint4(pl[0], pl[1], pl[2], pl[3]));
      const int vt = g * 8 + (n >> 2);
#pragma unroll
      for (int d = 0; d < 2 * VC; ++d) {
        const uint2 v0 = __builtin_bit_cast(uint2, sink_read_tr16(&Vs[vt][d * 16 + (n & 3) * 4]));
        const uint2 v1 = __builtin_bit_cast(uint2, sink_read_tr16(&Vs[vt + 4][d * 16 + (n & 3) * 4]));
        const bf16x8 vb = __builtin_bit_cast(bf16x8, make_uint4(v0.x, v0.y, v1.x, v1.y));
        acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, hi8, acc[d], 0, 0, 0);
        acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, lo8, acc[d], 0, 0, 0);
      }
    }
    l = sum_lanes_16_32_48(l);
  }
  __syncthreads();                                      // every wave is done with its V rows
  float *ow = reinterpret_cast<float *>(lds);
#pragma unroll
  for (int d = 0; d < 2 * VC; ++d)
    *reinterpret_cast<float4 *>(&ow[(wave * 16 + n) * LO + d * 16 + g * 4]) = make_float4(acc[d][0], acc[d][1], acc[d][2], acc[d][3]);
  if (g == 0) ml[wave][n][0] = m, ml[wave][n][1] = l;
  __syncthreads();
  sink_join_waves<unsigned short>(a, ow, LO, 16, ml, row, split, h0, nh, used);
}

// LPK lanes per key; every group of LPK lanes keeps its own running maximum, sum and mix for GH heads.
template <typename T, int LPK, int GH>
__global__ __launch_bounds__(256) void sink_rows_kernel(const SinkRowsArgs a) {
  constexpr int KPW = 64 / LPK, U = 2;
  __shared__ __attribute__((aligned(16))) float red[4][GH][LPK * 8];
  __shared__ float ml[4][16][2];
  const SinkCache &c = a.c;
  const int64_t row = blockIdx.y;
  const int split = blockIdx.z, kvh = blockIdx.x / a.passes, pass = blockIdx.x % a.passes;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, sub = lane / LPK, dl = lane % LPK;
  const int seq = a.row_seq ? a.row_seq[row] : static_cast<int>(row);
  int lo, hi;
  const int used = sink_split(a, row, split, lo, hi);
  if (split >= max(used, 1)) return;                    // workgroup uniform; split 0 of a padding row writes its zeros
  const int h0 = kvh * a.group + pass * a.per_pass, nh = min(a.per_pass, a.group - pass * a.per_pass);
  const bool k_ok = dl * 8 < c.Dp, v_ok = dl * 8 < c.Vp;
  const int kcol = k_ok ? dl * 8 : 0, vcol = v_ok ? dl * 8 : 0;
  float qf[GH][8], o[GH][8], m[GH], l[GH];
#pragma unroll
  for (int g = 0; g < GH; ++g) {
    m[g] = -INFINITY;
    l[g] = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) qf[g][e] = o[g][e] = 0.f;
    if (g < nh && k_ok) Elem<T>::ld8(static_cast<const T *>(a.q) + (row * a.H + h0 + g) * c.Dp + kcol, qf[g]);
  }
  const int32_t *bt = c.bt + seq * c.bt_stride;
  for (int base = lo + wave * U * KPW; base < hi; base += 4 * U * KPW) {
    typename Elem<T>::Raw8 kr[U], vr[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int j = min(base + u * KPW + sub, hi - 1), pg = sink_page_of(c, j);
      const int64_t r = sink_row(c, bt[pg], pg, kvh, j);
      Elem<T>::raw8(static_cast<const T *>(c.k) + r * c.Dp + kcol, kr[u]);
      Elem<T>::raw8(static_cast<const T *>(c.v) + r * c.Vp + vcol, vr[u]);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const bool ok = base + u * KPW + sub < hi;
      float kf[8], vf[8];
      Elem<T>::cvt8(kr[u], kf);
      Elem<T>::cvt8(vr[u], vf);
#pragma unroll
      for (int g = 0; g < GH; ++g) {
        float s = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) s = fmaf(qf[g][e], kf[e], s);
        s = group_sum<LPK>(k_ok ? s : 0.f);
        if (a.cap_log2 > 0.f) s = a.cap_log2 * tanhf(s * (0.5f / kSinkLog2e));
        if (ok) {
          const float mn = fmaxf(m[g], s);
          const float f = __builtin_amdgcn_exp2f(m[g] - mn), w = __builtin_amdgcn_exp2f(s - mn);
          m[g] = mn;
          l[g] = fmaf(l[g], f, w);
#pragma unroll
          for (int e = 0; e < 8; ++e) o[g][e] = fmaf(o[g][e], f, w * vf[e]);
        }
      }
    }
  }
  // keys side by side in a wave, then the four waves
#pragma unroll
  for (int g = 0; g < GH; ++g) {
    float top = m[g];
#pragma unroll
    for (int s = LPK; s < 64; s <<= 1) top = fmaxf(top, __shfl_xor(top, s, 64));
    const float f = m[g] > -INFINITY ? __builtin_amdgcn_exp2f(m[g] - top) : 0.f;
    l[g] *= f;
#pragma unroll
    for (int s = LPK; s < 64; s <<= 1) l[g] += __shfl_xor(l[g], s, 64);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      o[g][e] *= f;
#pragma unroll
      for (int s = LPK; s < 64; s <<= 1) o[g][e] += __shfl_xor(o[g][e], s, 64);
      if (sub == 0) red[wave][g][dl * 8 + e] = o[g][e];
    }
    if (lane == 0) ml[wave][g][0] = top, ml[wave][g][1] = l[g];
  }
  __syncthreads();
  sink_join_waves<T>(a, &red[0][0][0], LPK * 8, GH, ml, row, split, h0, nh, used);
}

// The splits of a row joined: 4 value dimensions per thread.
template <typename T>
__global__ __launch_bounds__(256) void sink_merge_kernel(const SinkRowsArgs a) {
  const int chunks = a.c.Vp / 4, Dv = a.c.Dv;
  const int64_t at = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (at >= static_cast<int64_t>(a.rows) * a.H * chunks) return;
  const int64_t rh = at / chunks, row = rh / a.H;
  const int d = static_cast<int>(at - rh * chunks) * 4, head = static_cast<int>(rh - row * a.H);
  if (d >= Dv) return;
  const int64_t plane = static_cast<int64_t>(a.rows) * a.H;
  T *out = static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(head) * Dv + d;
  int lo, hi;
  const int used = sink_split(a, row, 0, lo, hi);
  if (used <= 1) return;                                // finished by its one workgroup
  float m = -INFINITY, l = 0.f, o[4] = {0.f, 0.f, 0.f, 0.f};
  for (int s0 = 0; s0 < used; s0 += 8) {               // eight splits' loads in flight
    float2 ml[8];
    float4 p[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int64_t at = min(s0 + i, used - 1) * plane + rh;
      ml[i] = *reinterpret_cast<const float2 *>(a.part_ml + at * 2);
      p[i] = *reinterpret_cast<const float4 *>(a.part_o + at * a.c.Vp + d);
    }
    float top = m;
#pragma unroll
    for (int i = 0; i < 8; ++i) top = fmaxf(top, ml[i].x);
    const float back = __builtin_amdgcn_exp2f(m - top);
    m = top;
    l *= back;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] *= back;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      if (s0 + i < used && ml[i].y > 0.f) {
        const float f = __builtin_amdgcn_exp2f(ml[i].x - m);
        l = fmaf(f, ml[i].y, l);
        o[0] = fmaf(f, p[i].x, o[0]); o[1] = fmaf(f, p[i].y, o[1]);
        o[2] = fmaf(f, p[i].z, o[2]); o[3] = fmaf(f, p[i].w, o[3]);
      }
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (d + e < Dv) Elem<T>::st(out + e, sink_finish<T>(a, row, head, d + e, o[e], m, l));
}

int sink_splits(int64_t groups, int64_t max_keys) {
  const int64_t want = (2048 + groups - 1) / groups, most = (max_keys + 127) / 128;
  return static_cast<int>(std::max<int64_t>(1, std::min<int64_t>({want, most, 64})));
}
bool sink_tiles(const SinkCache &c, int32_t dtype) { return dtype == TLF_DT_BF16 && c.Dp <= 256 && c.Vp <= 256; }
int sink_heads_per_pass(int group, bool tiles) {
  if (tiles) return group < 16 ? group : 16;
  return group <= 1 ? 1 : group <= 2 ? 2 : 4;
}
size_t sink_rows_bytes(int64_t splits, int64_t rows, int64_t H, int64_t Vp) { return splits > 1 ? splits * rows * H * (Vp + 2) * 4 : 0; }

template <typename T>
int launch_sink_rows(const SinkRowsArgs &a, hipStream_t s) {
  const dim3 grid(a.c.G * a.passes, a.rows, a.splits);      // splits outermost: the unused ones come last, on all XCDs alike
  const int most = a.c.Dp > a.c.Vp ? a.c.Dp : a.c.Vp;
#define TLF_SR(LPK, GH) TLF_LAUNCH((sink_rows_kernel<T, LPK, GH>), grid, dim3(256), 0, s, a)
#define TLF_SR_GH(LPK)                    \
  do {                                    \
    if (a.per_pass == 1) TLF_SR(LPK, 1);  \
    else if (a.per_pass == 2) TLF_SR(LPK, 2); \
    else TLF_SR(LPK, 4);                  \
  } while (0)
  if (most <= 32) TLF_SR_GH(4);
  else if (most <= 64) TLF_SR_GH(8);
  else if (most <= 128) TLF_SR_GH(16);
  else if (most <= 256) TLF_SR_GH(32);
  else TLF_SR_GH(64);
#undef TLF_SR_GH
#undef TLF_SR
  return launch_status();
}
int launch_sink_tiles(const SinkRowsArgs &a, hipStream_t s) {
  const dim3 grid(a.c.G * a.passes, a.rows, a.splits);      // splits outermost: the unused ones come last, on all XCDs alike
  const int dc = a.c.Dp / 32, vc = a.c.Vp / 32;
#define TLF_ST(DC, VC)                                                                                   \
  do {                                                                                                   \
    if (a.cap_log2 > 0.f) TLF_LAUNCH((sink_tile_kernel<DC, VC, true>), grid, dim3(256), 0, s, a);  \
    else TLF_LAUNCH((sink_tile_kernel<DC, VC, false>), grid, dim3(256), 0, s, a);                        \
  } while (0)
#define TLF_ST_V(DC)                \
  do {                              \
    if (vc <= 1) TLF_ST(DC, 1);     \
    else if (vc <= 2) TLF_ST(DC, 2); \
    else if (vc <= 4) TLF_ST(DC, 4); \
    else TLF_ST(DC, 8);             \
  } while (0)
  if (dc <= 1) TLF_ST_V(1);
  else if (dc <= 2) TLF_ST_V(2);
  else if (dc <= 4) TLF_ST_V(4);
  else if (dc <= 6) TLF_ST_V(6);
  else TLF_ST_V(8);
#undef TLF_ST_V
#undef TLF_ST
  return launch_status();
}

}  // namespace tlf

extern "C" size_t tlf_sink_attn_rows_workspace_bytes(int32_t rows, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim,
                                                     int32_t max_len, int32_t dtype) {
  using namespace tlf;
  if (rows <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || dim <= 0 || vdim <= 0 || max_len <= 0) return 0;
  SinkCache c{};
  c.Dp = (dim + 31) / 32 * 32; c.Vp = (vdim + 31) / 32 * 32;
  const int group = heads / kv_heads, per = sink_heads_per_pass(group, sink_tiles(c, dtype)), passes = (group + per - 1) / per;
  return sink_rows_bytes(sink_splits(static_cast<int64_t>(rows) * kv_heads * passes, max_len), rows, heads, c.Vp);
}

extern "C" int tlf_sink_attn_rows(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables,
                                  int64_t bt_stride, const int64_t *positions, const int32_t *slot_mapping, const int32_t *row_seq,
                                  const void *sink, const void *gate, int64_t gate_stride, void *out, int64_t out_stride,
                                  int32_t rows, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size,
                                  int32_t max_len, int64_t num_pages, float cap, int32_t dtype, void *workspace,
                                  size_t workspace_bytes, void *stream) {
  using namespace tlf;
  if (rows < 0 || rows > 65535 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || max_len <= 0 || cap < 0.f) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  const int64_t cols = static_cast<int64_t>(heads) * vdim;
  if (out_stride < cols || (gate && gate_stride < cols)) return TLF_E_SHAPE;
  if (rows == 0) return TLF_OK;
  SinkRowsArgs a{};
  if (int rc = sink_cache_make(a.c, k_cache, v_cache, block_tables, bt_stride, block_size, kv_heads, dim, vdim, num_pages)) return rc;
  if (!q || !block_tables || !positions || !slot_mapping || !out) return TLF_E_NULL;
  if (!aligned16(q)) return TLF_E_ALIGN;
  if (bt_stride < (max_len + block_size - 1) / block_size) return TLF_E_SHAPE;
  a.cap_log2 = cap * kSinkLog2e;
  a.q = q; a.sink = sink; a.gate = gate; a.positions = positions; a.slots = slot_mapping; a.row_seq = row_seq; a.out = out;
  a.ldo = out_stride; a.ldg = gate_stride; a.rows = rows; a.H = heads; a.group = heads / kv_heads; a.max_len = max_len;
  const bool tiles = sink_tiles(a.c, dtype);
  a.per_pass = sink_heads_per_pass(a.group, tiles);
  a.passes = (a.group + a.per_pass - 1) / a.per_pass;
  if (static_cast<int64_t>(kv_heads) * a.passes > 65535) return TLF_E_SHAPE;
  a.splits = sink_splits(static_cast<int64_t>(rows) * kv_heads * a.passes, max_len);
  a.least = static_cast<int64_t>(rows) * kv_heads * a.passes >= 256 ? 512 : 128;      // short pieces only where workgroups are few
  if (a.splits > 1) {
    if (!workspace || workspace_bytes < sink_rows_bytes(a.splits, rows, heads, a.c.Vp)) return TLF_E_WORKSPACE;
    if (!aligned16(workspace)) return TLF_E_ALIGN;
    a.part_o = static_cast<float *>(workspace);
    a.part_ml = a.part_o + static_cast<int64_t>(a.splits) * rows * heads * a.c.Vp;
  }
  hipStream_t s = static_cast<hipStream_t>(stream);
  int rc = tiles ? launch_sink_tiles(a, s) : dtype == TLF_DT_BF16 ? launch_sink_rows<unsigned short>(a, s) : launch_sink_rows<float>(a, s);
  if (rc != TLF_OK || a.splits == 1) return rc;
  const int64_t items = static_cast<int64_t>(rows) * heads * (a.c.Vp / 4);
  const dim3 grid(static_cast<unsigned>((items + 255) / 256));
  if (dtype == TLF_DT_BF16) TLF_LAUNCH((sink_merge_kernel<unsigned short>), grid, dim3(256), 0, s, a);
  else TLF_LAUNCH((sink_merge_kernel<float>), grid, dim3(256), 0, s, a);
  return launch_status();
}
