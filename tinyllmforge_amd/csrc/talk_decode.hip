// Attention of talk_attn.h for single rows: decoded tokens, the rows of short portions, and every row in 32-bit mode.
//
//   talk_scores    scores of a row's keys and, per split of the keys, their maximum and sum of exponentials
//   talk_values    weights of all heads from the scores and the splits' maxima and sums, mixed by talk, times the values
//   talk_merge     sum over the splits
//
// The scores are written and read once (4 H bytes per key beside 2 G (D + Dv) of the caches); K and V are read once for all
// query heads that share them.  HBM bound.  bf16 on the matrix cores, a workgroup per (row, KV head, split), its four waves
// walk 32-key tiles:
//   S^T[key, head] = K . Q^T           K straight from memory in operand order
//   M^T[key, head] = W^T . talk^T      W^T (keys x all heads) from the scores in operand order, as a bf16 hi + lo pair
//   O^T[dim, head] += V^T . M^T        V through LDS rows of the wave's own and transpose reads, M as a pair
// The rows of the two 16-key halves are picked so that their accumulators are the next product's operand.  The kernels
// talk_scores_any / talk_values_any take any size and dtype on the vector ALU.
#include <algorithm>

#include "talk_attn.h"

namespace tlf {

constexpr int kTalkTileHeads = 128;       // heads the matrix-core kernel takes
constexpr int kTalkAnyHeads = 1024;

// The four waves' maximum and sum per head -> one, written as the split's.
template <int N>
__device__ __forceinline__ void talk_store_ml(const TalkRowsArgs &a, const float (*ml)[N][2], int64_t row, int split, int h0, int nh) {
  if (static_cast<int>(threadIdx.x) >= nh) return;
  const int h = threadIdx.x;
  float m = -INFINITY, l = 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) m = fmaxf(m, ml[w][h][0]);
#pragma unroll
  for (int w = 0; w < 4; ++w)
    if (ml[w][h][1] > 0.f) l += ml[w][h][1] * __builtin_amdgcn_exp2f(ml[w][h][0] - m);
  const int64_t at = (static_cast<int64_t>(split) * a.rows + row) * a.H + h0 + h;
  a.part_ml[at * 2] = m;
  a.part_ml[at * 2 + 1] = l;
}

template <int DC>
__global__ __launch_bounds__(256) void talk_scores_kernel(const TalkRowsArgs a) {
  __shared__ float ml[4][16][2];
  const SinkCache &c = a.c;
  const int64_t row = blockIdx.y;
  const int split = blockIdx.z, kvh = blockIdx.x / a.passes, pass = blockIdx.x % a.passes;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, n = lane & 15, g = lane >> 4;
  const int seq = a.row_seq ? a.row_seq[row] : static_cast<int>(row);
  int lo, hi;
  if (split >= talk_split(a, row, split, lo, hi)) return;      // workgroup uniform
  const int h0 = kvh * a.group + pass * a.per_pass, nh = min(a.per_pass, a.group - pass * a.per_pass);
  bf16x8 qf[DC];
  const unsigned short *qp = static_cast<const unsigned short *>(a.q) + (row * a.H + h0 + min(n, nh - 1)) * c.Dp + g * 8;
#pragma unroll
  for (int kc = 0; kc < DC; ++kc) {
    Pack16 t;
    t.u = kc * 32 < c.Dp && n < nh ? *reinterpret_cast<const uint4 *>(qp + kc * 32) : make_uint4(0, 0, 0, 0);
    qf[kc] = t.v;
  }
  float m = -INFINITY, l = 0.f;
  int j0 = lo + wave * 32;
  if (j0 < hi) {
    const int32_t *bt = c.bt + seq * c.bt_stride;
    uint4 kreg[2][DC];
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int kc = 0; kc < DC; ++kc) kreg[s][kc] = make_uint4(0, 0, 0, 0);
    const int krow = (n >> 2) * 8 + (n & 3);
    auto load_k = [&](int j, int page) __attribute__((always_inline)) {
      const int64_t r0 = sink_row(c, page, sink_page_of(c, j), kvh, j);
      const unsigned short *kp = static_cast<const unsigned short *>(c.k) + (r0 + krow) * c.Dp + g * 8;
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int kc = 0; kc < DC; ++kc)
          if (kc * 32 < c.Dp) kreg[s][kc] = load_nt_u4(kp + s * 4 * c.Dp + kc * 32);
    };
    float *sp = a.scores + (row * a.H + h0 + min(n, nh - 1)) * a.keys + g * 8;
    load_k(j0, bt[sink_page_of(c, j0)]);
    int next_page = bt[sink_page_of(c, min(j0 + 128, hi - 1))];
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
      if (j0 + 128 < hi) {                                // wave uniform
        load_k(j0 + 128, next_page);
        next_page = bt[sink_page_of(c, min(j0 + 256, hi - 1))];
      }
      // lane (n, g) holds head n, keys j0 + g * 8 + e
      float w[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) w[e] = e < 4 ? s0[e & 3] : s1[e & 3];
      if (j0 + 32 > hi) {
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = j0 + g * 8 + e < hi ? w[e] : -INFINITY;
      }
      if (n < nh) Elem<float>::st8(sp + j0, w);
      float mt = w[0];
#pragma unroll
      for (int e = 1; e < 8; ++e) mt = fmaxf(mt, w[e]);
      const float mn = fmaxf(m, mt);
      if (mn > -INFINITY) {                               // a lane's own maximum
        l *= __builtin_amdgcn_exp2f(m - mn);
        m = mn;
#pragma unroll
        for (int e = 0; e < 8; ++e) l += __builtin_amdgcn_exp2f(w[e] - m);
      }
    }
  }
  const float top = max_lanes_16_32_48(m);
  l = sum_lanes_16_32_48(l > 0.f ? l * __builtin_amdgcn_exp2f(m - top) : 0.f);
  if (g == 0) ml[wave][n][0] = top, ml[wave][n][1] = l;
  __syncthreads();
  talk_store_ml<16>(a, ml, row, split, h0, nh);
}

// Maximum and inverse sum over a row's splits for every head, [Hp] entries (past H: weight 0).
__device__ __forceinline__ void talk_totals(const TalkRowsArgs &a, int64_t row, int used, int Hp, float *sm, float *si) {
  for (int h = threadIdx.x; h < Hp; h += 256) {
    const float *p = a.part_ml + (row * a.H + min(h, a.H - 1)) * 2;
    const int64_t step = static_cast<int64_t>(a.rows) * a.H * 2;
    float m = -INFINITY, l = 0.f;
    for (int s0 = 0; s0 < used; s0 += 8) {               // eight splits' loads in flight
      float2 v[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = *reinterpret_cast<const float2 *>(p + min(s0 + i, used - 1) * step);
      float top = m;
#pragma unroll
      for (int i = 0; i < 8; ++i) top = fmaxf(top, v[i].x);
      l = l > 0.f ? l * __builtin_amdgcn_exp2f(m - top) : 0.f;
      m = top;
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (s0 + i < used && v[i].y > 0.f) l = fmaf(v[i].y, __builtin_amdgcn_exp2f(v[i].x - m), l);
    }
    sm[h] = m;
    si[h] = h < a.H && l > 0.f ? 1.0f / l : 0.f;
  }
}

template <int VC>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2))) void talk_values_kernel(const TalkRowsArgs a) {
  constexpr int VP = VC * 32, LV = VP + 16, LO = VP + 4;
  constexpr int kBytes = 4 * 32 * LV * 2 > 4 * 16 * LO * 4 ? 4 * 32 * LV * 2 : 4 * 16 * LO * 4;
  __shared__ __attribute__((aligned(16))) unsigned char lds[kBytes];
  __shared__ __attribute__((aligned(16))) unsigned short tk[16][kTalkTileHeads + 8];
  __shared__ __attribute__((aligned(16))) float sm[kTalkTileHeads], si[kTalkTileHeads];
  const SinkCache &c = a.c;
  const int64_t row = blockIdx.y;
  const int split = blockIdx.z, kvh = blockIdx.x / a.passes, pass = blockIdx.x % a.passes;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int seq = a.row_seq ? a.row_seq[row] : static_cast<int>(row);
  int lo, hi;
  const int used = talk_split(a, row, split, lo, hi);
  if (split >= max(used, 1)) return;                    // workgroup uniform; split 0 of a padding row writes its zeros
  const int h0 = kvh * a.group + pass * a.per_pass, nh = min(a.per_pass, a.group - pass * a.per_pass);
  const int Hp = (a.H + 31) & ~31;
  unsigned short(*Vs)[LV] = reinterpret_cast<unsigned short(*)[LV]>(lds) + wave * 32;
  floatx4 acc[2 * VC];
#pragma unroll
  for (int d = 0; d < 2 * VC; ++d) acc[d] = floatx4{0.f, 0.f, 0.f, 0.f};
  if (used) {
    for (int t = tid; t < 16 * Hp; t += 256) {
      const int h = t / Hp, k = t - h * Hp;
      tk[h][k] = h < nh && k < a.H ? static_cast<const unsigned short *>(a.talk)[(h0 + h) * a.H + k] : 0;
    }
    talk_totals(a, row, used, Hp, sm, si);
  }
  __syncthreads();
  int j0 = lo + wave * 32;
  if (j0 < hi) {
    const int32_t *bt = c.bt + seq * c.bt_stride;
    uint4 vreg[2 * VC];
#pragma unroll
    for (int p = 0; p < 2 * VC; ++p) vreg[p] = make_uint4(0, 0, 0, 0);
    auto load_v = [&](int j, int page) __attribute__((always_inline)) {
      const unsigned short *vp = static_cast<const unsigned short *>(c.v) + sink_row(c, page, sink_page_of(c, j), kvh, j) * c.Vp;
#pragma unroll
      for (int p = 0; p < 2 * VC; ++p) {
        const int item = lane + p * 64, r = item / (4 * VC), ch = item % (4 * VC);
        if (ch * 8 < c.Vp) vreg[p] = load_nt_u4(vp + r * c.Vp + ch * 8);
      }
    };
    const int krow = (n >> 2) * 8 + (n & 3);
    const float *sp = a.scores + row * a.H * a.keys + krow;
    float sc[2][8];
    auto load_s = [&](int j, int k0) __attribute__((always_inline)) {      // keys j + krow (+ 4), heads k0 + 8 g + e
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float *p = sp + static_cast<int64_t>(min(k0 + g * 8 + e, a.H - 1)) * a.keys + j;
        sc[0][e] = p[0];
        sc[1][e] = p[4];
      }
    };
    load_v(j0, bt[sink_page_of(c, j0)]);
    load_s(j0, 0);
    int next_page = bt[sink_page_of(c, min(j0 + 128, hi - 1))];
    for (; j0 < hi; j0 += 128) {
      const bool more = j0 + 128 < hi;                  // wave uniform
      wave_lds_fence();
#pragma unroll
      for (int p = 0; p < 2 * VC; ++p) {
        const int item = lane + p * 64, r = item / (4 * VC), ch = item % (4 * VC);
        *reinterpret_cast<uint4 *>(&Vs[r][ch * 8]) = vreg[p];
      }
      wave_lds_fence();
      if (more) {
        load_v(j0 + 128, next_page);
        next_page = bt[sink_page_of(c, min(j0 + 256, hi - 1))];
      }
      floatx4 m0 = floatx4{0.f, 0.f, 0.f, 0.f}, m1 = m0;
      for (int k0 = 0; k0 < Hp; k0 += 32) {
        if (k0) load_s(j0, k0);
        float mx[8], inv[8];
        Elem<float>::ld8(&sm[k0 + g * 8], mx);
        Elem<float>::ld8(&si[k0 + g * 8], inv);
        Pack16 t;
        t.u = *reinterpret_cast<const uint4 *>(&tk[n][k0 + g * 8]);
        float w0[8], w1[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          w0[e] = __builtin_amdgcn_exp2f(sc[0][e] - mx[e]) * inv[e];
          w1[e] = __builtin_amdgcn_exp2f(sc[1][e] - mx[e]) * inv[e];
        }
        bf16x8 ph, pl;
        talk_pair(w0, ph, pl);
        m0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph, t.v, m0, 0, 0, 0);
        m0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, t.v, m0, 0, 0, 0);
        talk_pair(w1, ph, pl);
        m1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph, t.v, m1, 0, 0, 0);
        m1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, t.v, m1, 0, 0, 0);
      }
      if (more) load_s(j0 + 128, 0);
      // lane (n, g): head n, keys j0 + g * 8 + e (keys past the end have weight 0)
      const float w[8] = {m0[0], m0[1], m0[2], m0[3], m1[0], m1[1], m1[2], m1[3]};
      bf16x8 ph, pl;
      talk_pair(w, ph, pl);
      const int vt = g * 8 + (n >> 2);
#pragma unroll
      for (int d = 0; d < 2 * VC; ++d) {
        const uint2 v0 = __builtin_bit_cast(uint2, talk_read_tr16(&Vs[vt][d * 16 + (n & 3) * 4]));
        const uint2 v1 = __builtin_bit_cast(uint2, talk_read_tr16(&Vs[vt + 4][d * 16 + (n & 3) * 4]));
        const bf16x8 vb = __builtin_bit_cast(bf16x8, make_uint4(v0.x, v0.y, v1.x, v1.y));
        acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, ph, acc[d], 0, 0, 0);
        acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, pl, acc[d], 0, 0, 0);
      }
    }
  }
  __syncthreads();                                      // every wave is done with its V rows
  float *ow = reinterpret_cast<float *>(lds);
#pragma unroll
  for (int d = 0; d < 2 * VC; ++d)
    *reinterpret_cast<float4 *>(&ow[(wave * 16 + n) * LO + d * 16 + g * 4]) = make_float4(acc[d][0], acc[d][1], acc[d][2], acc[d][3]);
  __syncthreads();
  for (int t = tid; t < nh * c.Vp; t += 256) {
    const int h = t / c.Vp, d = t - h * c.Vp;
    float o = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) o += ow[(w * 16 + h) * LO + d];
    if (used > 1) a.part_o[((static_cast<int64_t>(split) * a.rows + row) * a.H + h0 + h) * c.Vp + d] = o;
    else if (d < c.Dv) Elem<unsigned short>::st(static_cast<unsigned short *>(a.out) + row * a.ldo + static_cast<int64_t>(h0 + h) * c.Dv + d, o);
  }
}

// ---------------------------------------------------------------------------------------------------------------
// One workgroup per (row, head); a wave takes every fourth key, lanes its dimensions.
template <typename T>
__global__ __launch_bounds__(256) void talk_scores_any_kernel(const TalkRowsArgs a) {
  __shared__ float ml[4][1][2];
  const SinkCache &c = a.c;
  const int64_t row = blockIdx.y;
  const int h = blockIdx.x, kvh = h / a.group, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int seq = a.row_seq ? a.row_seq[row] : static_cast<int>(row);
  int lo, hi;
  if (talk_split(a, row, 0, lo, hi) == 0) return;         // one split: all keys
  constexpr int E = 8;                                    // D <= 512
  float q[E];
#pragma unroll
  for (int e = 0; e < E; ++e) q[e] = e * 64 + lane < c.Dp ? Elem<T>::ld(static_cast<const T *>(a.q) + (row * a.H + h) * c.Dp + e * 64 + lane) : 0.f;
  const int32_t *bt = c.bt + seq * c.bt_stride;
  float *sp = a.scores + (row * a.H + h) * a.keys;
  float m = -INFINITY, l = 0.f;
  for (int j = wave; j < hi; j += 4) {
    const int pg = sink_page_of(c, j);
    const T *kr = static_cast<const T *>(c.k) + sink_row(c, bt[pg], pg, kvh, j) * c.Dp;
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < E; ++e)
      if (e * 64 + lane < c.Dp) s = fmaf(q[e], Elem<T>::ld(kr + e * 64 + lane), s);
    s = wave_sum(s);
    if (lane == 0) sp[j] = s;
    const float mn = fmaxf(m, s);
    l = fmaf(l, exp2f(m - mn), exp2f(s - mn));
    m = mn;
  }
  if (lane == 0) ml[wave][0][0] = m, ml[wave][0][1] = l;
  __syncthreads();
  talk_store_ml<1>(a, ml, row, 0, h, 1);
}

// One workgroup per (row, head): mixed weights of 256 keys at a time, a thread each, then the values, a thread per dimension.
template <typename T>
__global__ __launch_bounds__(256) void talk_values_any_kernel(const TalkRowsArgs a) {
  __shared__ float sm[kTalkAnyHeads], si[kTalkAnyHeads], mix[256];
  const SinkCache &c = a.c;
  const int64_t row = blockIdx.y;
  const int h = blockIdx.x, kvh = h / a.group, tid = threadIdx.x;
  const int seq = a.row_seq ? a.row_seq[row] : static_cast<int>(row);
  int lo, hi;
  const int used = talk_split(a, row, 0, lo, hi);
  T *out = static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(h) * c.Dv;
  float o[2] = {0.f, 0.f};                               // Dv <= 512
  if (used) {
    talk_totals(a, row, used, a.H, sm, si);
    for (int k = tid; k < a.H; k += 256) si[k] *= Elem<T>::ld(static_cast<const T *>(a.talk) + static_cast<int64_t>(h) * a.H + k);
    const int32_t *bt = c.bt + seq * c.bt_stride;
    for (int j0 = 0; j0 < hi; j0 += 256) {
      __syncthreads();
      float w = 0.f;
      if (j0 + tid < hi)
        for (int k = 0; k < a.H; ++k) w = fmaf(exp2f(a.scores[(row * a.H + k) * a.keys + j0 + tid] - sm[k]), si[k], w);
      mix[tid] = w;
      __syncthreads();
      const int count = min(256, hi - j0);
      for (int j = 0; j < count; ++j) {
        const int pg = sink_page_of(c, j0 + j);
        const T *vr = static_cast<const T *>(c.v) + sink_row(c, bt[pg], pg, kvh, j0 + j) * c.Vp;
#pragma unroll
        for (int i = 0; i < 2; ++i)
          if (tid + i * 256 < c.Dv) o[i] = fmaf(mix[j], Elem<T>::ld(vr + tid + i * 256), o[i]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
    if (tid + i * 256 < c.Dv) Elem<T>::st(out + tid + i * 256, o[i]);
}

// The splits of a row added up: 4 value dimensions per thread.
__global__ __launch_bounds__(256) void talk_merge_kernel(const TalkRowsArgs a) {
  const int chunks = a.c.Vp / 4, Dv = a.c.Dv;
  const int64_t at = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (at >= static_cast<int64_t>(a.rows) * a.H * chunks) return;
  const int64_t rh = at / chunks, row = rh / a.H;
  const int d = static_cast<int>(at - rh * chunks) * 4, head = static_cast<int>(rh - row * a.H);
  if (d >= Dv) return;
  int lo, hi;
  const int used = talk_split(a, row, 0, lo, hi);
  if (used <= 1) return;                                // finished by its one workgroup
  const int64_t step = static_cast<int64_t>(a.rows) * a.H * a.c.Vp;
  const float *p = a.part_o + rh * a.c.Vp + d;
  float o[4] = {0.f, 0.f, 0.f, 0.f};
  for (int s0 = 0; s0 < used; s0 += 8) {                // eight splits' loads in flight
    float4 v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = *reinterpret_cast<const float4 *>(p + min(s0 + i, used - 1) * step);
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (s0 + i < used) { o[0] += v[i].x; o[1] += v[i].y; o[2] += v[i].z; o[3] += v[i].w; }
  }
  unsigned short *out = static_cast<unsigned short *>(a.out) + row * a.ldo + static_cast<int64_t>(head) * Dv + d;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (d + e < Dv) out[e] = float_to_bf16_bits(o[e]);
}

struct TalkPlan {
  bool tiles;
  int per_pass, passes, splits, keys;
  int64_t scores, ml, o;                 // floats of the workspace
};
TalkPlan talk_plan(int64_t rows, int H, int G, int dim, int vdim, int max_len, int dtype) {
  TalkPlan p{};
  const int group = H / G;
  p.tiles = dtype == TLF_DT_BF16 && dim <= 256 && vdim <= 256 && H <= kTalkTileHeads;
  p.per_pass = p.tiles ? std::min(group, 16) : 1;
  p.passes = (group + p.per_pass - 1) / p.per_pass;
  const int64_t groups = rows * G * p.passes, want = (2048 + groups - 1) / groups, most = (max_len + 127) / 128;
  p.splits = p.tiles ? static_cast<int>(std::max<int64_t>(1, std::min<int64_t>({want, most, 64}))) : 1;
  p.keys = (max_len + 63) / 64 * 64;
  p.scores = rows * H * p.keys;
  p.ml = p.splits * rows * H * 2;
  p.o = p.splits > 1 ? p.splits * rows * H * ((vdim + 31) / 32 * 32) : 0;
  return p;
}

}  // namespace tlf

extern "C" size_t tlf_talk_attn_rows_workspace_bytes(int32_t rows, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim,
                                                     int32_t max_len, int32_t dtype) {
  if (rows <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || dim <= 0 || vdim <= 0 || max_len <= 0) return 0;
  const tlf::TalkPlan p = tlf::talk_plan(rows, heads, kv_heads, dim, vdim, max_len, dtype);
  return static_cast<size_t>(p.scores + p.ml + p.o) * 4;
}

extern "C" int tlf_talk_attn_rows(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables,
                                  int64_t bt_stride, const int64_t *positions, const int32_t *slot_mapping, const int32_t *row_seq,
                                  const void *talk, void *out, int64_t out_stride, int32_t rows, int32_t heads, int32_t kv_heads,
                                  int32_t dim, int32_t vdim, int32_t block_size, int32_t max_len, int64_t num_pages, int32_t dtype,
                                  void *workspace, size_t workspace_bytes, void *stream) {
  using namespace tlf;
  if (rows < 0 || rows > 65535 || heads <= 0 || heads > kTalkAnyHeads || kv_heads <= 0 || heads % kv_heads || max_len <= 0) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (out_stride < static_cast<int64_t>(heads) * vdim) return TLF_E_SHAPE;
  if (rows == 0) return TLF_OK;
  TalkRowsArgs a{};
  if (int rc = sink_cache_make(a.c, k_cache, v_cache, block_tables, bt_stride, block_size, kv_heads, dim, vdim, num_pages)) return rc;
  if (!q || !block_tables || !positions || !slot_mapping || !talk || !out) return TLF_E_NULL;
  if (!aligned16(q)) return TLF_E_ALIGN;
  if (bt_stride < (max_len + block_size - 1) / block_size) return TLF_E_SHAPE;
  const TalkPlan p = talk_plan(rows, heads, kv_heads, dim, vdim, max_len, dtype);
  if (!workspace || workspace_bytes < static_cast<size_t>(p.scores + p.ml + p.o) * 4) return TLF_E_WORKSPACE;
  if (!aligned16(workspace)) return TLF_E_ALIGN;
  a.q = q; a.talk = talk; a.positions = positions; a.slots = slot_mapping; a.row_seq = row_seq; a.out = out; a.ldo = out_stride;
  a.keys = p.keys; a.rows = rows; a.H = heads; a.group = heads / kv_heads; a.per_pass = p.per_pass; a.passes = p.passes;
  a.splits = p.splits; a.max_len = max_len;
  const int64_t wgs = static_cast<int64_t>(rows) * kv_heads * p.passes;
  a.least = !p.tiles ? p.keys : wgs >= 256 ? 512 : 128;          // short pieces only where workgroups are few
  a.scores = static_cast<float *>(workspace);
  a.part_o = a.scores + p.scores;
  a.part_ml = a.part_o + p.o;
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (!p.tiles) {
    const dim3 grid(heads, rows);
    if (dtype == TLF_DT_BF16) {
      TLF_LAUNCH((talk_scores_any_kernel<unsigned short>), grid, dim3(256), 0, s, a);
      TLF_LAUNCH((talk_values_any_kernel<unsigned short>), grid, dim3(256), 0, s, a);
    } else {
      TLF_LAUNCH((talk_scores_any_kernel<float>), grid, dim3(256), 0, s, a);
      TLF_LAUNCH((talk_values_any_kernel<float>), grid, dim3(256), 0, s, a);
    }
    return launch_status();
  }
  const dim3 grid(kv_heads * p.passes, rows, p.splits);         // splits outermost: the unused ones come last, on all XCDs alike
  const int dc = a.c.Dp / 32, vc = a.c.Vp / 32;
  if (dc <= 1) TLF_LAUNCH((talk_scores_kernel<1>), grid, dim3(256), 0, s, a);
  else if (dc <= 2) TLF_LAUNCH((talk_scores_kernel<2>), grid, dim3(256), 0, s, a);
  else if (dc <= 4) TLF_LAUNCH((talk_scores_kernel<4>), grid, dim3(256), 0, s, a);
  else TLF_LAUNCH((talk_scores_kernel<8>), grid, dim3(256), 0, s, a);
  if (vc <= 1) TLF_LAUNCH((talk_values_kernel<1>), grid, dim3(256), 0, s, a);
  else if (vc <= 2) TLF_LAUNCH((talk_values_kernel<2>), grid, dim3(256), 0, s, a);
  else if (vc <= 4) TLF_LAUNCH((talk_values_kernel<4>), grid, dim3(256), 0, s, a);
  else TLF_LAUNCH((talk_values_kernel<8>), grid, dim3(256), 0, s, a);
  if (p.splits > 1) {
    const int64_t items = static_cast<int64_t>(rows) * heads * (a.c.Vp / 4);
    TLF_LAUNCH(talk_merge_kernel, dim3(static_cast<unsigned>((items + 255) / 256)), dim3(256), 0, s, a);
  }
  return launch_status();
}
