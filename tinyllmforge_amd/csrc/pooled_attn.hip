// Sigmoid attention over a sliding window plus pooled blocks (see pooled_attn.h for the geometry): what happens
// between the projections and the output projection, except the matrix-core kernel for prompt portions
// (pooled_prefill.hip).
//
//   attn_prep_kernel    projection row [q | k | gate] -> biases, V store (the projected key), interleaved RoPE on the
//                       first rot_dims dimensions, unit RMS per head, K store, q, sigmoid of the per-head gate
//   pool_blocks_kernel  means of the blocks that a step's prompt portions complete
//   rows_kernel         one workgroup per (query row, KV head, split of the keys): decode, and every row in 32-bit mode
//   rows_merge_kernel   sum of the splits (the weights are not normalised, so partial outputs just add) and the gate
#include <algorithm>

#include "pooled_attn.h"

namespace tlf {

int pooled_cache_check(const PooledCache &c, int32_t dtype) {
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (!c.k || !c.v || !c.pk || !c.pv || !c.bt) return TLF_E_NULL;
  if (c.bs <= 0 || c.bs % 64 || c.pool <= 0 || c.size <= 0 || c.G <= 0 || c.pages <= 0) return TLF_E_SHAPE;
  if (c.D <= 0 || c.D > 256 || c.Dp != (c.D + 31) / 32 * 32) return TLF_E_SHAPE;
  if (!aligned16(c.k) || !aligned16(c.v) || !aligned16(c.pk) || !aligned16(c.pv)) return TLF_E_ALIGN;
  return TLF_OK;
}

// ---------------------------------------------------------------------------------------------------------------
struct AttnPrepArgs {
  const void *proj;        // [n, ld]: q heads, k heads, one gate value per q head
  Partials part;           // or its partial sums
  int64_t ld;
  const void *q_bias, *k_bias;
  const int64_t *positions;
  const float *cos_sin;    // [max_pos, rot_dims]: cos of the pairs, then sin
  int32_t max_pos, rot_dims;
  const int32_t *slots;    // cache row per token, negative: no store
  int64_t num_slots;
  void *q_out;             // [n, H, Dp]
  void *k_cache, *v_cache; // [slots, G, Dp]
  float *gate;             // [n, H]
  int32_t n, H, G, D, Dp;
  float eps;
  int32_t vec;             // rows may be read 8 elements at a time
};

// 16 lanes per (token, head), any size; head H + G is the token's gate row.
template <typename T, int MAXC>
__global__ __launch_bounds__(256) void attn_prep_kernel(const AttnPrepArgs a) {
  const int heads = a.H + a.G + 1;
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 16 + threadIdx.x / 16;
  const int j = threadIdx.x % 16;
  if (item >= static_cast<int64_t>(a.n) * heads) return;  // whole 16-lane groups leave together
  const int64_t tok = item / heads;
  const int head = static_cast<int>(item - tok * heads);
  const T *row = static_cast<const T *>(a.proj) + tok * a.ld;
  if (head == a.H + a.G) {
    const T *gr = row + static_cast<int64_t>(heads - 1) * a.D;
    for (int h = j; h < a.H; h += 16) a.gate[tok * a.H + h] = sigmoid_f32(Elem<T>::ld(gr + h));
    return;
  }
  const bool is_q = head < a.H;
  const T *src = row + static_cast<int64_t>(head) * a.D;
  const T *bias = is_q ? static_cast<const T *>(a.q_bias) : static_cast<const T *>(a.k_bias);
  if (bias) bias += static_cast<int64_t>(is_q ? head : head - a.H) * a.D;
  const int64_t pos = a.positions[tok];
  const bool pos_ok = pos >= 0 && pos < a.max_pos;
  const float *cs = a.cos_sin + (pos_ok ? pos : 0) * a.rot_dims;
  const int half = a.rot_dims / 2, nch = a.Dp / 8;
  const int64_t slot = a.slots[tok];
  const bool store = slot >= 0 && slot < a.num_slots;
  float x[MAXC][8];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = j + c * 16;
#pragma unroll
    for (int e = 0; e < 8; ++e) x[c][e] = 0.f;
    if (ch < nch) {
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (ch * 8 + e < a.D) x[c][e] = Elem<T>::ld(src + ch * 8 + e) + (bias ? Elem<T>::ld(bias + ch * 8 + e) : 0.f);
      if (!is_q && store)
        Elem<T>::st8(static_cast<T *>(a.v_cache) + (slot * a.G + (head - a.H)) * a.Dp + ch * 8, x[c]);
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const int i = ch * 4 + e / 2;
        if (i < half && pos_ok) {
          const float co = cs[i], si = cs[half + i];
          const float u = x[c][e], v = x[c][e + 1];
          x[c][e] = __fmul_rn(u, co) - __fmul_rn(v, si);
          x[c][e + 1] = __fmul_rn(v, co) + __fmul_rn(u, si);
        }
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) ss = fmaf(x[c][e], x[c][e], ss);
    }
  }
  ss = group_sum<16>(ss);
  const float inv = 1.0f / sqrtf(ss / static_cast<float>(a.D) + a.eps);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = j + c * 16;
    if (ch < nch) {
#pragma unroll
      for (int e = 0; e < 8; ++e) x[c][e] *= inv;
      if (is_q)
        Elem<T>::st8(static_cast<T *>(a.q_out) + (tok * a.H + head) * a.Dp + ch * 8, x[c]);
      else if (store)
        Elem<T>::st8(static_cast<T *>(a.k_cache) + (slot * a.G + (head - a.H)) * a.Dp + ch * 8, x[c]);
    }
  }
}

// The same for rows that can be read 8 elements at a time (head_dim and rot_dims multiples of 8): a team keeps one head
// and takes TOK consecutive tokens, with the loads of all of them in flight before the first is touched.
template <typename T, int MAXC, int TOK, bool PART>
__global__ __launch_bounds__(256) void attn_prep_vec_kernel(const AttnPrepArgs a) {
  const int head = blockIdx.y * 16 + threadIdx.x / 16, j = threadIdx.x % 16;
  const int64_t tok0 = static_cast<int64_t>(blockIdx.x) * TOK;
  if (head > a.H + a.G) return;                      // whole 16-lane groups leave together
  const T *base = static_cast<const T *>(a.proj);
  if (head == a.H + a.G) {
    for (int k = 0; k < TOK; ++k) {
      if (tok0 + k >= a.n) return;
      const T *gr = base + (tok0 + k) * a.ld + static_cast<int64_t>(head) * a.D;
      for (int h = j; h < a.H; h += 16)
        a.gate[(tok0 + k) * a.H + h] = sigmoid_f32(PART ? a.part.ld(tok0 + k, head * a.D + h) : Elem<T>::ld(gr + h));
    }
    return;
  }
  const bool is_q = head < a.H;
  const T *bias = is_q ? static_cast<const T *>(a.q_bias) : static_cast<const T *>(a.k_bias);
  if (bias) bias += static_cast<int64_t>(is_q ? head : head - a.H) * a.D;
  const int half = a.rot_dims / 2, nch = a.Dp / 8;
  typename Elem<T>::Raw8 raw[TOK][MAXC];
  int64_t pos[TOK], slot[TOK];
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const int64_t tok = min(tok0 + k, static_cast<int64_t>(a.n) - 1);
    const T *src = base + tok * a.ld + static_cast<int64_t>(head) * a.D;
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
      if (!PART) Elem<T>::raw8(src + min((j + c * 16) * 8, a.D - 8), raw[k][c]);
    pos[k] = a.positions[tok];
    slot[k] = a.slots[tok];
  }
  float4 co[TOK][MAXC], si[TOK][MAXC];
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const bool ok = pos[k] >= 0 && pos[k] < a.max_pos;
    const float *cs = a.cos_sin + (ok ? pos[k] : 0) * a.rot_dims;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int i = (j + c * 16) * 4;
      co[k][c] = make_float4(1.f, 1.f, 1.f, 1.f);
      si[k][c] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (ok && i < half) {
        co[k][c] = *reinterpret_cast<const float4 *>(cs + i);
        si[k][c] = *reinterpret_cast<const float4 *>(cs + half + i);
      }
    }
  }
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    if (tok0 + k >= a.n) return;
    const int64_t tok = tok0 + k;
    const bool store = !is_q && slot[k] >= 0 && slot[k] < a.num_slots;
    const int64_t crow = (slot[k] * a.G + (head - a.H)) * a.Dp;
    float x[MAXC][8], ss = 0.f;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int ch = j + c * 16;
      if constexpr (PART) a.part.ld8(tok, head * a.D + min(ch * 8, a.D - 8), x[c]);
      else Elem<T>::cvt8(raw[k][c], x[c]);
      if (ch * 8 >= a.D) {
#pragma unroll
        for (int e = 0; e < 8; ++e) x[c][e] = 0.f;
      } else if (bias) {
        float b[8];
        Elem<T>::ld8(bias + ch * 8, b);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[c][e] += b[e];
      }
      if (store && ch < nch) Elem<T>::st8(static_cast<T *>(a.v_cache) + crow + ch * 8, x[c]);
      const float cv[4] = {co[k][c].x, co[k][c].y, co[k][c].z, co[k][c].w}, sv[4] = {si[k][c].x, si[k][c].y, si[k][c].z, si[k][c].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float u = x[c][2 * e], v = x[c][2 * e + 1];
        x[c][2 * e] = __fmul_rn(u, cv[e]) - __fmul_rn(v, sv[e]);
        x[c][2 * e + 1] = __fmul_rn(v, cv[e]) + __fmul_rn(u, sv[e]);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) ss = fmaf(x[c][e], x[c][e], ss);
    }
    ss = group_sum<16>(ss);
    const float inv = 1.0f / sqrtf(ss / static_cast<float>(a.D) + a.eps);
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int ch = j + c * 16;
      if (ch < nch) {
#pragma unroll
        for (int e = 0; e < 8; ++e) x[c][e] *= inv;
        if (is_q) Elem<T>::st8(static_cast<T *>(a.q_out) + (tok * a.H + head) * a.Dp + ch * 8, x[c]);
        else if (store) Elem<T>::st8(static_cast<T *>(a.k_cache) + crow + ch * 8, x[c]);
      }
    }
  }
}

template <typename T>
int launch_attn_prep(const AttnPrepArgs &a, hipStream_t s) {
  const int heads = a.H + a.G + 1;
  if (a.vec) {
    const bool part = a.part.splits > 1;
    const int tok = !part && a.n > 1024 ? 4 : 1;
    const dim3 grid((a.n + tok - 1) / tok, (heads + 15) / 16);
#define TLF_PREP(MAXC)                                                                         \
  do {                                                                                         \
    if (part) TLF_LAUNCH((attn_prep_vec_kernel<unsigned short, MAXC, 1, true>), grid, dim3(256), 0, s, a); \
    else if (tok == 4) TLF_LAUNCH((attn_prep_vec_kernel<T, MAXC, 4, false>), grid, dim3(256), 0, s, a);    \
    else TLF_LAUNCH((attn_prep_vec_kernel<T, MAXC, 1, false>), grid, dim3(256), 0, s, a);      \
  } while (0)
    if (a.Dp <= 128) TLF_PREP(1);
    else TLF_PREP(2);
#undef TLF_PREP
    return launch_status();
  }
  const dim3 grid(static_cast<unsigned>((static_cast<int64_t>(a.n) * heads + 15) / 16));
  if (a.Dp <= 128) TLF_LAUNCH((attn_prep_kernel<T, 1>), grid, dim3(256), 0, s, a);
  else TLF_LAUNCH((attn_prep_kernel<T, 2>), grid, dim3(256), 0, s, a);
  return launch_status();
}

// ---------------------------------------------------------------------------------------------------------------
// Sequence s of the step holds tokens [start, start + n): the blocks it completes are floor(start / pool) ..
// floor((start + n) / pool) - 1.
template <typename T>
__global__ __launch_bounds__(256) void pool_blocks_kernel(const PooledCache c, const int32_t *cu_q,
                                                          const int32_t *starts, int32_t seq0) {
  const int seq = seq0 + blockIdx.y;
  const int start = starts[seq], n = cu_q[seq + 1] - cu_q[seq];
  const int first = start / c.pool, last = (start + n) / c.pool;
  const int per = 2 * (c.Dp / 8), items = c.G * per;
  const int32_t *bt = c.bt + seq * c.bt_stride;
  const int64_t at = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  const int b = first + static_cast<int>(at / items), t = static_cast<int>(at % items);
  if (b < last) pool_block_chunk<T>(c, bt, b, t / per, t % per);
}

// ---------------------------------------------------------------------------------------------------------------
struct RowsArgs {
  PooledCache c;
  const void *q;             // [rows, H, Dp]
  const void *bias;          // [H], added to the score
  const float *gate;         // [rows, H]
  const int64_t *positions;  // [rows]
  const int32_t *slots;      // [rows], negative: padding row
  const int32_t *row_seq;    // [rows] or NULL: row r belongs to sequence r
  void *out;                 // [rows, ldo]
  int64_t ldo;
  float *partial;            // [splits, rows, H, Dp] when splits > 1
  int32_t rows, H, group, passes, splits, pool_new;
  float scale_log2;
};

template <typename T, int LPK, int GH>
__global__ __launch_bounds__(256) void rows_kernel(const RowsArgs a) {
  constexpr int KPW = 64 / LPK;                     // keys a wave looks at side by side
  constexpr int U = 4;                              // and one after the other, all loads in flight
  constexpr int kStep = 4 * U * KPW;
  __shared__ __attribute__((aligned(16))) float red[4][GH][LPK * 8];
  const PooledCache &c = a.c;
  const int row = blockIdx.z, split = blockIdx.x;
  const int kvh = blockIdx.y / a.passes, pass = blockIdx.y % a.passes;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int sub = lane / LPK, l = lane % LPK;
  const int seq = a.row_seq ? a.row_seq[row] : row;
  const int i = static_cast<int>(a.positions[row]);
  const bool live = a.slots[row] >= 0 && i >= 0;    // workgroup uniform
  const int32_t *bt = c.bt + seq * c.bt_stride;
  const int h0 = kvh * a.group + pass * GH;
  const int nh = min(GH, a.group - pass * GH);
  const bool lane_ok = l * 8 < c.Dp;
  const int dcol = lane_ok ? l * 8 : 0;

  float qf[GH][8], o[GH][8], pb[GH];
#pragma unroll
  for (int g = 0; g < GH; ++g) {
#pragma unroll
    for (int e = 0; e < 8; ++e) qf[g][e] = o[g][e] = 0.f;
    pb[g] = 0.f;
    if (g < nh) {
      if (lane_ok) Elem<T>::ld8(static_cast<const T *>(a.q) + (static_cast<int64_t>(row) * a.H + h0 + g) * c.Dp + dcol, qf[g]);
#pragma unroll
      for (int e = 0; e < 8; ++e) qf[g][e] *= -a.scale_log2;
      pb[g] = -kLog2e * Elem<T>::ld(static_cast<const T *>(a.bias) + h0 + g);
    }
  }
  if (live) {
    const int nb = pooled_visible(i, c.size, c.pool);
    const int w0 = max(0, i - c.size + 1);
    const int total = nb + (i - w0 + 1);
    const int per = ((total + a.splits - 1) / a.splits + U * KPW - 1) / (U * KPW) * (U * KPW);
    const int lo = split * per, hi = min(total, lo + per);
    const int64_t rs = static_cast<int64_t>(c.G) * c.Dp;
    const int64_t off = static_cast<int64_t>(kvh) * c.Dp + dcol;
    for (int base = lo + wave * U * KPW; base < hi; base += kStep) {
      typename Elem<T>::Raw8 kr[U], vr[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int item = min(base + u * KPW + sub, hi - 1);
        const bool pooled = item < nb;
        const int64_t at = (pooled ? block_row(c, bt, item) : token_row(c, bt, w0 + item - nb)) * rs + off;
        Elem<T>::raw8(static_cast<const T *>(pooled ? c.pk : c.k) + at, kr[u]);
        Elem<T>::raw8(static_cast<const T *>(pooled ? c.pv : c.v) + at, vr[u]);
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
          if (!lane_ok) s = 0.f;
          s = group_sum<LPK>(s) + pb[g];
          const float w = ok ? sigmoid_neg_log2(s) : 0.f;
#pragma unroll
          for (int e = 0; e < 8; ++e) o[g][e] = fmaf(w, vf[e], o[g][e]);
        }
      }
    }
  }
  // keys side by side in a wave, then the four waves
#pragma unroll
  for (int g = 0; g < GH; ++g)
#pragma unroll
    for (int e = 0; e < 8; ++e) {
#pragma unroll
      for (int s = LPK; s < 64; s <<= 1) o[g][e] += __shfl_xor(o[g][e], s, 64);
      if (sub == 0) red[wave][g][l * 8 + e] = o[g][e];
    }
  __syncthreads();
  for (int t = tid; t < nh * c.Dp; t += 256) {
    const int g = t / c.Dp, d = t - g * c.Dp;
    const float s = red[0][g][d] + red[1][g][d] + red[2][g][d] + red[3][g][d];
    const int head = h0 + g;
    if (a.splits > 1)
      a.partial[((static_cast<int64_t>(split) * a.rows + row) * a.H + head) * c.Dp + d] = s;
    else if (d < c.D)
      Elem<T>::st(static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(head) * c.D + d,
                  live ? s * a.gate[static_cast<int64_t>(row) * a.H + head] : 0.f);
  }
  // a block that this token completes leaves the window one step later at the earliest: nobody reads it in this step
  if (a.pool_new && live && split == 0 && pass == 0 && (i + 1) % c.pool == 0 && tid < 2 * (c.Dp / 8))
    pool_block_chunk<T>(c, bt, (i + 1) / c.pool - 1, kvh, tid);
}

template <typename T>
__global__ __launch_bounds__(256) void rows_merge_kernel(const RowsArgs a) {
  const int64_t at = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  const int D = a.c.D;
  if (at >= static_cast<int64_t>(a.rows) * a.H * D) return;
  const int64_t rh = at / D;
  const int d = static_cast<int>(at - rh * D);
  const int64_t row = rh / a.H;
  const int head = static_cast<int>(rh - row * a.H);
  const int64_t stride = static_cast<int64_t>(a.rows) * a.H * a.c.Dp;
  float s = 0.f;
  for (int k = 0; k < a.splits; ++k) s += a.partial[k * stride + rh * a.c.Dp + d];
  Elem<T>::st(static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(head) * D + d,
              a.slots[row] >= 0 ? s * a.gate[rh] : 0.f);
}

template <typename T>
int launch_rows(const RowsArgs &a, int gh, hipStream_t stream) {
  const dim3 grid(a.splits, a.c.G * a.passes, a.rows);
#define TLF_ROWS(LPK, GH) TLF_LAUNCH((rows_kernel<T, LPK, GH>), grid, dim3(256), 0, stream, a)
#define TLF_ROWS_GH(LPK)                    \
  do {                                      \
    if (gh == 1) TLF_ROWS(LPK, 1);          \
    else if (gh == 2) TLF_ROWS(LPK, 2);     \
    else if (gh == 4) TLF_ROWS(LPK, 4);     \
    else TLF_ROWS(LPK, 8);                  \
  } while (0)
  if (a.c.Dp <= 32) TLF_ROWS_GH(4);
  else if (a.c.Dp <= 64) TLF_ROWS_GH(8);
  else if (a.c.Dp <= 128) TLF_ROWS_GH(16);
  else TLF_ROWS_GH(32);
#undef TLF_ROWS_GH
#undef TLF_ROWS
  int rc = launch_status();
  if (rc != TLF_OK || a.splits == 1) return rc;
  const int64_t total = static_cast<int64_t>(a.rows) * a.H * a.c.D;
  TLF_LAUNCH((rows_merge_kernel<T>), dim3(static_cast<unsigned>((total + 255) / 256)), dim3(256), 0, stream, a);
  return launch_status();
}

// Splits of the keys: enough workgroups to fill the chip, at least 128 keys each.
int rows_splits(int64_t groups, int64_t max_keys) {
  const int64_t want = (1024 + groups - 1) / groups;
  const int64_t most = (max_keys + 127) / 128;
  return static_cast<int>(std::max<int64_t>(1, std::min<int64_t>({want, most, 32})));
}
int rows_heads_per_pass(int group) { return group <= 1 ? 1 : group <= 2 ? 2 : group <= 4 ? 4 : 8; }

}  // namespace tlf

extern "C" int tlf_attn_prep(const void *proj, int64_t proj_stride, const float *partials, int32_t splits,
                             const float *scale, const void *q_bias, const void *k_bias,
                             const int64_t *positions, const float *cos_sin, int32_t max_pos, int32_t rot_dims,
                             const int32_t *slot_mapping, int64_t num_slots, void *q_out, void *k_cache, void *v_cache,
                             float *gate, int32_t n, int32_t num_q_heads, int32_t num_kv_heads, int32_t head_dim,
                             int32_t padded_dim, float eps, int32_t dtype, void *stream) {
  using namespace tlf;
  if (n < 0 || num_q_heads <= 0 || num_kv_heads <= 0 || head_dim <= 0 || head_dim > 256) return TLF_E_SHAPE;
  if (padded_dim != (head_dim + 31) / 32 * 32 || rot_dims < 0 || rot_dims % 2 || rot_dims > head_dim) return TLF_E_SHAPE;
  if (proj_stride < static_cast<int64_t>(num_q_heads + num_kv_heads) * head_dim + num_q_heads) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (n == 0) return TLF_OK;
  if (int rc = partials_check(partials, scale, splits, dtype)) return rc;
  if ((!proj && splits <= 1) || !positions || (rot_dims && !cos_sin) || !slot_mapping || !q_out || !k_cache || !v_cache || !gate) return TLF_E_NULL;
  if (!aligned16(q_out) || !aligned16(k_cache) || !aligned16(v_cache)) return TLF_E_ALIGN;
  AttnPrepArgs a{proj, Partials{partials, scale, n * proj_stride, static_cast<int32_t>(proj_stride), splits}, proj_stride, q_bias, k_bias, positions, cos_sin, max_pos, rot_dims, slot_mapping, num_slots,
                 q_out, k_cache, v_cache, gate, n, num_q_heads, num_kv_heads, head_dim, padded_dim, eps, 0};
  a.vec = head_dim % 8 == 0 && rot_dims % 8 == 0 && proj_stride % 8 == 0 && aligned16(proj) && aligned16(q_bias) &&
          aligned16(k_bias) && aligned16(cos_sin) && (num_q_heads + num_kv_heads + 16) / 16 <= 65535;
  if (splits > 1 && !a.vec) return TLF_E_UNSUPPORTED;
  hipStream_t s = static_cast<hipStream_t>(stream);
  return dtype == TLF_DT_BF16 ? launch_attn_prep<unsigned short>(a, s) : launch_attn_prep<float>(a, s);
}

extern "C" int tlf_pool_blocks(const void *k_cache, const void *v_cache, void *pk_cache, void *pv_cache,
                               const int32_t *block_tables, int64_t bt_stride, const int32_t *cu_seqlens_q,
                               const int32_t *seq_starts, int32_t first_seq, int32_t num_seqs, int32_t max_tokens,
                               int32_t num_kv_heads, int32_t head_dim, int32_t block_size, int32_t pool, int32_t window,
                               int64_t num_pages, int32_t dtype, void *stream) {
  using namespace tlf;
  if (num_seqs <= 0 || max_tokens <= 0) return num_seqs < 0 || max_tokens < 0 ? TLF_E_SHAPE : TLF_OK;
  if (num_seqs > 65535 || first_seq < 0) return TLF_E_SHAPE;
  PooledCache c{k_cache, v_cache, pk_cache, pv_cache, block_tables, bt_stride, block_size, pool, 0, window,
                num_kv_heads, head_dim, (head_dim + 31) / 32 * 32, num_pages, -1};
  if (int rc = pooled_cache_check(c, dtype)) return rc;
  if (!cu_seqlens_q || !seq_starts) return TLF_E_NULL;
  pooled_cache_finish(c);
  const int64_t items = static_cast<int64_t>(c.G) * 2 * (c.Dp / 8) * (max_tokens / pool + 1);
  const dim3 grid(static_cast<unsigned>((items + 255) / 256), num_seqs);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == TLF_DT_BF16) TLF_LAUNCH((pool_blocks_kernel<unsigned short>), grid, dim3(256), 0, s, c, cu_seqlens_q, seq_starts, first_seq);
  else TLF_LAUNCH((pool_blocks_kernel<float>), grid, dim3(256), 0, s, c, cu_seqlens_q, seq_starts, first_seq);
  return launch_status();
}

extern "C" size_t tlf_pooled_attn_rows_workspace_bytes(int32_t rows, int32_t num_q_heads, int32_t num_kv_heads,
                                                       int32_t head_dim, int32_t pool, int32_t window, int32_t max_len) {
  using namespace tlf;
  if (rows <= 0 || num_q_heads <= 0 || num_kv_heads <= 0 || num_q_heads % num_kv_heads || head_dim <= 0 || pool <= 0) return 0;
  const int group = num_q_heads / num_kv_heads, gh = rows_heads_per_pass(group), passes = (group + gh - 1) / gh;
  const int64_t keys = std::min<int64_t>(window, max_len) + max_len / pool;
  const int splits = rows_splits(static_cast<int64_t>(rows) * num_kv_heads * passes, keys);
  if (splits == 1) return 0;
  return static_cast<size_t>(splits) * rows * num_q_heads * ((head_dim + 31) / 32 * 32) * 4;
}

extern "C" int tlf_pooled_attn_rows(const void *q, const void *score_bias, const float *gate, const void *k_cache,
                                    const void *v_cache, void *pk_cache, void *pv_cache, const int32_t *block_tables,
                                    int64_t bt_stride, const int64_t *positions, const int32_t *slot_mapping,
                                    const int32_t *row_seq, void *out, int64_t out_stride, int32_t rows,
                                    int32_t num_q_heads, int32_t num_kv_heads, int32_t head_dim, int32_t block_size,
                                    int32_t pool, int32_t window, int32_t max_len, int64_t num_pages, float scale,
                                    int32_t pool_new, int32_t dtype, void *workspace, size_t workspace_bytes,
                                    void *stream) {
  using namespace tlf;
  if (rows < 0 || rows > 65535 || num_q_heads <= 0 || num_kv_heads <= 0 || num_q_heads % num_kv_heads) return TLF_E_SHAPE;
  if (out_stride < static_cast<int64_t>(num_q_heads) * head_dim || max_len <= 0) return TLF_E_SHAPE;
  if (rows == 0) return TLF_OK;
  PooledCache c{k_cache, v_cache, pk_cache, pv_cache, block_tables, bt_stride, block_size, pool, 0, window,
                num_kv_heads, head_dim, (head_dim + 31) / 32 * 32, num_pages, -1};
  if (int rc = pooled_cache_check(c, dtype)) return rc;
  if (!q || !score_bias || !gate || !positions || !slot_mapping || !out) return TLF_E_NULL;
  if (!aligned16(q)) return TLF_E_ALIGN;
  pooled_cache_finish(c);
  RowsArgs a{c, q, score_bias, gate, positions, slot_mapping, row_seq, out, out_stride, static_cast<float *>(workspace),
             rows, num_q_heads, num_q_heads / num_kv_heads, 1, 1, pool_new, scale * kLog2e};
  const int gh = rows_heads_per_pass(a.group);
  a.passes = (a.group + gh - 1) / gh;
  if (static_cast<int64_t>(num_kv_heads) * a.passes > 65535) return TLF_E_SHAPE;
  const int64_t keys = std::min<int64_t>(window, max_len) + max_len / pool;
  a.splits = rows_splits(static_cast<int64_t>(rows) * num_kv_heads * a.passes, keys);
  if (a.splits > 1 && (!workspace || workspace_bytes < tlf_pooled_attn_rows_workspace_bytes(
                                         rows, num_q_heads, num_kv_heads, head_dim, pool, window, max_len)))
    return TLF_E_WORKSPACE;
  return dtype == TLF_DT_BF16 ? launch_rows<unsigned short>(a, gh, static_cast<hipStream_t>(stream))
                              : launch_rows<float>(a, gh, static_cast<hipStream_t>(stream));
}
