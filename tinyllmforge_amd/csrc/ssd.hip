// State-space layer with a scalar decay per head (Mamba-2).  Per head h of group g, with fp32 state S [N, P]:
//
//   [x | B | C] = silu(short causal convolution over time per channel + bias)
//   dt_t = softplus(dt_t + dt_bias_h),  S_t = exp(-exp(A_log_h) dt_t) S_(t-1) + dt_t B_t x_t^T,  y_t = S_t^T C_t + D_h x_t
//   out = y * silu(z)
//
// Input is one projection row per token, [z: H P | x: H P | B: G N | C: G N | dt: H].  dt, decays and the state are fp32; x, B
// and C are of the activations' dtype.  The convolution's state is a ring of `taps` projected rows per sequence, position p in
// row p mod taps; positions below 0 are zeros and position 0 starts from a zero state, so nothing is ever cleared.
//
//   ssd_decode_kernel  one token: one workgroup per (row, head), everything from the projection to the gate; the state is
//                      streamed through once (HBM bound: 8 N P bytes per head)
//   portions of prompts:
//   ssd_conv_kernel    convolution, silu, dt and log2 decays of all rows
//   ssd_chunk_kernel   bf16, matrix cores: one workgroup per (sequence or segment, head, 16 PT columns of P), sequential over
//                      chunks of 64 tokens.  With c_t the sum of the log2 decays within the chunk:
//                        G^T[s, t] = B_s . C_t;  M^T[s, t] = G^T 2^(c_t - c_s) dt_s for s <= t
//                        Y^T[p, t] = X^T M^T + 2^(c_t) (S^T C^T)
//                        S = 2^(c_end) S + (dt_s 2^(c_end - c_s) B)^T X
//                      Every exponent is <= 0.  x, B and C are exact in bf16; M, the scaled B and S enter as bf16 hi + lo pairs (16
//                      significant bits), S itself stays in fp32 accumulators.  The s rows of two 16-row tiles are picked so that
//                      their accumulators are the next product's operand.  Where (sequences, heads, columns) alone leave CUs idle
//                      a sequence is cut into segments: a first pass gathers each segment's own contribution from zero,
//                      ssd_segments_kernel chains them, and the second pass starts every segment from its state.
//   ssd_scan_kernel    any size and dtype, token by token
#include <algorithm>

#include "elem.h"

namespace tlf {

constexpr int kSsdMaxN = 512, kSsdMaxP = 512, kSC = 64;   // kSC: tokens per chunk

struct SsdArgs {
  const void *proj;        // [n, ld]
  Partials part;           // decode: or its partial sums
  int64_t ld;
  const void *conv, *conv_bias;              // [taps, channels], [channels]
  const void *dt_bias, *A_log, *D;           // [H]
  void *ring;              // [slots, taps, channels]
  float *state;            // [slots, H, N, P]
  const int32_t *state_slots;                // per sequence
  int32_t num_slots;
  const int64_t *positions;                  // per row
  const int32_t *row_seq, *cu_q, *starts;
  void *xbc;               // [rows, channels] activated
  float *dt, *decay;       // [rows, H]: step size, log2 of the decay
  void *out;               // [n, ldo]
  int64_t ldo;
  int32_t rows, H, P, N, G, taps, inner, channels;
  int32_t first_seq, seqs, first_row, segs, slices;
  float *seg_state, *seg_decay;              // [seqs, segs, H, N, P], [seqs, segs, H]
};

template <typename T>
__device__ __forceinline__ float ssd_step(const SsdArgs &a, float raw, int h) {
  return softplus_f32(raw + Elem<T>::ld(static_cast<const T *>(a.dt_bias) + h));
}
template <typename T>
__device__ __forceinline__ float ssd_log2_decay(const SsdArgs &a, float dt, int h) {
  return -expf(Elem<T>::ld(static_cast<const T *>(a.A_log) + h)) * dt * 1.4426950408889634f;
}

// 32-bit rows: the library's exponential; bf16 rows: the hardware's, far more exact than the rounding that follows.
template <typename T>
__device__ __forceinline__ float ssd_silu(float z) {
  if constexpr (sizeof(T) == 4) return silu_f32(z);
  return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

// The state's N rows are dealt to teams of lanes_v threads, VEC columns each; osum[team][P] gets the teams' parts of S^T C.
template <int VEC>
__device__ __forceinline__ void ssd_update(float *st, const float *xs, const float *bs, const float *cs, float keep, bool fresh, float dt,
                                           int N, int P, int lanes_v, float *osum) {
  const int tid = threadIdx.x, team = tid / lanes_v, lane = tid % lanes_v, teams = 256 / lanes_v;
  for (int c = lane; c < P / VEC; c += lanes_v) {
    float o[VEC], x[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      o[e] = 0.f;
      x[e] = xs[c * VEC + e] * dt;
    }
    constexpr int U = 8;
    for (int d0 = team; d0 < N; d0 += teams * U) {
      float s[U][VEC];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float *p = st + static_cast<int64_t>(min(d0 + u * teams, N - 1)) * P + c * VEC;
        if constexpr (VEC == 4) {
          const float4 t = *reinterpret_cast<const float4 *>(p);
          s[u][0] = t.x; s[u][1] = t.y; s[u][2] = t.z; s[u][3] = t.w;
        } else {
          s[u][0] = *p;
        }
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int d = d0 + u * teams;
        if (d < N) {
          const float b = bs[d], cc = cs[d];
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            s[u][e] = fresh ? b * x[e] : fmaf(keep, s[u][e], b * x[e]);
            o[e] = fmaf(s[u][e], cc, o[e]);
          }
          float *p = st + static_cast<int64_t>(d) * P + c * VEC;
          if constexpr (VEC == 4) *reinterpret_cast<float4 *>(p) = make_float4(s[u][0], s[u][1], s[u][2], s[u][3]);
          else *p = s[u][0];
        }
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) osum[team * P + c * VEC + e] = o[e];
  }
}

template <typename T, int VEC, bool PART>
__global__ __launch_bounds__(256) void ssd_decode_kernel(const SsdArgs a, int lanes_v) {
  __shared__ float xs[kSsdMaxP], bs[kSsdMaxN], cs[kSsdMaxN], sdt;
  __shared__ __attribute__((aligned(16))) float osum[2048];
  const int64_t row = blockIdx.y;
  const int h = blockIdx.x, tid = threadIdx.x, share = a.H / a.G, grp = h / share;
  const int slot = a.state_slots[row];
  const int64_t pos = a.positions[row];
  T *out = static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(h) * a.P;
  if (slot < 0 || slot >= a.num_slots || pos < 0) {    // padding row of a captured graph
    for (int v = tid; v < a.P; v += 256) Elem<T>::st(out + v, 0.f);
    return;
  }
  const T *pr = static_cast<const T *>(a.proj) + row * a.ld;
  auto in = [&](int col) __attribute__((always_inline)) { return PART ? a.part.ld(row, col) : Elem<T>::ld(pr + col); };
  T *ring = static_cast<T *>(a.ring) + static_cast<int64_t>(slot) * a.taps * a.channels;
  for (int i = tid; i < a.P + 2 * a.N; i += 256) {
    const bool own = i < a.P;
    const int ch = own ? h * a.P + i : a.inner + (i < a.P + a.N ? grp * a.N + i - a.P : (a.G + grp) * a.N + i - a.P - a.N);
    const float now = in(a.inner + ch);
    float y = Elem<T>::ld(static_cast<const T *>(a.conv_bias) + ch);
    for (int b = a.taps - 1; b > 0; --b)
      if (pos >= b) y = fmaf(Elem<T>::ld(static_cast<const T *>(a.conv) + static_cast<int64_t>(a.taps - 1 - b) * a.channels + ch),
                             Elem<T>::ld(ring + (pos - b) % a.taps * a.channels + ch), y);
    y = fmaf(Elem<T>::ld(static_cast<const T *>(a.conv) + static_cast<int64_t>(a.taps - 1) * a.channels + ch), now, y);
    y = Elem<T>::rnd(ssd_silu<T>(y));
    // the row written is none of those read: heads that share a group do not disturb each other
    if (own || h == grp * share) Elem<T>::st(ring + pos % a.taps * a.channels + ch, now);
    if (own) xs[i] = y;
    else if (i < a.P + a.N) bs[i - a.P] = y;
    else cs[i - a.P - a.N] = y;
  }
  if (tid == 0) sdt = ssd_step<T>(a, in(a.inner + a.channels + h), h);
  __syncthreads();
  const float dt = sdt;
  const bool fresh = pos == 0;
  const int teams = 256 / lanes_v;
  float *st = a.state + (static_cast<int64_t>(slot) * a.H + h) * a.N * a.P;
  ssd_update<VEC>(st, xs, bs, cs, exp2f(ssd_log2_decay<T>(a, dt, h)), fresh, dt, a.N, a.P, lanes_v, osum);
  __syncthreads();
  const float D = Elem<T>::ld(static_cast<const T *>(a.D) + h);
  for (int v = tid; v < a.P; v += 256) {
    float y = 0.f;
    for (int t = 0; t < teams; ++t) y += osum[t * a.P + v];
    Elem<T>::st(out + v, fmaf(D, xs[v], y) * ssd_silu<T>(in(h * a.P + v)));
  }
}

// ---------------------------------------------------------------------------------------------------------------
// TOK consecutive rows and VEC channels per thread; TAPS > 0: the rows are read once, 0: any number of taps, rows read again.
// The last blockIdx.y holds step sizes and decays.  Rows are counted from `first_row`.
template <typename T, int VEC, int TAPS, int TOK>
__global__ __launch_bounds__(256) void ssd_conv_kernel(const SsdArgs a) {
  const int64_t r0 = static_cast<int64_t>(blockIdx.x) * TOK;
  if (blockIdx.y == gridDim.y - 1) {
    for (int i = threadIdx.x; i < TOK * a.H; i += 256) {
      const int64_t r = r0 + i / a.H;
      const int h = i % a.H;
      if (r >= a.rows) return;
      const float raw = Elem<T>::ld(static_cast<const T *>(a.proj) + (a.first_row + r) * a.ld + a.inner + a.channels + h);
      const float dt = ssd_step<T>(a, raw, h);
      a.dt[r * a.H + h] = dt;
      a.decay[r * a.H + h] = ssd_log2_decay<T>(a, dt, h);
    }
    return;
  }
  const int ch = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (ch >= a.channels) return;
  constexpr int kBack = TAPS > 0 ? TAPS - 1 : 0;
  auto ldv = [](const T *p, float (&f)[VEC]) __attribute__((always_inline)) {
    if constexpr (VEC == 8) Elem<T>::ld8(p, f);
    else f[0] = Elem<T>::ld(p);
  };
  const T *base = static_cast<const T *>(a.proj) + a.inner + ch, *w = static_cast<const T *>(a.conv) + ch;
  float bias[VEC];
  ldv(static_cast<const T *>(a.conv_bias) + ch, bias);
  auto put = [&](int64_t r, float (&y)[VEC]) __attribute__((always_inline)) {
    T *o = static_cast<T *>(a.xbc) + r * a.channels + ch;
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = ssd_silu<T>(y[e]);
    if constexpr (VEC == 8) Elem<T>::st8(o, y);
    else Elem<T>::st(o, y[0]);
  };
  if constexpr (TAPS > 0 && VEC == 8) {
    // one sequence from the first row looked at to the last: all loads in flight, every row read once
    const int64_t first = a.first_row + r0 - kBack, last = a.first_row + r0 + TOK - 1;
    if (r0 + TOK <= a.rows && first >= a.first_row && a.row_seq[first] == a.row_seq[last]) {
      typename Elem<T>::Raw8 u[TOK + kBack], wt[TAPS];
#pragma unroll
      for (int i = 0; i < TOK + kBack; ++i) Elem<T>::raw8(base + (first + i) * a.ld, u[i]);
#pragma unroll
      for (int t = 0; t < TAPS; ++t) Elem<T>::raw8(w + static_cast<int64_t>(t) * a.channels, wt[t]);
#pragma unroll
      for (int k = 0; k < TOK; ++k) {
        float y[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[e] = bias[e];
#pragma unroll
        for (int t = 0; t < TAPS; ++t) {
          float f[8], wf[8];
          Elem<T>::cvt8(u[k + t], f);
          Elem<T>::cvt8(wt[t], wf);
#pragma unroll
          for (int e = 0; e < VEC; ++e) y[e] = fmaf(wf[e], f[e], y[e]);
        }
        put(r0 + k, y);
      }
      return;
    }
  }
  for (int k = 0; k < TOK; ++k) {
    const int64_t r = r0 + k, row = a.first_row + r;
    if (r >= a.rows) return;
    const int seq = a.row_seq[row];
    const int64_t begin = a.cu_q[seq], pos = a.positions[row], slot = a.state_slots[seq];
    const bool held = slot >= 0 && slot < a.num_slots;
    const T *ring = static_cast<const T *>(a.ring) + (held ? slot : 0) * a.taps * a.channels + ch;
    float y[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = bias[e];
    for (int b = a.taps - 1; b >= 0; --b) {          // rows back
      if (pos < b || (row - b < begin && !held)) continue;
      float f[VEC], wf[VEC];
      ldv(row - b >= begin ? base + (row - b) * a.ld : ring + (pos - b) % a.taps * a.channels, f);
      ldv(w + static_cast<int64_t>(a.taps - 1 - b) * a.channels, wf);
#pragma unroll
      for (int e = 0; e < VEC; ++e) y[e] = fmaf(wf[e], f[e], y[e]);
    }
    put(r, y);
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void ssd_scan_kernel(const SsdArgs a, int lanes_v) {
  __shared__ float xs[kSsdMaxP], bs[kSsdMaxN], cs[kSsdMaxN];
  __shared__ __attribute__((aligned(16))) float osum[2048];
  const int h = blockIdx.x, seq = a.first_seq + blockIdx.y, tid = threadIdx.x, grp = h / (a.H / a.G), teams = 256 / lanes_v;
  const int slot = a.state_slots[seq];
  if (slot < 0 || slot >= a.num_slots) return;
  float *st = a.state + (static_cast<int64_t>(slot) * a.H + h) * a.N * a.P;
  const float D = Elem<T>::ld(static_cast<const T *>(a.D) + h);
  const int begin = a.cu_q[seq], end = a.cu_q[seq + 1];
  bool fresh = a.starts[seq] == 0;
  for (int row = begin; row < end; ++row, fresh = false) {
    const int64_t r = row - a.first_row;
    const T *p = static_cast<const T *>(a.xbc) + r * a.channels;
    __syncthreads();
    for (int i = tid; i < a.P + 2 * a.N; i += 256) {
      if (i < a.P) xs[i] = Elem<T>::ld(p + h * a.P + i);
      else if (i < a.P + a.N) bs[i - a.P] = Elem<T>::ld(p + a.inner + grp * a.N + i - a.P);
      else cs[i - a.P - a.N] = Elem<T>::ld(p + a.inner + (a.G + grp) * a.N + i - a.P - a.N);
    }
    __syncthreads();
    ssd_update<VEC>(st, xs, bs, cs, exp2f(a.decay[r * a.H + h]), fresh, a.dt[r * a.H + h], a.N, a.P, lanes_v, osum);
    __syncthreads();
    const T *z = static_cast<const T *>(a.proj) + row * a.ld + h * a.P;
    T *out = static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(h) * a.P;
    for (int v = tid; v < a.P; v += 256) {
      float y = 0.f;
      for (int t = 0; t < teams; ++t) y += osum[t * a.P + v];
      Elem<T>::st(out + v, fmaf(D, xs[v], y) * ssd_silu<T>(Elem<T>::ld(z + v)));
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
__device__ __forceinline__ bf16x8 ssd_tr(const unsigned short *p, int ld) {   // rows p, p + 4 ld .. as an operand of 8 rows per lane group
  const uint2 a = __builtin_bit_cast(uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p)));
  const uint2 b = __builtin_bit_cast(uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((shortx4 __attribute__((address_space(3))) *)(p + 4 * ld)));
  return __builtin_bit_cast(bf16x8, make_uint4(a.x, a.y, b.x, b.y));
}
__device__ __forceinline__ void ssd_pair(const float (&w)[8], uint4 &hi, uint4 &lo) {
  unsigned int h[4], l[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    h[e] = pack_bf16x2(w[2 * e], w[2 * e + 1]);
    l[e] = pack_bf16x2(w[2 * e] - __uint_as_float(h[e] << 16), w[2 * e + 1] - __uint_as_float(h[e] & 0xffff0000u));
  }
  hi = make_uint4(h[0], h[1], h[2], h[3]);
  lo = make_uint4(l[0], l[1], l[2], l[3]);
}

// Inclusive sum over the wave's 64 lanes, on the vector ALU.
template <int CTRL, int ROWS>
__device__ __forceinline__ float ssd_dpp_add(float v) {
  return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, ROWS, 0xf, false));
}
__device__ __forceinline__ float ssd_wave_scan(float v) {
  v = ssd_dpp_add<0x111, 0xf>(v);      // row_shr 1, 2, 4, 8: within rows of 16 lanes
  v = ssd_dpp_add<0x112, 0xf>(v);
  v = ssd_dpp_add<0x114, 0xf>(v);
  v = ssd_dpp_add<0x118, 0xf>(v);
  v = ssd_dpp_add<0x142, 0xa>(v);      // row_bcast 15 into rows 1 and 3
  return ssd_dpp_add<0x143, 0xc>(v);   // row_bcast 31 into rows 2 and 3
}

// NN: N in units of 32, PT: columns of P in units of 16.  MODE 0: the whole portion from the state slot and back, 1: a
// segment's own contribution from zero, 2: a segment from the state ssd_segments_kernel left for it.
// Eight waves (four where P has 16 columns only): for Y a wave has 16 tokens and half of the columns, for S some of its 16 x 16 tiles.
template <int PT>
constexpr int ssd_waves() { return PT >= 2 ? 8 : 4; }
template <int NN, int PT, int MODE, bool VEC>
__global__ __launch_bounds__(ssd_waves<PT>() * 64) void ssd_chunk_kernel(const SsdArgs a) {
  typedef unsigned short T;
  constexpr int NW = ssd_waves<PT>(), TH = NW * 64;
  constexpr int NP = NN * 32, PS = PT * 16, LN = NP + 8, LX = PS + 8, NT = 2 * NN;
  constexpr int PTY = PT * 4 / NW;                   // column tiles of a wave's Y
  constexpr int NTW = NT >= NW ? NT / NW : 1;        // row tiles of a wave's S, waves that share one, their column tiles
  constexpr int WPN = NT >= NW ? 1 : NW / NT < PT ? NW / NT : PT, PTU = PT / WPN;
  constexpr int CN = (kSC * NP / 8 + TH - 1) / TH, CX = (kSC * PS / 8 + TH - 1) / TH;   // 16-byte pieces per thread
  __shared__ __attribute__((aligned(16))) T Cs[MODE == 1 ? 1 : kSC][LN], Bs[kSC][LN], Xs[kSC][LX];
  __shared__ __attribute__((aligned(16))) T Sh[MODE == 1 ? 1 : NP][LX], Sl[MODE == 1 ? 1 : NP][LX];
  __shared__ __attribute__((aligned(16))) float cum[kSC], dts[kSC], into_end[kSC];
  const int tid = threadIdx.x, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  // workgroup w runs on XCD w % 8: neighbouring heads, which share B and C, on one
  const int h = a.H % 8 == 0 ? blockIdx.x % 8 * (a.H / 8) + blockIdx.x / 8 : blockIdx.x;
  const int slice = blockIdx.y, sq = MODE == 0 ? blockIdx.z : blockIdx.z / a.segs, seg = MODE == 0 ? 0 : blockIdx.z % a.segs;
  const bool last_seg = MODE == 0 || seg == a.segs - 1;
  if (MODE == 1 && last_seg) return;                 // nobody starts behind the last segment
  const int seq = a.first_seq + sq, grp = h / (a.H / a.G), p0 = slice * PS;
  const int slot = a.state_slots[seq];
  const bool slot_ok = slot >= 0 && slot < a.num_slots;
  const int begin = a.cu_q[seq], tokens = a.cu_q[seq + 1] - begin;
  const int chunks = (tokens + kSC - 1) / kSC;
  int c0 = 0, c1 = chunks;
  if (MODE != 0) {
    const int per = (chunks + a.segs - 1) / a.segs;
    c0 = min(seg * per, chunks);
    c1 = min(c0 + per, chunks);
  }
  const int64_t plane = static_cast<int64_t>(a.N) * a.P, sg = (static_cast<int64_t>(sq) * a.segs + seg) * a.H + h;
  float *st = a.state + (static_cast<int64_t>(slot_ok ? slot : 0) * a.H + h) * plane;
  float *gst = MODE == 0 ? st : a.seg_state + sg * plane;
  const bool from_zero = MODE == 1 || (MODE == 0 && (!slot_ok || a.starts[seq] == 0));

  // S^T tiles: column n of tile j is row (nt0 + j) 16 + n of the state, rows 4 g + r of tile i its columns (pt0 + i) 16 + 4 g + r
  const bool has_state = wave < NT * WPN;            // wave uniform
  const int nt0 = wave / WPN * NTW, pt0 = wave % WPN * PTU;
  floatx4 S[NTW][PTU];
#pragma unroll
  for (int j = 0; j < NTW; ++j)
#pragma unroll
    for (int i = 0; i < PTU; ++i) {
      const int d = (nt0 + j) * 16 + n, p = p0 + (pt0 + i) * 16 + g * 4;
      S[j][i] = floatx4{0.f, 0.f, 0.f, 0.f};
      if (has_state && !from_zero && d < a.N) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (p + r < a.P) S[j][i][r] = gst[static_cast<int64_t>(d) * a.P + p + r];
      }
    }
  auto put_state = [&]() __attribute__((always_inline)) {
    if (MODE == 1 || !has_state) return;
#pragma unroll
    for (int j = 0; j < NTW; ++j)
#pragma unroll
      for (int i = 0; i < PTU; ++i) {
        const int d = MODE == 1 ? 0 : (nt0 + j) * 16 + n;
        const floatx4 v = S[j][i];
        const unsigned int h0 = pack_bf16x2(v[0], v[1]), h1 = pack_bf16x2(v[2], v[3]);
        *reinterpret_cast<uint2 *>(&Sh[d][(pt0 + i) * 16 + g * 4]) = make_uint2(h0, h1);
        *reinterpret_cast<uint2 *>(&Sl[d][(pt0 + i) * 16 + g * 4]) =
            make_uint2(pack_bf16x2(v[0] - __uint_as_float(h0 << 16), v[1] - __uint_as_float(h0 & 0xffff0000u)),
                       pack_bf16x2(v[2] - __uint_as_float(h1 << 16), v[3] - __uint_as_float(h1 & 0xffff0000u)));
      }
  };

  // a chunk's rows, registers one chunk ahead
  uint4 creg[CN], breg[CN], xreg[CX];
#pragma unroll
  for (int i = 0; i < CN; ++i) creg[i] = breg[i] = make_uint4(0, 0, 0, 0);
#pragma unroll
  for (int i = 0; i < CX; ++i) xreg[i] = make_uint4(0, 0, 0, 0);
  float dt_now = 0.f, dec_now = 0.f;
  auto piece = [&](const T *row, int d, int len) __attribute__((always_inline)) {     // 8 values from d on, zeros from len on
    Pack16 t;
    t.u = make_uint4(0, 0, 0, 0);
    if (VEC) {
      if (d < len) t.u = *reinterpret_cast<const uint4 *>(row + d);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (d + e < len) t.s[e] = row[d + e];
    }
    return t.u;
  };
  // byte offsets of this thread's pieces in a full chunk
  unsigned int boff[CN], xoff[CX];
#pragma unroll
  for (int i = 0; i < CN; ++i) {
    const int item = tid + i * TH, r = min(item / (NP / 8), kSC - 1), d = item % (NP / 8) * 8;
    boff[i] = static_cast<unsigned int>(r * a.channels + (d < a.N ? d : 0)) * 2;
  }
#pragma unroll
  for (int i = 0; i < CX; ++i) {
    const int item = tid + i * TH, r = min(item / (PS / 8), kSC - 1), d = item % (PS / 8) * 8;
    xoff[i] = static_cast<unsigned int>(r * a.channels + (d < a.P - p0 ? d : 0)) * 2;
  }
  auto load = [&](int c) __attribute__((always_inline)) {
    const int64_t r0 = begin - a.first_row + static_cast<int64_t>(c) * kSC;
    const int len = min(kSC, tokens - c * kSC);
    const T *first = static_cast<const T *>(a.xbc) + r0 * a.channels;               // uniform
    const T *bp = first + a.inner + grp * a.N, *cp = bp + a.G * a.N, *xp = first + h * a.P + p0;
    const int64_t at = (r0 + min(lane, len - 1)) * a.H + h;
    dt_now = lane < len ? a.dt[at] : 0.f;
    dec_now = lane < len ? a.decay[at] : 0.f;
    if (VEC && len == kSC) {
#pragma unroll
      for (int i = 0; i < CN; ++i) {
        breg[i] = *reinterpret_cast<const uint4 *>(reinterpret_cast<const char *>(bp) + boff[i]);
        if (MODE != 1) creg[i] = *reinterpret_cast<const uint4 *>(reinterpret_cast<const char *>(cp) + boff[i]);
      }
#pragma unroll
      for (int i = 0; i < CX; ++i) xreg[i] = *reinterpret_cast<const uint4 *>(reinterpret_cast<const char *>(xp) + xoff[i]);
      return;
    }
#pragma unroll
    for (int i = 0; i < CN; ++i) {
      const int item = tid + i * TH, r = min(item / (NP / 8), len - 1), d = item % (NP / 8) * 8;
      breg[i] = piece(bp + static_cast<int64_t>(r) * a.channels, d, a.N);
      if (MODE != 1) creg[i] = piece(cp + static_cast<int64_t>(r) * a.channels, d, a.N);
    }
#pragma unroll
    for (int i = 0; i < CX; ++i) {
      const int item = tid + i * TH, r = min(item / (PS / 8), len - 1), d = item % (PS / 8) * 8;
      xreg[i] = piece(xp + static_cast<int64_t>(r) * a.channels, d, a.P - p0);
    }
  };
  float total = 0.f;                                 // log2 decay of the whole segment
  float end_decay = 1.f;                             // 2^(c_end) of the chunk in LDS
  auto store = [&]() __attribute__((always_inline)) {
    const float c = ssd_wave_scan(dec_now);          // every wave has all 64 tokens, a lane each
    const float c_end = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(c), 63));
    total += c_end;
    end_decay = __builtin_amdgcn_exp2f(c_end);
    if (wave == 0) {
      cum[lane] = c;
      dts[lane] = dt_now;
      into_end[lane] = dt_now * __builtin_amdgcn_exp2f(c_end - c);
    }
#pragma unroll
    for (int i = 0; i < CN; ++i) {
      const int item = tid + i * TH, r = item / (NP / 8), d = item % (NP / 8) * 8;
      if (r < kSC) {
        const bool in = !VEC || d < a.N;             // pads are zeros
        *reinterpret_cast<uint4 *>(&Bs[r][d]) = in ? breg[i] : make_uint4(0, 0, 0, 0);
        if (MODE != 1) *reinterpret_cast<uint4 *>(&Cs[MODE == 1 ? 0 : r][d]) = in ? creg[i] : make_uint4(0, 0, 0, 0);
      }
    }
#pragma unroll
    for (int i = 0; i < CX; ++i) {
      const int item = tid + i * TH, r = item / (PS / 8), d = item % (PS / 8) * 8;
      if (r < kSC) *reinterpret_cast<uint4 *>(&Xs[r][d]) = !VEC || d < a.P - p0 ? xreg[i] : make_uint4(0, 0, 0, 0);
    }
  };

  const float D = MODE == 1 ? 0.f : Elem<T>::ld(static_cast<const T *>(a.D) + h);
  const int krow = (n >> 2) * 8 + (n & 3);           // s rows of a 32-row block as two 16-row tiles (+ 4)
  const int vrow = g * 8 + (n >> 2), vcol = (n & 3) * 4;
  const int tt = wave & 3, py = NW == 8 ? wave / 4 * PTY : 0;        // this wave's tokens and first column tile of Y
  if (c0 < c1) {
    load(c0);
    put_state();
    store();
  }
  for (int c = c0; c < c1; ++c) {
    const int t = tt * 16 + n, tok = c * kSC + t;    // this lane's token
    const int64_t row = begin + min(tok, tokens - 1);
    uint2 zr[PTY];
    if constexpr (MODE != 1) {
      const T *zp = static_cast<const T *>(a.proj) + row * a.ld + h * a.P + p0;
#pragma unroll
      for (int i = 0; i < PTY; ++i) {
        const int p = (py + i) * 16 + g * 4;
        zr[i] = make_uint2(0, 0);
        if (VEC) {
          if (p0 + p < a.P) zr[i] = *reinterpret_cast<const uint2 *>(zp + p);
        } else {
          unsigned int z[4] = {0, 0, 0, 0};
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (p0 + p + r < a.P) z[r] = zp[p + r];
          zr[i] = make_uint2(z[0] | z[1] << 16, z[2] | z[3] << 16);
        }
      }
    }
    if (c + 1 < c1) load(c + 1);
    lds_barrier();
    if constexpr (MODE != 1) {
      bf16x8 cf[NN];
#pragma unroll
      for (int k = 0; k < NN; ++k) {
        Pack16 x;
        x.u = *reinterpret_cast<const uint4 *>(&Cs[t][k * 32 + g * 8]);
        cf[k] = x.v;
      }
      floatx4 y[PTY], yl[PTY], yi[PTY], yil[PTY];    // sums over the pairs' halves apart: neighbouring products do not wait for each other
#pragma unroll
      for (int i = 0; i < PTY; ++i) y[i] = yl[i] = yi[i] = yil[i] = floatx4{0.f, 0.f, 0.f, 0.f};
      const float ct = cum[t];
#pragma unroll
      for (int k = 0; k < NN; ++k)
#pragma unroll
        for (int i = 0; i < PTY; ++i) {
          yi[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ssd_tr(&Sh[k * 32 + vrow][(py + i) * 16 + vcol], LX), cf[k], yi[i], 0, 0, 0);
          yil[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ssd_tr(&Sl[k * 32 + vrow][(py + i) * 16 + vcol], LX), cf[k], yil[i], 0, 0, 0);
        }
      for (int blk = 0; blk <= tt / 2; ++blk) {      // 32 tokens s; none lies wholly behind the wave's
        floatx4 g0 = floatx4{0.f, 0.f, 0.f, 0.f}, g1 = g0;
#pragma unroll
        for (int k = 0; k < NN; ++k) {
          Pack16 b0, b1;
          b0.u = *reinterpret_cast<const uint4 *>(&Bs[blk * 32 + krow][k * 32 + g * 8]);
          b1.u = *reinterpret_cast<const uint4 *>(&Bs[blk * 32 + krow + 4][k * 32 + g * 8]);
          g0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b0.v, cf[k], g0, 0, 0, 0);
          g1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b1.v, cf[k], g1, 0, 0, 0);
        }
        float cs8[8], d8[8], m[8];
        Elem<float>::ld8(&cum[blk * 32 + g * 8], cs8);
        Elem<float>::ld8(&dts[blk * 32 + g * 8], d8);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float v = e < 4 ? g0[e & 3] : g1[e & 3];
          m[e] = v * d8[e] * __builtin_amdgcn_exp2f(ct - cs8[e]);
        }
        if (blk == tt / 2) {                         // the diagonal; an exponent above 0 is dropped here
          const int last = t - blk * 32 - g * 8;
#pragma unroll
          for (int e = 0; e < 8; ++e) m[e] = e <= last ? m[e] : 0.f;
        }
        uint4 mh, ml;
        ssd_pair(m, mh, ml);
#pragma unroll
        for (int i = 0; i < PTY; ++i) {
          const bf16x8 xv = ssd_tr(&Xs[blk * 32 + vrow][(py + i) * 16 + vcol], LX);
          y[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xv, __builtin_bit_cast(bf16x8, mh), y[i], 0, 0, 0);
          yl[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xv, __builtin_bit_cast(bf16x8, ml), yl[i], 0, 0, 0);
        }
      }
      const float into = __builtin_amdgcn_exp2f(ct);
      if (tok < tokens) {
        T *op = static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(h) * a.P + p0;
#pragma unroll
        for (int i = 0; i < PTY; ++i) {
          const int p = (py + i) * 16 + g * 4;
          if (p0 + p >= a.P) continue;
          float o[4];
          const uint2 xr = *reinterpret_cast<const uint2 *>(&Xs[t][p]);
          const float x[4] = {__uint_as_float(xr.x << 16), __uint_as_float(xr.x & 0xffff0000u), __uint_as_float(xr.y << 16), __uint_as_float(xr.y & 0xffff0000u)};
          const float z[4] = {__uint_as_float(zr[i].x << 16), __uint_as_float(zr[i].x & 0xffff0000u), __uint_as_float(zr[i].y << 16),
                              __uint_as_float(zr[i].y & 0xffff0000u)};
#pragma unroll
          for (int r = 0; r < 4; ++r) o[r] = fmaf(D, x[r], fmaf(into, yi[i][r] + yil[i][r], y[i][r] + yl[i][r])) * ssd_silu<T>(z[r]);
          if (VEC) *reinterpret_cast<uint2 *>(op + p) = make_uint2(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]));
          else
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (p0 + p + r < a.P) Elem<T>::st(op + p + r, o[r]);
        }
      }
    }
    if (has_state) {
#pragma unroll
      for (int j = 0; j < NTW; ++j)
#pragma unroll
        for (int i = 0; i < PTU; ++i) S[j][i] *= end_decay;
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        float f[8];
        Elem<float>::ld8(&into_end[ks * 32 + g * 8], f);
        uint4 bh[NTW], bl[NTW];                      // B rows times dt 2^(c_end - c)
#pragma unroll
        for (int j = 0; j < NTW; ++j) {
          float b[8];
          unpack8(__builtin_bit_cast(uint4, ssd_tr(&Bs[ks * 32 + vrow][(nt0 + j) * 16 + vcol], LN)), b);
#pragma unroll
          for (int e = 0; e < 8; ++e) b[e] *= f[e];
          ssd_pair(b, bh[j], bl[j]);
        }
        bf16x8 xv[PTU];
#pragma unroll
        for (int i = 0; i < PTU; ++i) xv[i] = ssd_tr(&Xs[ks * 32 + vrow][(pt0 + i) * 16 + vcol], LX);
#pragma unroll
        for (int j = 0; j < NTW; ++j) {
#pragma unroll
          for (int i = 0; i < PTU; ++i) S[j][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xv[i], __builtin_bit_cast(bf16x8, bh[j]), S[j][i], 0, 0, 0);
#pragma unroll
          for (int i = 0; i < PTU; ++i) S[j][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xv[i], __builtin_bit_cast(bf16x8, bl[j]), S[j][i], 0, 0, 0);
        }
      }
    }
    lds_barrier();
    if (c + 1 < c1) {
      put_state();
      store();
    }
  }
  if constexpr (MODE == 1) {
    if (tid == 0 && slice == 0) a.seg_decay[sg] = __builtin_amdgcn_exp2f(total);
  } else {
    if (!last_seg || !slot_ok || tokens == 0) return;
  }
  if (!has_state) return;
  float *dst = MODE == 1 ? gst : st;
#pragma unroll
  for (int j = 0; j < NTW; ++j)
#pragma unroll
    for (int i = 0; i < PTU; ++i) {
      const int d = (nt0 + j) * 16 + n, p = p0 + (pt0 + i) * 16 + g * 4;
      if (d < a.N) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (p + r < a.P) dst[static_cast<int64_t>(d) * a.P + p + r] = S[j][i][r];
      }
    }
}

// Contributions of the segments -> the state each of them starts from, in place.
__global__ __launch_bounds__(256) void ssd_segments_kernel(const SsdArgs a) {
  const int64_t plane = static_cast<int64_t>(a.N) * a.P, e = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  const int h = blockIdx.y, sq = blockIdx.z;
  if (e >= plane) return;
  const int slot = a.state_slots[a.first_seq + sq];
  const bool from_zero = slot < 0 || slot >= a.num_slots || a.starts[a.first_seq + sq] == 0;
  float run = from_zero ? 0.f : a.state[(static_cast<int64_t>(slot) * a.H + h) * plane + e];
  for (int s = 0; s < a.segs; ++s) {
    const int64_t sg = (static_cast<int64_t>(sq) * a.segs + s) * a.H + h;
    const bool more = s < a.segs - 1;
    const float own = more ? a.seg_state[sg * plane + e] : 0.f, dec = more ? a.seg_decay[sg] : 0.f;
    a.seg_state[sg * plane + e] = run;
    run = fmaf(dec, run, own);
  }
}

// Columns of P per workgroup in units of 16: what fits LDS beside the state.
int ssd_columns(int N, int P) {
  const int most = N <= 128 ? 4 : 2, need = (P + 15) / 16;
  return need <= 1 ? 1 : need <= 2 || most == 2 ? 2 : 4;
}
bool ssd_chunked(int N, int P, int dtype) { return dtype == TLF_DT_BF16 && N <= 256; }
// Segments per sequence: enough workgroups for the chip, segments of at least 4 chunks.
int ssd_segments(int64_t wgs, int max_tokens) {
  const int64_t want = wgs >= 192 ? 1 : (384 + wgs - 1) / wgs, most = (max_tokens + kSC - 1) / kSC / 4;
  return static_cast<int>(std::max<int64_t>(1, std::min<int64_t>({want, most, 64})));
}

struct SsdPlan {
  bool chunked;
  int pt, slices, segs;
  size_t xbc, steps, seg_state, seg_decay;           // bytes; `steps` twice
};
SsdPlan ssd_plan(int rows, int seqs, int max_tokens, int H, int P, int N, int G, int dtype) {
  SsdPlan p{};
  const size_t item = dtype == TLF_DT_BF16 ? 2 : 4;
  auto up = [](size_t v) { return (v + 255) & ~static_cast<size_t>(255); };
  p.chunked = ssd_chunked(N, P, dtype);
  p.pt = ssd_columns(N, P);
  p.slices = (P + 16 * p.pt - 1) / (16 * p.pt);
  p.segs = p.chunked ? ssd_segments(static_cast<int64_t>(H) * p.slices * seqs, max_tokens) : 1;
  if (static_cast<int64_t>(seqs) * p.segs > 65535) p.segs = 1;
  p.xbc = up(item * rows * (static_cast<size_t>(H) * P + 2 * static_cast<size_t>(G) * N));
  p.steps = up(4 * static_cast<size_t>(rows) * H);
  const size_t sg = p.segs > 1 ? static_cast<size_t>(seqs) * p.segs * H : 0;
  p.seg_decay = up(4 * sg);
  p.seg_state = up(4 * sg * N * P);
  return p;
}

int ssd_check(SsdArgs &a, int32_t dtype) {
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (a.rows < 0 || a.H <= 0 || a.H > 65535 || a.P <= 0 || a.N <= 0 || a.G <= 0 || a.H % a.G || a.P > kSsdMaxP || a.N > kSsdMaxN) return TLF_E_SHAPE;
  if (a.taps < 1 || a.taps > 64 || a.num_slots <= 0) return TLF_E_SHAPE;
  const int64_t inner = static_cast<int64_t>(a.H) * a.P, channels = inner + 2ll * a.G * a.N;
  if (inner + channels + a.H > (1 << 28) || a.ld < inner + channels + a.H || a.ldo < inner) return TLF_E_SHAPE;
  a.inner = static_cast<int32_t>(inner);
  a.channels = static_cast<int32_t>(channels);
  if (a.rows == 0) return TLF_OK;
  if ((!a.proj && a.part.splits <= 1) || !a.conv || !a.conv_bias || !a.dt_bias || !a.A_log || !a.D || !a.ring || !a.state || !a.state_slots ||
      !a.positions || !a.out)
    return TLF_E_NULL;
  return TLF_OK;
}
int ssd_lanes(int P, bool vec) {
  int lanes = 4;
  while (lanes < 64 && lanes * (vec ? 4 : 1) < P) lanes *= 2;
  return lanes;
}

template <typename T>
int launch_ssd_conv(const SsdArgs &a, hipStream_t s) {
  const bool vec = a.channels % 8 == 0 && a.inner % 8 == 0 && a.ld % 8 == 0 && aligned16(a.proj) && aligned16(a.conv) && aligned16(a.conv_bias) &&
                   aligned16(a.ring) && aligned16(a.xbc);
#define TLF_SC(VEC, TAPS, TOK)                                                                                                    \
  TLF_LAUNCH((ssd_conv_kernel<T, VEC, TAPS, TOK>),                                                                                \
             dim3((a.rows + (TOK) - 1) / (TOK), (a.channels + 256 * (VEC) - 1) / (256 * (VEC)) + 1), dim3(256), 0, s, a)
  if (vec) {
    switch (a.taps) {
      case 2: if (a.rows >= 2048) TLF_SC(8, 2, 8); else TLF_SC(8, 2, 2); break;
      case 3: if (a.rows >= 2048) TLF_SC(8, 3, 8); else TLF_SC(8, 3, 2); break;
      case 4: if (a.rows >= 2048) TLF_SC(8, 4, 8); else TLF_SC(8, 4, 2); break;
      default: TLF_SC(8, 0, 1); break;
    }
  } else {
    TLF_SC(1, 0, 1);
  }
#undef TLF_SC
  return launch_status();
}

template <int NN, int PT, bool VEC>
void launch_ssd_chunks(const SsdArgs &a, hipStream_t s) {
  const dim3 grid(a.H, a.slices, a.seqs * a.segs);
  const dim3 block(ssd_waves<PT>() * 64);
  if (a.segs == 1) {
    TLF_LAUNCH((ssd_chunk_kernel<NN, PT, 0, VEC>), grid, block, 0, s, a);
    return;
  }
  TLF_LAUNCH((ssd_chunk_kernel<NN, PT, 1, VEC>), grid, block, 0, s, a);
  TLF_LAUNCH(ssd_segments_kernel, dim3((a.N * a.P + 255) / 256, a.H, a.seqs), dim3(256), 0, s, a);
  TLF_LAUNCH((ssd_chunk_kernel<NN, PT, 2, VEC>), grid, block, 0, s, a);
}

}  // namespace tlf

extern "C" int tlf_ssd_decode(const void *proj, int64_t proj_stride, const float *partials, int32_t splits, const float *scale,
                              const void *conv, const void *conv_bias, int32_t taps, const void *dt_bias, const void *A_log,
                              const void *D, void *ring, float *state, const int32_t *state_slots, int32_t num_slots,
                              const int64_t *positions, void *out, int64_t out_stride, int32_t rows, int32_t heads, int32_t vdim,
                              int32_t state_dim, int32_t groups, int32_t dtype, void *stream) {
  using namespace tlf;
  SsdArgs a{};
  a.proj = proj; a.ld = proj_stride; a.part = Partials{partials, scale, rows * proj_stride, static_cast<int32_t>(proj_stride), splits};
  a.conv = conv; a.conv_bias = conv_bias; a.taps = taps; a.dt_bias = dt_bias; a.A_log = A_log; a.D = D; a.ring = ring; a.state = state;
  a.state_slots = state_slots; a.num_slots = num_slots; a.positions = positions; a.out = out; a.ldo = out_stride; a.rows = rows;
  a.H = heads; a.P = vdim; a.N = state_dim; a.G = groups;
  if (int rc = partials_check(partials, scale, splits, dtype)) return rc;
  if (int rc = ssd_check(a, dtype)) return rc;
  if (rows > 65535) return TLF_E_SHAPE;
  if (rows == 0) return TLF_OK;
  const bool vec = vdim % 4 == 0 && aligned16(state);
  const int lanes = ssd_lanes(vdim, vec);
  const dim3 grid(heads, rows);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define TLF_SD(T, PART)                                                                                         \
  do {                                                                                                          \
    if (vec) TLF_LAUNCH((ssd_decode_kernel<T, 4, PART>), grid, dim3(256), 0, s, a, lanes);                      \
    else TLF_LAUNCH((ssd_decode_kernel<T, 1, PART>), grid, dim3(256), 0, s, a, lanes);                          \
  } while (0)
  if (splits > 1) TLF_SD(unsigned short, true);
  else if (dtype == TLF_DT_BF16) TLF_SD(unsigned short, false);
  else TLF_SD(float, false);
#undef TLF_SD
  return launch_status();
}

extern "C" size_t tlf_ssd_portions_workspace_bytes(int32_t rows, int32_t num_seqs, int32_t max_tokens, int32_t heads, int32_t vdim,
                                                   int32_t state_dim, int32_t groups, int32_t dtype) {
  if (rows <= 0 || num_seqs <= 0 || max_tokens <= 0 || heads <= 0 || vdim <= 0 || state_dim <= 0 || groups <= 0) return 0;
  const tlf::SsdPlan p = tlf::ssd_plan(rows, num_seqs, max_tokens, heads, vdim, state_dim, groups, dtype);
  return p.xbc + 2 * p.steps + p.seg_decay + p.seg_state;
}

extern "C" int tlf_ssd_portions(const void *proj, int64_t proj_stride, const void *conv, const void *conv_bias, int32_t taps,
                                const void *dt_bias, const void *A_log, const void *D, void *ring, float *state,
                                const int32_t *state_slots, int32_t num_slots, const int64_t *positions, const int32_t *row_seq,
                                const int32_t *cu_seqlens_q, const int32_t *seq_starts, int32_t first_seq, int32_t num_seqs,
                                int32_t first_row, int32_t max_tokens, void *out, int64_t out_stride, int32_t rows, int32_t heads,
                                int32_t vdim, int32_t state_dim, int32_t groups, int32_t dtype, void *workspace,
                                size_t workspace_bytes, void *stream) {
  using namespace tlf;
  SsdArgs a{};
  a.proj = proj; a.ld = proj_stride; a.conv = conv; a.conv_bias = conv_bias; a.taps = taps; a.dt_bias = dt_bias; a.A_log = A_log;
  a.D = D; a.ring = ring; a.state = state; a.state_slots = state_slots; a.num_slots = num_slots; a.positions = positions;
  a.row_seq = row_seq; a.cu_q = cu_seqlens_q; a.starts = seq_starts; a.out = out; a.ldo = out_stride; a.rows = rows;
  a.H = heads; a.P = vdim; a.N = state_dim; a.G = groups; a.first_seq = first_seq; a.seqs = num_seqs; a.first_row = first_row;
  if (int rc = ssd_check(a, dtype)) return rc;
  if (first_seq < 0 || num_seqs < 0 || num_seqs > 65535 || first_row < 0 || max_tokens < 0) return TLF_E_SHAPE;
  if (rows == 0 || num_seqs == 0 || max_tokens == 0) return TLF_OK;
  if (!row_seq || !cu_seqlens_q || !seq_starts) return TLF_E_NULL;
  const SsdPlan p = ssd_plan(rows, num_seqs, max_tokens, heads, vdim, state_dim, groups, dtype);
  if (!workspace || !aligned16(workspace) || workspace_bytes < p.xbc + 2 * p.steps + p.seg_decay + p.seg_state) return TLF_E_WORKSPACE;
  char *ws = static_cast<char *>(workspace);
  a.xbc = ws;
  a.dt = reinterpret_cast<float *>(ws + p.xbc);
  a.decay = reinterpret_cast<float *>(ws + p.xbc + p.steps);
  a.seg_decay = reinterpret_cast<float *>(ws + p.xbc + 2 * p.steps);
  a.seg_state = reinterpret_cast<float *>(ws + p.xbc + 2 * p.steps + p.seg_decay);
  a.segs = p.segs; a.slices = p.slices;
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (int rc = dtype == TLF_DT_BF16 ? launch_ssd_conv<unsigned short>(a, s) : launch_ssd_conv<float>(a, s)) return rc;
  if (!p.chunked) {
    const bool vec = vdim % 4 == 0 && aligned16(state);
    const int lanes = ssd_lanes(vdim, vec);
    const dim3 grid(heads, num_seqs);
    if (dtype == TLF_DT_BF16) {
      if (vec) TLF_LAUNCH((ssd_scan_kernel<unsigned short, 4>), grid, dim3(256), 0, s, a, lanes);
      else TLF_LAUNCH((ssd_scan_kernel<unsigned short, 1>), grid, dim3(256), 0, s, a, lanes);
    } else {
      if (vec) TLF_LAUNCH((ssd_scan_kernel<float, 4>), grid, dim3(256), 0, s, a, lanes);
      else TLF_LAUNCH((ssd_scan_kernel<float, 1>), grid, dim3(256), 0, s, a, lanes);
    }
    return launch_status();
  }
  // pieces of 8: channels, groups and heads begin at multiples of 8
  const bool vec = vdim % 8 == 0 && state_dim % 8 == 0 && a.channels % 8 == 0 && a.ld % 4 == 0 && out_stride % 4 == 0 &&
                   (reinterpret_cast<uintptr_t>(proj) & 7) == 0 && (reinterpret_cast<uintptr_t>(out) & 7) == 0;
#define TLF_SK(NN, PT)                                      \
  do {                                                      \
    if (vec) launch_ssd_chunks<NN, PT, true>(a, s);         \
    else launch_ssd_chunks<NN, PT, false>(a, s);            \
  } while (0)
#define TLF_SK_P(NN)              \
  do {                            \
    if (p.pt == 1) TLF_SK(NN, 1); \
    else if (p.pt == 2) TLF_SK(NN, 2); \
    else TLF_SK(NN, 4);           \
  } while (0)
  if (state_dim <= 32) TLF_SK_P(1);
  else if (state_dim <= 64) TLF_SK_P(2);
  else if (state_dim <= 128) TLF_SK_P(4);
  else if (p.pt == 1) TLF_SK(8, 1);
  else TLF_SK(8, 2);
#undef TLF_SK_P
#undef TLF_SK
  return launch_status();
}
