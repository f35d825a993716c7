// Gated linear attention with a decay per key channel.  Per head, with fp32 state S [dk, dv]:
//
//   z_t = W_a2 r_t + b,  alpha_t = sigmoid(z_t)^(1/tau),  S_t = diag(alpha_t) S_{t-1} + k_t v_t^T,  o_t = S_t^T q_t
//   out = rms_norm(o) * w * silu(g)            (norm over dv, one weight for all heads)
//
// Input is one projection row per token, [q | k | v | g | r] (H*dk, H*dk, H*dv, H*dv, R values); q is scaled by
// dk^-1/2 here.  Everything from z on is fp32.
//
//   gla_decode_kernel  one token: one workgroup per (row, head) streams the state through once (HBM bound: 8 dk dv
//                      bytes per head), norm and output gate included
//   portions of prompts, three kernels over chunks of 16 tokens (a chunk never crosses a sequence):
//   gla_chunk_kernel   per (chunk, head), parallel: decays b_t = sum of log2 alpha within the chunk,
//                      Qd = q 2^b_t, Kd = k 2^(b_end - b_t), A[t, s] = sum_d q k 2^(b_t - b_s) for s <= t.  The
//                      exponents of A are formed pair by pair: every factor is <= 1, whatever the decay
//   gla_scan_kernel    per (sequence, head, 16 columns of v), one wave each, sequential over the chunks:
//                      O = Qd S + A V;  S = diag(2^b_end) S + Kd^T V.  All products are v_mfma_f32_16x16x4_f32; the
//                      state stays in accumulator registers, whose layout (row 4 g + r of a tile in register r of
//                      lane group g) is the B operand of the next product when its summation index is labelled
//                      4 g + r in step r.  Where (sequences, heads, columns) alone leave SIMDs
//                      idle, a sequence is cut into segments: a first pass carries each segment's own contribution
//                      from zero (half the work), gla_segments_kernel chains them, and the scan starts every segment
//                      from its state
//   gla_out_kernel     norm and output gate
#include "elem.h"

namespace tlf {

constexpr int kGlaMaxDk = 256, kGlaMaxDv = 512, kGlaMaxR = 256;

struct GlaArgs {
  const void *proj;        // [n, ld]
  Partials part;           // decode: or its partial sums
  int64_t ld;
  const void *a2;          // [H * dk, R]
  const void *a2_bias;     // [H * dk]
  const void *norm_w;      // [dv]
  float *state;            // [slots, H, dk, dv]
  const int32_t *state_slots;
  int32_t num_slots;
  const int64_t *positions;   // decode: [rows]
  void *out;               // [n, ldo]
  int64_t ldo;
  int32_t rows, H, dk, dv, R;
  float inv_tau, q_scale, eps;
  // portions
  const int32_t *chunk_tok, *chunk_len;   // [chunks]: first row of the chunk in the step, tokens in it
  const int32_t *cu_chunks;               // [seqs + 1]
  const int32_t *starts;                  // [seqs]: tokens before this step, 0: the state starts at zero
  int32_t chunks, seqs;
  // workspace.  One record per (chunk, head): Qd, Kd, A, decays, 64 floats of padding (records a power of two apart
  // would fall into few sets of the L2); o: [chunks, H, 16, dv]
  float *rec, *o;
  int32_t vec;                            // bf16 projection rows may be read 8 bytes at a time, key dim a full row
  int32_t segs;                           // segments per sequence
  float *seg_state, *seg_dec;             // [seqs, segs, H, dk, dv], [seqs, segs, H, DKP]
};

// log2 of sigmoid(z)^(1/tau) = -(max(-z, 0) log2 e + log2(1 + e)) / tau with e = 2^(-|z| log2 e).  log2(1 + e) keeps its
// relative accuracy for small e: the rounding of u = 1 + e is undone by the factor e / (u - 1).
__device__ __forceinline__ float log2_alpha(float z, float inv_tau) {
  const float kL2e = 1.4426950408889634f;
  const float e = __builtin_amdgcn_exp2f(-fabsf(z) * kL2e);
  const float u = 1.0f + e, d = u - 1.0f;
  const float l = d == 0.f ? e * kL2e : __builtin_amdgcn_logf(u) * e * __builtin_amdgcn_rcpf(d);
  return -fmaf(fmaxf(-z, 0.f), kL2e, l) * inv_tau;
}

template <int VEC>
struct Vf {
  float f[VEC];
};
template <int VEC>
__device__ __forceinline__ Vf<VEC> ldf(const float *p) {
  Vf<VEC> r;
  if constexpr (VEC == 4) {
    const float4 t = *reinterpret_cast<const float4 *>(p);
    r.f[0] = t.x; r.f[1] = t.y; r.f[2] = t.z; r.f[3] = t.w;
  } else {
    r.f[0] = *p;
  }
  return r;
}
template <int VEC>
__device__ __forceinline__ void stf(float *p, const Vf<VEC> &v) {
  if constexpr (VEC == 4) *reinterpret_cast<float4 *>(p) = make_float4(v.f[0], v.f[1], v.f[2], v.f[3]);
  else *p = v.f[0];
}

template <typename T, int VEC, bool PART>
__global__ __launch_bounds__(256) void gla_decode_kernel(const GlaArgs a, int lanes_v) {
  __shared__ float qs[kGlaMaxDk], ks[kGlaMaxDk], al[kGlaMaxDk], rs[kGlaMaxR];
  __shared__ __attribute__((aligned(16))) float osum[2048];
  __shared__ float part[4];
  const int row = blockIdx.y, h = blockIdx.x, tid = threadIdx.x;
  const int slot = a.state_slots[row];
  T *out = static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(h) * a.dv;
  if (slot < 0 || slot >= a.num_slots) {             // padding row of a captured graph
    for (int v = tid; v < a.dv; v += 256) Elem<T>::st(out + v, 0.f);
    return;
  }
  const T *pr = static_cast<const T *>(a.proj) + row * a.ld;
  const int64_t hk = static_cast<int64_t>(a.H) * a.dk, hv = static_cast<int64_t>(a.H) * a.dv;
  auto in = [&](int64_t col) __attribute__((always_inline)) {
    return PART ? a.part.ld(row, static_cast<int>(col)) : Elem<T>::ld(pr + col);
  };
  const int64_t q0 = h * a.dk, k0 = hk + h * a.dk, v0 = 2 * hk + h * a.dv, g0 = v0 + hv, r0 = 2 * hk + 2 * hv;
  for (int r = tid; r < a.R; r += 256) rs[r] = in(r0 + r);
  if (tid < a.dk) {
    qs[tid] = in(q0 + tid) * a.q_scale;
    ks[tid] = in(k0 + tid);
  }
  __syncthreads();
  const bool fresh = a.positions[row] == 0;
  if (tid < a.dk) {
    const T *w = static_cast<const T *>(a.a2) + (static_cast<int64_t>(h) * a.dk + tid) * a.R;
    float z = Elem<T>::ld(static_cast<const T *>(a.a2_bias) + h * a.dk + tid);
    for (int r = 0; r < a.R; ++r) z = fmaf(Elem<T>::ld(w + r), rs[r], z);
    al[tid] = fresh ? 0.f : exp2f(log2_alpha(z, a.inv_tau));
  }
  __syncthreads();
  const int team = tid / lanes_v, lane = tid % lanes_v, teams = 256 / lanes_v;
  const int nvc = a.dv / VEC;
  float *st = a.state + (static_cast<int64_t>(slot) * a.H + h) * a.dk * a.dv;
  for (int c = lane; c < nvc; c += lanes_v) {
    Vf<VEC> o, v;
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      o.f[e] = 0.f;
      v.f[e] = in(v0 + c * VEC + e);
    }
    constexpr int U = 8;
    for (int d0 = team; d0 < a.dk; d0 += teams * U) {
      Vf<VEC> s[U];
#pragma unroll
      for (int u = 0; u < U; ++u) s[u] = ldf<VEC>(st + static_cast<int64_t>(min(d0 + u * teams, a.dk - 1)) * a.dv + c * VEC);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int d = d0 + u * teams;
        if (d < a.dk) {
          const float al_d = al[d], k_d = ks[d], q_d = qs[d];
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            s[u].f[e] = fresh ? k_d * v.f[e] : fmaf(al_d, s[u].f[e], k_d * v.f[e]);
            o.f[e] = fmaf(s[u].f[e], q_d, o.f[e]);
          }
          stf<VEC>(st + static_cast<int64_t>(d) * a.dv + c * VEC, s[u]);
        }
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) osum[team * a.dv + c * VEC + e] = o.f[e];
  }
  __syncthreads();
  float ov[2], ss = 0.f;                             // dv <= 512: at most two columns per thread
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int v = tid + i * 256;
    ov[i] = 0.f;
    if (v < a.dv)
      for (int t = 0; t < teams; ++t) ov[i] += osum[t * a.dv + v];
    ss = fmaf(ov[i], ov[i], ss);
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) part[tid >> 6] = ss;
  __syncthreads();
  ss = part[0] + part[1] + part[2] + part[3];
  const float inv = 1.0f / sqrtf(ss / static_cast<float>(a.dv) + a.eps);
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int v = tid + i * 256;
    if (v < a.dv)
      Elem<T>::st(out + v, ov[i] * inv * Elem<T>::ld(static_cast<const T *>(a.norm_w) + v) * silu_f32(in(g0 + v)));
  }
}

// ---------------------------------------------------------------------------------------------------------------
constexpr int kGC = 16;   // tokens per chunk
// offsets inside a record, in floats
template <int DKP>
struct GlaRec {
  static constexpr int kKd = DKP * kGC, kA = 2 * DKP * kGC, kDec = kA + kGC * kGC, kSize = kDec + DKP + 64;
};
int gla_rec_size(int dkp) { return 2 * dkp * kGC + kGC * kGC + dkp + 64; }

template <typename T, int NT>
__global__ __launch_bounds__(256) void gla_chunk_kernel(const GlaArgs a) {
  constexpr int DKP = NT * 16, LD = DKP + 4;
  __shared__ __attribute__((aligned(16))) float ks[kGC][LD], bs[kGC][LD], kh[8][LD];
  __shared__ __attribute__((aligned(16))) float rs[kGC][kGlaMaxR];
  const int chunk = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int64_t tok0 = a.chunk_tok[chunk];
  const int len = a.chunk_len[chunk];
  const int64_t hk = static_cast<int64_t>(a.H) * a.dk, hv = static_cast<int64_t>(a.H) * a.dv;
  const T *pr = static_cast<const T *>(a.proj) + tok0 * a.ld;
  for (int i = tid; i < kGC * a.R; i += 256) {
    const int t = i / a.R, r = i - t * a.R;
    rs[t][r] = t < len ? Elem<T>::ld(pr + t * a.ld + 2 * hk + 2 * hv + r) : 0.f;
  }
  __syncthreads();
  // decays: a thread has one channel and TPT of the 16 tokens, then one thread per channel sums them up
  constexpr int TEAMS = DKP <= 16 ? 16 : DKP <= 32 ? 8 : DKP <= 64 ? 4 : DKP <= 128 ? 2 : 1, TPT = kGC / TEAMS;
  {
    const int d = tid % (256 / TEAMS), t0 = tid / (256 / TEAMS) * TPT;
    if (d < DKP) {
      float z[TPT];
      const bool in = d < a.dk;
      const T *w = static_cast<const T *>(a.a2) + (static_cast<int64_t>(h) * a.dk + (in ? d : 0)) * a.R;
      const float b = Elem<T>::ld(static_cast<const T *>(a.a2_bias) + h * a.dk + (in ? d : 0));
#pragma unroll
      for (int t = 0; t < TPT; ++t) z[t] = b;
      int r = 0;
      for (; r + 4 <= a.R; r += 4) {
        float wr[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) wr[e] = Elem<T>::ld(w + r + e);
#pragma unroll
        for (int t = 0; t < TPT; ++t) {
          const float4 x = *reinterpret_cast<const float4 *>(&rs[t0 + t][r]);
          z[t] = fmaf(wr[0], x.x, z[t]);
          z[t] = fmaf(wr[1], x.y, z[t]);
          z[t] = fmaf(wr[2], x.z, z[t]);
          z[t] = fmaf(wr[3], x.w, z[t]);
        }
      }
      for (; r < a.R; ++r) {
        const float wr = Elem<T>::ld(w + r);
#pragma unroll
        for (int t = 0; t < TPT; ++t) z[t] = fmaf(wr, rs[t0 + t][r], z[t]);
      }
#pragma unroll
      for (int t = 0; t < TPT; ++t) bs[t0 + t][d] = in && t0 + t < len ? log2_alpha(z[t], a.inv_tau) : 0.f;
    }
  }
  // 16 lanes per token; lane l holds channels dmap(i): four at a time where the row length allows 16-byte LDS reads
  const int t = tid / 16, l = tid % 16;
  auto dmap = [&](int i) { return NT % 4 == 0 ? (i / 4) * 64 + l * 4 + i % 4 : l + 16 * i; };
  float q[NT];
  bool plain = true;
  if constexpr (NT % 4 == 0 && sizeof(T) == 2) {
    if (a.vec) {                                     // uniform: full rows, 8-byte aligned
      plain = false;
#pragma unroll
      for (int i = 0; i < NT; i += 4) {
        const T *p = pr + min(t, len - 1) * a.ld + h * a.dk + (i / 4) * 64 + l * 4;
        uint2 qr = *reinterpret_cast<const uint2 *>(p), kr = *reinterpret_cast<const uint2 *>(p + hk);
        if (t >= len) qr = kr = make_uint2(0, 0);
        q[i] = __uint_as_float(qr.x << 16) * a.q_scale; q[i + 1] = __uint_as_float(qr.x & 0xffff0000u) * a.q_scale;
        q[i + 2] = __uint_as_float(qr.y << 16) * a.q_scale; q[i + 3] = __uint_as_float(qr.y & 0xffff0000u) * a.q_scale;
        *reinterpret_cast<float4 *>(&ks[t][(i / 4) * 64 + l * 4]) =
            make_float4(__uint_as_float(kr.x << 16), __uint_as_float(kr.x & 0xffff0000u), __uint_as_float(kr.y << 16),
                        __uint_as_float(kr.y & 0xffff0000u));
      }
    }
  }
  if (plain) {
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int d = dmap(i);
      const bool in = d < a.dk && t < len;
      q[i] = in ? Elem<T>::ld(pr + t * a.ld + h * a.dk + d) * a.q_scale : 0.f;
      ks[t][d] = in ? Elem<T>::ld(pr + t * a.ld + hk + h * a.dk + d) : 0.f;
    }
  }
  __syncthreads();
  if (tid < DKP) {
    float b = 0.f;
#pragma unroll
    for (int s = 0; s < kGC; ++s) bs[s][tid] = b += bs[s][tid];
  }
  __syncthreads();
  const int64_t ch = static_cast<int64_t>(chunk) * a.H + h;
  float bt[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) bt[i] = bs[t][dmap(i)];
  // operand order of the scan: Qd [tile][t][16 channels], Kd [tile][channel][16 tokens]
  float *qd = a.rec + ch * GlaRec<DKP>::kSize, *kd = qd + GlaRec<DKP>::kKd;
  if constexpr (NT % 4 == 0) {
#pragma unroll
    for (int i = 0; i < NT; i += 4) {
      const int d = dmap(i);
      *reinterpret_cast<float4 *>(&qd[(d / 16) * 256 + t * 16 + d % 16]) =
          make_float4(q[i] * __builtin_amdgcn_exp2f(bt[i]), q[i + 1] * __builtin_amdgcn_exp2f(bt[i + 1]),
                      q[i + 2] * __builtin_amdgcn_exp2f(bt[i + 2]), q[i + 3] * __builtin_amdgcn_exp2f(bt[i + 3]));
    }
  } else {
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int d = dmap(i);
      qd[(d / 16) * 256 + t * 16 + d % 16] = q[i] * __builtin_amdgcn_exp2f(bt[i]);
    }
  }
  for (int i = tid; i < DKP * kGC; i += 256) {
    const int d = i / kGC, s = i % kGC;
    kd[i] = ks[s][d] * __builtin_amdgcn_exp2f(bs[kGC - 1][d] - bs[s][d]);
  }
  if (tid < DKP) qd[GlaRec<DKP>::kDec + tid] = __builtin_amdgcn_exp2f(bs[kGC - 1][tid]);
  // A[t, s].  For t >= 8 > s the factors 2^(b_t - b_7) and 2^(b_7 - b_s) are both <= 1 and the product needs no exponential
  // per pair; within each half the exponents are formed pair by pair.
  for (int i = tid; i < 8 * DKP; i += 256) {
    const int s = i / DKP, d = i % DKP;
    kh[s][d] = ks[s][d] * __builtin_amdgcn_exp2f(bs[7][d] - bs[s][d]);
  }
  __syncthreads();
  float *am = qd + GlaRec<DKP>::kA + t * kGC;
  const int half = tid / 128 * 8, smax = (tid / 64) * 4 + 3;   // wave uniform: first token of its half, its last token
  auto load_row = [&](const float *row, float (&v)[NT]) __attribute__((always_inline)) {
    if constexpr (NT % 4 == 0) {
#pragma unroll
      for (int i = 0; i < NT; i += 4) {
        const float4 x = *reinterpret_cast<const float4 *>(row + (i / 4) * 64 + l * 4);
        v[i] = x.x; v[i + 1] = x.y; v[i + 2] = x.z; v[i + 3] = x.w;
      }
    } else {
#pragma unroll
      for (int i = 0; i < NT; ++i) v[i] = row[l + 16 * i];
    }
  };
  float keep = 0.f;                                  // lane l of a token's 16 keeps A[t, l]
  if (half) {
    float b7[NT], qh[NT];
    load_row(bs[7], b7);
#pragma unroll
    for (int i = 0; i < NT; ++i) qh[i] = q[i] * __builtin_amdgcn_exp2f(bt[i] - b7[i]);
#pragma unroll
    for (int s = 0; s < 8; ++s) {
      float kv[NT], acc = 0.f;
      load_row(kh[s], kv);
#pragma unroll
      for (int i = 0; i < NT; ++i) acc = fmaf(qh[i], kv[i], acc);
      acc = group_sum<16>(acc);
      if (l == s) keep = acc;
    }
  }
  for (int s = half; s <= smax; ++s) {
    float kv[NT], bv[NT], acc = 0.f;
    load_row(ks[s], kv);
    load_row(bs[s], bv);
#pragma unroll
    for (int i = 0; i < NT; ++i) acc = fmaf(q[i] * kv[i], __builtin_amdgcn_exp2f(fminf(bt[i] - bv[i], 0.f)), acc);
    acc = group_sum<16>(acc);
    if (l == s) keep = acc;
  }
  am[l] = l <= t ? keep : 0.f;
}

// MODE 0: the whole sequence from the state slot and back.  MODE 1: a segment's own contribution from zero.  MODE 2: a
// segment from the state gla_segments_kernel left for it.  Operands come straight from the chunk's record, which holds
// them in operand order (1 KiB per tile and instruction): Qd of the next chunk is fetched behind the products with this
// one's, Kd and the decays while those run, V and A one chunk ahead.
template <typename T, int NT, int MODE>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(NT <= 8 ? 2 : 1))) void gla_scan_kernel(const GlaArgs a, int first_seq) {
  constexpr int DKP = NT * 16;
  using Rec = GlaRec<DKP>;
  const int tid = threadIdx.x, lane = tid & 63, n = lane & 15, g = lane >> 4;
  // heads vary fastest: with a multiple of 8 heads the workgroups of one head (same records) share an XCD's L2
  const int h = blockIdx.x, seq = MODE == 0 ? blockIdx.z : blockIdx.z / a.segs, seg = MODE == 0 ? 0 : blockIdx.z % a.segs;
  const bool last_seg = MODE == 0 || seg == a.segs - 1;
  if (MODE == 1 && last_seg) return;                 // nobody starts behind the last segment
  const int tile = blockIdx.y * 4 + (tid >> 6);      // 16 columns of v
  if (tile * 16 >= a.dv) return;                     // no barrier below: a wave may leave on its own
  const int slot = a.state_slots[first_seq + seq];
  const bool slot_ok = slot >= 0 && slot < a.num_slots;
  const bool fresh = a.starts[first_seq + seq] == 0;
  float *st = a.state + (static_cast<int64_t>(slot_ok ? slot : 0) * a.H + h) * a.dk * a.dv;
  const int64_t sg = ((static_cast<int64_t>(seq) * a.segs + seg) * a.H + h);
  float *gst = MODE == 0 ? st : a.seg_state + sg * a.dk * a.dv;
  const bool from_zero = MODE == 1 || (MODE == 0 && (fresh || !slot_ok));
  const bool cok = tile * 16 + n < a.dv;
  const int col = cok ? tile * 16 + n : 0;
  floatx4 S[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = i * 16 + g * 4 + r;
      S[i][r] = !from_zero && d < a.dk && cok ? gst[static_cast<int64_t>(d) * a.dv + col] : 0.f;
    }
  const int64_t hk = static_cast<int64_t>(a.H) * a.dk;
  const T *vbase = static_cast<const T *>(a.proj) + 2 * hk + static_cast<int64_t>(h) * a.dv + col;
  // a sequence's chunks follow each other and all but its last hold 16 tokens: rows come without a table lookup
  const int cbeg = a.cu_chunks[seq], cend = a.cu_chunks[seq + 1];
  const int64_t row_first = cbeg < cend ? a.chunk_tok[cbeg] : 0;
  const int len_last = cbeg < cend ? a.chunk_len[cend - 1] : 0;
  int c0 = cbeg, c1 = cend;
  if (MODE != 0) {
    const int per = (cend - cbeg + a.segs - 1) / a.segs;
    c0 = min(cbeg + seg * per, cend);
    c1 = min(c0 + per, cend);
  }
  float sd[MODE == 1 ? NT : 1][4];                   // decay of the whole segment
#pragma unroll
  for (int i = 0; i < (MODE == 1 ? NT : 1); ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) sd[i][r] = 1.f;

  const int at = n * 16 + g * 4;
  auto record = [&](int c) __attribute__((always_inline)) { return a.rec + (static_cast<int64_t>(c) * a.H + h) * Rec::kSize; };
  float4 qf[NT], an = make_float4(0.f, 0.f, 0.f, 0.f);
  T vn[4];                                           // converted when used: touching them earlier would wait for them
  auto load_q = [&](int c) __attribute__((always_inline)) {
    const float *p = record(c) + at;
#pragma unroll
    for (int i = 0; i < NT; ++i) qf[i] = *reinterpret_cast<const float4 *>(p + i * 256);
  };
  auto load_va = [&](int c) __attribute__((always_inline)) {
    const int64_t tok = row_first + static_cast<int64_t>(c - cbeg) * kGC;
    const int len = c == cend - 1 ? len_last : kGC;
#pragma unroll
    for (int r = 0; r < 4; ++r) vn[r] = vbase[(tok + min(g * 4 + r, len - 1)) * a.ld];
    if (MODE != 1) an = *reinterpret_cast<const float4 *>(record(c) + Rec::kA + at);
  };
  if (c0 < c1) {
    load_va(c0);
    if (MODE != 1) load_q(c0);
  }
  for (int c = c0; c < c1; ++c) {
    const int next = min(c + 1, c1 - 1);             // past the end: the last chunk once more
    const int len = c == cend - 1 ? len_last : kGC;
    const float *rec = record(c);
    float4 kf[NT], df[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      kf[i] = *reinterpret_cast<const float4 *>(rec + Rec::kKd + i * 256 + at);
      df[i] = *reinterpret_cast<const float4 *>(rec + Rec::kDec + i * 16 + g * 4);
    }
    float vf[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) vf[r] = g * 4 + r < len ? Elem<T>::ld(&vn[r]) : 0.f;
    const float4 a4 = an;
    load_va(next);
    if constexpr (MODE != 1) {
      // two accumulators: neighbouring products do not wait for each other
      floatx4 o0 = floatx4{0.f, 0.f, 0.f, 0.f}, o1 = o0;
      o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a4.x, vf[0], o0, 0, 0, 0);
      o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a4.y, vf[1], o1, 0, 0, 0);
      o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a4.z, vf[2], o0, 0, 0, 0);
      o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a4.w, vf[3], o1, 0, 0, 0);
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[i].x, S[i][0], o0, 0, 0, 0);
        o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[i].y, S[i][1], o1, 0, 0, 0);
        o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[i].z, S[i][2], o0, 0, 0, 0);
        o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[i].w, S[i][3], o1, 0, 0, 0);
      }
      load_q(next);
      float *op = a.o + ((static_cast<int64_t>(c) * a.H + h) * kGC + g * 4) * a.dv + col;
      if (cok) {
#pragma unroll
        for (int r = 0; r < 4; ++r) op[r * a.dv] = o0[r] + o1[r];
      }
    }
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      S[i][0] *= df[i].x; S[i][1] *= df[i].y; S[i][2] *= df[i].z; S[i][3] *= df[i].w;
      if constexpr (MODE == 1) {
        sd[i][0] *= df[i].x; sd[i][1] *= df[i].y; sd[i][2] *= df[i].z; sd[i][3] *= df[i].w;
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const float kv = r == 0 ? kf[i].x : r == 1 ? kf[i].y : r == 2 ? kf[i].z : kf[i].w;
        S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(kv, vf[r], S[i], 0, 0, 0);
      }
  }
  if constexpr (MODE == 1) {
    if (tile == 0 && n == 0) {
#pragma unroll
      for (int i = 0; i < NT; ++i)
        *reinterpret_cast<float4 *>(a.seg_dec + sg * DKP + i * 16 + g * 4) = make_float4(sd[i][0], sd[i][1], sd[i][2], sd[i][3]);
    }
  } else {
    if (!last_seg || !slot_ok) return;
  }
  float *dst = MODE == 1 ? gst : st;
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = i * 16 + g * 4 + r;
      if (d < a.dk && cok) dst[static_cast<int64_t>(d) * a.dv + col] = S[i][r];
    }
}

// Contributions of the segments -> the state each of them starts from, in place.
__global__ __launch_bounds__(256) void gla_segments_kernel(const GlaArgs a, int first_seq, int dkp) {
  const int64_t plane = static_cast<int64_t>(a.dk) * a.dv;
  const int64_t e = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  const int h = blockIdx.y, seq = blockIdx.z;
  if (e >= plane) return;
  const int slot = a.state_slots[first_seq + seq];
  const bool from_zero = slot < 0 || slot >= a.num_slots || a.starts[first_seq + seq] == 0;
  float run = from_zero ? 0.f : a.state[(static_cast<int64_t>(slot) * a.H + h) * plane + e];
  const int d = static_cast<int>(e / a.dv);
  for (int s = 0; s < a.segs; ++s) {
    const int64_t sg = (static_cast<int64_t>(seq) * a.segs + s) * a.H + h;
    const bool more = s < a.segs - 1;
    const float own = more ? a.seg_state[sg * plane + e] : 0.f, dec = more ? a.seg_dec[sg * dkp + d] : 0.f;
    a.seg_state[sg * plane + e] = run;
    run = fmaf(dec, run, own);
  }
}

// One wave per (row of a chunk, head).
template <typename T, int VEC>
__global__ __launch_bounds__(256) void gla_out_kernel(const GlaArgs a) {
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= static_cast<int64_t>(a.chunks) * kGC * a.H) return;
  const int64_t crow = item / a.H;
  const int h = static_cast<int>(item - crow * a.H), chunk = static_cast<int>(crow / kGC), t = static_cast<int>(crow % kGC);
  if (t >= a.chunk_len[chunk]) return;
  const int64_t row = a.chunk_tok[chunk] + t;
  const int64_t hk = static_cast<int64_t>(a.H) * a.dk, hv = static_cast<int64_t>(a.H) * a.dv;
  const float *op = a.o + ((static_cast<int64_t>(chunk) * a.H + h) * kGC + t) * a.dv;
  const T *gp = static_cast<const T *>(a.proj) + row * a.ld + 2 * hk + hv + static_cast<int64_t>(h) * a.dv;
  T *out = static_cast<T *>(a.out) + row * a.ldo + static_cast<int64_t>(h) * a.dv;
  constexpr int MAXC = kGlaMaxDv / (64 * VEC);
  Vf<VEC> o[MAXC];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int v = (lane + c * 64) * VEC;
    if (v < a.dv) {
      o[c] = ldf<VEC>(op + v);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss = fmaf(o[c].f[e], o[c].f[e], ss);
    }
  }
  ss = wave_sum(ss);
  const float inv = 1.0f / sqrtf(ss / static_cast<float>(a.dv) + a.eps);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int v = (lane + c * 64) * VEC;
    if (v < a.dv) {
      float gt[VEC], y[VEC];
      if constexpr (VEC == 4 && sizeof(T) == 2) {
        const uint2 r = *reinterpret_cast<const uint2 *>(gp + v);
        gt[0] = __uint_as_float(r.x << 16); gt[1] = __uint_as_float(r.x & 0xffff0000u);
        gt[2] = __uint_as_float(r.y << 16); gt[3] = __uint_as_float(r.y & 0xffff0000u);
      } else {
#pragma unroll
        for (int e = 0; e < VEC; ++e) gt[e] = Elem<T>::ld(gp + v + e);
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e)
        y[e] = o[c].f[e] * inv * Elem<T>::ld(static_cast<const T *>(a.norm_w) + v + e) * gt[e] *
               __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * gt[e]));
      if constexpr (VEC == 4 && sizeof(T) == 2) {
        *reinterpret_cast<uint2 *>(out + v) = make_uint2(pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3]));
      } else {
#pragma unroll
        for (int e = 0; e < VEC; ++e) Elem<T>::st(out + v + e, y[e]);
      }
    }
  }
}

int gla_tiles(int dk) {   // compiled tile counts of the key dimension
  for (int nt : {1, 2, 3, 4, 6, 8, 12, 16})
    if (nt * 16 >= dk) return nt;
  return 0;
}

int gla_check(const GlaArgs &a, int32_t dtype) {
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (a.rows < 0 || a.H <= 0 || a.H > 65535 || a.dk <= 0 || a.dv <= 0 || a.R <= 0) return TLF_E_SHAPE;
  if (a.dk > kGlaMaxDk || a.dv > kGlaMaxDv || a.R > kGlaMaxR) return TLF_E_SHAPE;
  if (a.ld < 2ll * a.H * (a.dk + a.dv) + a.R || a.ldo < static_cast<int64_t>(a.H) * a.dv || a.num_slots <= 0) return TLF_E_SHAPE;
  if (a.rows == 0) return TLF_OK;
  if ((!a.proj && a.part.splits <= 1) || !a.a2 || !a.a2_bias || !a.norm_w || !a.state || !a.state_slots || !a.out) return TLF_E_NULL;
  return TLF_OK;
}

// Segments per sequence: enough waves for every SIMD, segments of at least 16 chunks.
int gla_segments(int chunks, int seqs, int heads, int dv) {
  if (seqs <= 0 || chunks <= 0) return 1;
  const int64_t waves = static_cast<int64_t>((dv + 15) / 16) * heads * seqs;
  const int64_t want = waves >= 1024 ? 1 : (2048 + waves - 1) / waves, most = chunks / seqs / 16;
  const int64_t s = want < most ? want : most;
  return static_cast<int>(s < 1 ? 1 : s > 32 ? 32 : s);
}

template <typename T>
int launch_gla_portions(GlaArgs &a, int first_seq, hipStream_t stream) {
  const int nt = gla_tiles(a.dk), tiles = (a.dv + 15) / 16;
  a.vec = sizeof(T) == 2 && a.dk == nt * 16 && a.ld % 4 == 0 && (reinterpret_cast<uintptr_t>(a.proj) & 7) == 0;
  const dim3 cgrid(a.chunks, a.H);
  const dim3 sgrid(a.H, (tiles + 3) / 4, a.seqs * a.segs);
#define TLF_GLA(NT)                                                                                       \
  do {                                                                                                    \
    TLF_LAUNCH((gla_chunk_kernel<T, NT>), cgrid, dim3(256), 0, stream, a);                                \
    if (a.segs == 1) {                                                                                    \
      TLF_LAUNCH((gla_scan_kernel<T, NT, 0>), sgrid, dim3(256), 0, stream, a, first_seq);              \
    } else {                                                                                              \
      TLF_LAUNCH((gla_scan_kernel<T, NT, 1>), sgrid, dim3(256), 0, stream, a, first_seq);              \
      TLF_LAUNCH(gla_segments_kernel, dim3((a.dk * a.dv + 255) / 256, a.H, a.seqs), dim3(256), 0, stream, \
                 a, first_seq, (NT) * 16);                                                                \
      TLF_LAUNCH((gla_scan_kernel<T, NT, 2>), sgrid, dim3(256), 0, stream, a, first_seq);              \
    }                                                                                                     \
  } while (0)
  switch (nt) {
    case 1: TLF_GLA(1); break;
    case 2: TLF_GLA(2); break;
    case 3: TLF_GLA(3); break;
    case 4: TLF_GLA(4); break;
    case 6: TLF_GLA(6); break;
    case 8: TLF_GLA(8); break;
    case 12: TLF_GLA(12); break;
    default: TLF_GLA(16); break;
  }
#undef TLF_GLA
  const dim3 ogrid(static_cast<unsigned>(static_cast<int64_t>(a.chunks) * (kGC / 4) * a.H));
  const bool vec = a.dv % 4 == 0 && a.ld % 4 == 0 && (2ll * a.H * a.dk) % 4 == 0 && a.ldo % 4 == 0 &&
                   aligned16(a.proj) && (reinterpret_cast<uintptr_t>(a.out) & 7) == 0;
  if (vec) TLF_LAUNCH((gla_out_kernel<T, 4>), ogrid, dim3(256), 0, stream, a);
  else TLF_LAUNCH((gla_out_kernel<T, 1>), ogrid, dim3(256), 0, stream, a);
  return launch_status();
}

}  // namespace tlf

extern "C" int tlf_gla_decode(const void *proj, int64_t proj_stride, const float *partials, int32_t splits,
                              const float *scale, const void *a2, const void *a2_bias,
                              const void *norm_weight, float *state, const int32_t *state_slots, int32_t num_slots,
                              const int64_t *positions, void *out, int64_t out_stride, int32_t rows, int32_t heads,
                              int32_t key_dim, int32_t value_dim, int32_t rank, float tau, float q_scale, float eps,
                              int32_t dtype, void *stream) {
  using namespace tlf;
  GlaArgs a{};
  a.proj = proj; a.ld = proj_stride; a.a2 = a2; a.a2_bias = a2_bias; a.norm_w = norm_weight; a.state = state;
  a.state_slots = state_slots; a.num_slots = num_slots; a.positions = positions; a.out = out; a.ldo = out_stride;
  a.rows = rows; a.H = heads; a.dk = key_dim; a.dv = value_dim; a.R = rank; a.inv_tau = 1.0f / tau;
  a.q_scale = q_scale; a.eps = eps;
  a.part = Partials{partials, scale, rows * proj_stride, static_cast<int32_t>(proj_stride), splits};
  if (int rc = partials_check(partials, scale, splits, dtype)) return rc;
  if (int rc = gla_check(a, dtype)) return rc;
  if (rows > 65535 || !(tau > 0.f)) return TLF_E_SHAPE;
  if (rows == 0) return TLF_OK;
  if (!positions) return TLF_E_NULL;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const bool vec = value_dim % 4 == 0 && aligned16(state);
  int lanes = 4;
  while (lanes < 64 && lanes * (vec ? 4 : 1) < value_dim) lanes *= 2;
  const dim3 grid(heads, rows);
  if (splits > 1) {
    if (vec) TLF_LAUNCH((gla_decode_kernel<unsigned short, 4, true>), grid, dim3(256), 0, s, a, lanes);
    else TLF_LAUNCH((gla_decode_kernel<unsigned short, 1, true>), grid, dim3(256), 0, s, a, lanes);
  } else if (dtype == TLF_DT_BF16) {
    if (vec) TLF_LAUNCH((gla_decode_kernel<unsigned short, 4, false>), grid, dim3(256), 0, s, a, lanes);
    else TLF_LAUNCH((gla_decode_kernel<unsigned short, 1, false>), grid, dim3(256), 0, s, a, lanes);
  } else {
    if (vec) TLF_LAUNCH((gla_decode_kernel<float, 4, false>), grid, dim3(256), 0, s, a, lanes);
    else TLF_LAUNCH((gla_decode_kernel<float, 1, false>), grid, dim3(256), 0, s, a, lanes);
  }
  return launch_status();
}

extern "C" size_t tlf_gla_portions_workspace_bytes(int32_t rows, int32_t chunks, int32_t num_seqs, int32_t heads,
                                                   int32_t key_dim, int32_t value_dim) {
  using namespace tlf;
  if (rows <= 0 || chunks <= 0 || num_seqs <= 0 || heads <= 0 || key_dim <= 0 || key_dim > kGlaMaxDk || value_dim <= 0) return 0;
  const size_t ch = static_cast<size_t>(chunks) * heads, dkp = gla_tiles(key_dim) * 16;
  const size_t segs = gla_segments(chunks, num_seqs, heads, value_dim);
  const size_t sg = segs > 1 ? segs * num_seqs * heads : 0;
  return 4 * (ch * (gla_rec_size(static_cast<int>(dkp)) + static_cast<size_t>(kGC) * ((value_dim + 3) / 4 * 4)) +
              sg * (dkp + static_cast<size_t>(key_dim) * value_dim));
}

extern "C" int tlf_gla_portions(const void *proj, int64_t proj_stride, const void *a2, const void *a2_bias,
                                const void *norm_weight, float *state, const int32_t *state_slots, int32_t num_slots,
                                const int32_t *seq_starts, const int32_t *chunk_rows, const int32_t *chunk_lens,
                                const int32_t *cu_chunks, int32_t chunks, int32_t first_seq, int32_t num_seqs,
                                void *out, int64_t out_stride, int32_t rows, int32_t heads, int32_t key_dim,
                                int32_t value_dim, int32_t rank, float tau, float q_scale, float eps, int32_t dtype,
                                void *workspace, size_t workspace_bytes, void *stream) {
  using namespace tlf;
  GlaArgs a{};
  a.proj = proj; a.ld = proj_stride; a.a2 = a2; a.a2_bias = a2_bias; a.norm_w = norm_weight; a.state = state;
  a.state_slots = state_slots; a.num_slots = num_slots; a.out = out; a.ldo = out_stride;
  a.rows = rows; a.H = heads; a.dk = key_dim; a.dv = value_dim; a.R = rank; a.inv_tau = 1.0f / tau;
  a.q_scale = q_scale; a.eps = eps; a.chunk_tok = chunk_rows; a.chunk_len = chunk_lens; a.cu_chunks = cu_chunks;
  a.starts = seq_starts; a.chunks = chunks; a.seqs = num_seqs;
  if (int rc = gla_check(a, dtype)) return rc;
  if (!(tau > 0.f) || chunks < 0 || num_seqs < 0 || num_seqs > 65535 || first_seq < 0) return TLF_E_SHAPE;
  if (rows == 0 || chunks == 0 || num_seqs == 0) return TLF_OK;
  if (!seq_starts || !chunk_rows || !chunk_lens || !cu_chunks) return TLF_E_NULL;
  if (!workspace || !aligned16(workspace) ||
      workspace_bytes < tlf_gla_portions_workspace_bytes(rows, chunks, num_seqs, heads, key_dim, value_dim))
    return TLF_E_WORKSPACE;
  const size_t ch = static_cast<size_t>(chunks) * heads, dkp = gla_tiles(key_dim) * 16;
  a.rec = static_cast<float *>(workspace);
  a.o = a.rec + ch * gla_rec_size(static_cast<int>(dkp));
  a.segs = gla_segments(chunks, num_seqs, heads, value_dim);
  if (static_cast<int64_t>(num_seqs) * a.segs > 65535) a.segs = 1;
  a.seg_dec = a.o + ch * kGC * ((value_dim + 3) / 4 * 4);
  a.seg_state = a.seg_dec + static_cast<size_t>(num_seqs) * a.segs * heads * dkp;
  hipStream_t s = static_cast<hipStream_t>(stream);
  return dtype == TLF_DT_BF16 ? launch_gla_portions<unsigned short>(a, first_seq, s)
                              : launch_gla_portions<float>(a, first_seq, s);
}
