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
//   gla_scan_kernel    per (sequence, head, 16 NV columns of v), one wave each, sequential over the chunks:
//                      O = Qd S + A V;  S = diag(2^b_end) S + Kd^T V.  All products are v_mfma_f32_16x16x4_f32; the
//                      state stays in accumulator registers, whose layout (row 4 g + r of a tile in register r of
//                      lane group g) is the B operand of the next product when its summation index is labelled
//                      4 g + r in step r.  No LDS, no barrier.
//   gla_out_kernel     norm and output gate
#include "elem.h"

namespace tlf {

constexpr int kGlaMaxDk = 256, kGlaMaxDv = 512, kGlaMaxR = 256;

struct GlaArgs {
  const void *proj;        // [n, ld]
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
  float *qd, *kd, *am, *dec, *o;          // workspace
};

// log2 of sigmoid(z)^(1/tau)
__device__ __forceinline__ float log2_alpha(float z, float inv_tau) {
  const float sp = fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)));   // softplus(-z)
  return -sp * inv_tau * 1.4426950408889634f;
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

template <typename T, int VEC>
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
  const T *qp = pr + h * a.dk, *kp = pr + hk + h * a.dk, *vp = pr + 2 * hk + h * a.dv, *gp = vp + hv;
  const T *rp = pr + 2 * hk + 2 * hv;
  for (int r = tid; r < a.R; r += 256) rs[r] = Elem<T>::ld(rp + r);
  if (tid < a.dk) {
    qs[tid] = Elem<T>::ld(qp + tid) * a.q_scale;
    ks[tid] = Elem<T>::ld(kp + tid);
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
      v.f[e] = Elem<T>::ld(vp + c * VEC + e);
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
      Elem<T>::st(out + v, ov[i] * inv * Elem<T>::ld(static_cast<const T *>(a.norm_w) + v) * silu_f32(Elem<T>::ld(gp + v)));
  }
}

// ---------------------------------------------------------------------------------------------------------------
constexpr int kGC = 16;   // tokens per chunk

template <typename T, int NT>
__global__ __launch_bounds__(256) void gla_chunk_kernel(const GlaArgs a) {
  constexpr int DKP = NT * 16, LD = DKP + 4;
  __shared__ __attribute__((aligned(16))) float ks[kGC][LD], bs[kGC][LD];
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
  if (tid < DKP) {
    float z[kGC];
    if (tid < a.dk) {
      const T *w = static_cast<const T *>(a.a2) + (static_cast<int64_t>(h) * a.dk + tid) * a.R;
      const float b = Elem<T>::ld(static_cast<const T *>(a.a2_bias) + h * a.dk + tid);
#pragma unroll
      for (int t = 0; t < kGC; ++t) z[t] = b;
      for (int r = 0; r < a.R; ++r) {
        const float wr = Elem<T>::ld(w + r);
#pragma unroll
        for (int t = 0; t < kGC; ++t) z[t] = fmaf(wr, rs[t][r], z[t]);
      }
    }
    float b = 0.f;
#pragma unroll
    for (int t = 0; t < kGC; ++t) {
      if (tid < a.dk && t < len) b += log2_alpha(z[t], a.inv_tau);
      bs[t][tid] = b;
    }
  }
  // 16 lanes per token; lane l holds channels dmap(i): four at a time where the row length allows 16-byte LDS reads
  const int t = tid / 16, l = tid % 16;
  auto dmap = [&](int i) { return NT % 4 == 0 ? (i / 4) * 64 + l * 4 + i % 4 : l + 16 * i; };
  float q[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int d = dmap(i);
    const bool in = d < a.dk && t < len;
    q[i] = in ? Elem<T>::ld(pr + t * a.ld + h * a.dk + d) * a.q_scale : 0.f;
    ks[t][d] = in ? Elem<T>::ld(pr + t * a.ld + hk + h * a.dk + d) : 0.f;
  }
  __syncthreads();
  const int64_t ch = static_cast<int64_t>(chunk) * a.H + h;
  float bt[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) bt[i] = bs[t][dmap(i)];
  // operand order of the scan: Qd [tile][t][16 channels], Kd [tile][channel][16 tokens]
  float *qd = a.qd + ch * (DKP * kGC), *kd = a.kd + ch * (DKP * kGC);
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int d = dmap(i);
    qd[(d / 16) * 256 + t * 16 + d % 16] = q[i] * __builtin_amdgcn_exp2f(bt[i]);
  }
  for (int i = tid; i < DKP * kGC; i += 256) {
    const int d = i / kGC, s = i % kGC;
    kd[i] = ks[s][d] * __builtin_amdgcn_exp2f(bs[kGC - 1][d] - bs[s][d]);
  }
  if (tid < DKP) a.dec[ch * DKP + tid] = __builtin_amdgcn_exp2f(bs[kGC - 1][tid]);
  float *am = a.am + ch * (kGC * kGC) + t * kGC;
  const int smax = (tid / 64) * 4 + 3;               // last token of this wave
  for (int s = 0; s < kGC; ++s) {
    float acc = 0.f;
    if (s <= smax) {                                 // wave uniform
      float kv[NT], bv[NT];
      if constexpr (NT % 4 == 0) {
#pragma unroll
        for (int i = 0; i < NT; i += 4) {
          const float4 k4 = *reinterpret_cast<const float4 *>(&ks[s][(i / 4) * 64 + l * 4]);
          const float4 b4 = *reinterpret_cast<const float4 *>(&bs[s][(i / 4) * 64 + l * 4]);
          kv[i] = k4.x; kv[i + 1] = k4.y; kv[i + 2] = k4.z; kv[i + 3] = k4.w;
          bv[i] = b4.x; bv[i + 1] = b4.y; bv[i + 2] = b4.z; bv[i + 3] = b4.w;
        }
      } else {
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          kv[i] = ks[s][l + 16 * i];
          bv[i] = bs[s][l + 16 * i];
        }
      }
#pragma unroll
      for (int i = 0; i < NT; ++i)
        acc = fmaf(q[i] * kv[i], __builtin_amdgcn_exp2f(fminf(bt[i] - bv[i], 0.f)), acc);
      acc = group_sum<16>(acc);
    }
    if (l == 0) am[s] = s <= t ? acc : 0.f;
  }
}

template <typename T, int NT, int NV>
__global__ __launch_bounds__(256) void gla_scan_kernel(const GlaArgs a, int first_seq) {
  constexpr int DKP = NT * 16;
  const int tid = threadIdx.x, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int h = blockIdx.y, seq = blockIdx.z;
  const int tile0 = (blockIdx.x * 4 + (tid >> 6)) * NV;
  if (tile0 * 16 >= a.dv) return;                    // no barrier below: a wave may leave on its own
  const int slot = a.state_slots[first_seq + seq];
  const bool slot_ok = slot >= 0 && slot < a.num_slots;
  const bool fresh = a.starts[first_seq + seq] == 0;
  float *st = a.state + (static_cast<int64_t>(slot_ok ? slot : 0) * a.H + h) * a.dk * a.dv;
  int col[NV];
  bool cok[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    col[j] = (tile0 + j) * 16 + n;
    cok[j] = col[j] < a.dv;
    if (!cok[j]) col[j] = 0;
  }
  floatx4 S[NT][NV];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = i * 16 + g * 4 + r;
        S[i][j][r] = !fresh && slot_ok && d < a.dk && cok[j] ? st[static_cast<int64_t>(d) * a.dv + col[j]] : 0.f;
      }
  const int64_t hk = static_cast<int64_t>(a.H) * a.dk, hv = static_cast<int64_t>(a.H) * a.dv;
  const T *vbase = static_cast<const T *>(a.proj) + 2 * hk + static_cast<int64_t>(h) * a.dv;
  const int c0 = a.cu_chunks[seq], c1 = a.cu_chunks[seq + 1];
  float4 qf[NT];
  auto load_q = [&](int c) {
    const float *p = a.qd + (static_cast<int64_t>(c) * a.H + h) * (DKP * kGC) + n * 16 + g * 4;
#pragma unroll
    for (int i = 0; i < NT; ++i) qf[i] = *reinterpret_cast<const float4 *>(p + i * 256);
  };
  if (c0 < c1) load_q(c0);
  for (int c = c0; c < c1; ++c) {
    const int64_t ch = static_cast<int64_t>(c) * a.H + h;
    const int64_t tok0 = a.chunk_tok[c];
    const int len = a.chunk_len[c];
    const float4 am = *reinterpret_cast<const float4 *>(a.am + ch * (kGC * kGC) + n * 16 + g * 4);
    const float av[4] = {am.x, am.y, am.z, am.w};
    float vf[NV][4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int s = g * 4 + r;
      const T *vp = vbase + (tok0 + min(s, len - 1)) * a.ld;
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const float x = Elem<T>::ld(vp + col[j]);
        vf[j][r] = s < len ? x : 0.f;
      }
    }
    float4 kf[NT], df[NT];
    const float *kp = a.kd + ch * (DKP * kGC) + n * 16 + g * 4, *dp = a.dec + ch * DKP + g * 4;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      kf[i] = *reinterpret_cast<const float4 *>(kp + i * 256);
      df[i] = *reinterpret_cast<const float4 *>(dp + i * 16);
    }
    floatx4 o[NV];
#pragma unroll
    for (int j = 0; j < NV; ++j) o[j] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const float qv[4] = {qf[i].x, qf[i].y, qf[i].z, qf[i].w};
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int j = 0; j < NV; ++j) o[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[r], S[i][j][r], o[j], 0, 0, 0);
    }
    if (c + 1 < c1) load_q(c + 1);
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int j = 0; j < NV; ++j) o[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[r], vf[j][r], o[j], 0, 0, 0);
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const float kv[4] = {kf[i].x, kf[i].y, kf[i].z, kf[i].w};
      const float dv[4] = {df[i].x, df[i].y, df[i].z, df[i].w};
#pragma unroll
      for (int j = 0; j < NV; ++j) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[i][j][r] *= dv[r];
#pragma unroll
        for (int r = 0; r < 4; ++r) S[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kv[r], vf[j][r], S[i][j], 0, 0, 0);
      }
    }
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = g * 4 + r;
        if (t < len && cok[j]) a.o[(tok0 + t) * hv + static_cast<int64_t>(h) * a.dv + col[j]] = o[j][r];
      }
  }
  if (!slot_ok) return;
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = i * 16 + g * 4 + r;
        if (d < a.dk && cok[j]) st[static_cast<int64_t>(d) * a.dv + col[j]] = S[i][j][r];
      }
}

// One wave per (row, head).
template <typename T, int VEC>
__global__ __launch_bounds__(256) void gla_out_kernel(const GlaArgs a) {
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= static_cast<int64_t>(a.rows) * a.H) return;
  const int64_t row = item / a.H;
  const int h = static_cast<int>(item - row * a.H);
  const int64_t hk = static_cast<int64_t>(a.H) * a.dk, hv = static_cast<int64_t>(a.H) * a.dv;
  const float *op = a.o + row * hv + static_cast<int64_t>(h) * a.dv;
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
#pragma unroll
      for (int e = 0; e < VEC; ++e)
        Elem<T>::st(out + v + e, o[c].f[e] * inv * Elem<T>::ld(static_cast<const T *>(a.norm_w) + v + e) *
                                     silu_f32(Elem<T>::ld(gp + v + e)));
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
  if (!a.proj || !a.a2 || !a.a2_bias || !a.norm_w || !a.state || !a.state_slots || !a.out) return TLF_E_NULL;
  return TLF_OK;
}

template <typename T>
int launch_gla_portions(const GlaArgs &a, int first_seq, hipStream_t stream) {
  const int nt = gla_tiles(a.dk), tiles = (a.dv + 15) / 16;
  // two column tiles per wave once all SIMDs have work and the state's registers leave room for them
  const bool wide = nt <= 8 && static_cast<int64_t>(tiles) * a.H * a.seqs >= 2048;
  const dim3 cgrid(a.chunks, a.H);
  const dim3 sgrid((tiles + (wide ? 8 : 4) - 1) / (wide ? 8 : 4), a.H, a.seqs);
#define TLF_GLA(NT)                                                                                       \
  do {                                                                                                    \
    TLF_LAUNCH((gla_chunk_kernel<T, NT>), cgrid, dim3(256), 0, stream, a);                                \
    if (wide) TLF_LAUNCH((gla_scan_kernel<T, (NT) <= 8 ? (NT) : 8, 2>), sgrid, dim3(256), 0, stream, a, first_seq);         \
    else TLF_LAUNCH((gla_scan_kernel<T, NT, 1>), sgrid, dim3(256), 0, stream, a, first_seq);              \
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
  const dim3 ogrid(static_cast<unsigned>((static_cast<int64_t>(a.rows) * a.H + 3) / 4));
  if (a.dv % 4 == 0) TLF_LAUNCH((gla_out_kernel<T, 4>), ogrid, dim3(256), 0, stream, a);
  else TLF_LAUNCH((gla_out_kernel<T, 1>), ogrid, dim3(256), 0, stream, a);
  return launch_status();
}

}  // namespace tlf

extern "C" int tlf_gla_decode(const void *proj, int64_t proj_stride, const void *a2, const void *a2_bias,
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
  if (int rc = gla_check(a, dtype)) return rc;
  if (rows > 65535 || !(tau > 0.f)) return TLF_E_SHAPE;
  if (rows == 0) return TLF_OK;
  if (!positions) return TLF_E_NULL;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const bool vec = value_dim % 4 == 0 && aligned16(state);
  int lanes = 4;
  while (lanes < 64 && lanes * (vec ? 4 : 1) < value_dim) lanes *= 2;
  const dim3 grid(heads, rows);
  if (dtype == TLF_DT_BF16) {
    if (vec) TLF_LAUNCH((gla_decode_kernel<unsigned short, 4>), grid, dim3(256), 0, s, a, lanes);
    else TLF_LAUNCH((gla_decode_kernel<unsigned short, 1>), grid, dim3(256), 0, s, a, lanes);
  } else {
    if (vec) TLF_LAUNCH((gla_decode_kernel<float, 4>), grid, dim3(256), 0, s, a, lanes);
    else TLF_LAUNCH((gla_decode_kernel<float, 1>), grid, dim3(256), 0, s, a, lanes);
  }
  return launch_status();
}

extern "C" size_t tlf_gla_portions_workspace_bytes(int32_t rows, int32_t chunks, int32_t heads, int32_t key_dim,
                                                   int32_t value_dim) {
  using namespace tlf;
  if (rows <= 0 || chunks <= 0 || heads <= 0 || key_dim <= 0 || key_dim > kGlaMaxDk || value_dim <= 0) return 0;
  const size_t ch = static_cast<size_t>(chunks) * heads, dkp = gla_tiles(key_dim) * 16;
  return 4 * (ch * (2 * dkp * kGC + kGC * kGC + dkp) + (static_cast<size_t>(rows) * heads * value_dim + 63) / 64 * 64);
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
      workspace_bytes < tlf_gla_portions_workspace_bytes(rows, chunks, heads, key_dim, value_dim))
    return TLF_E_WORKSPACE;
  const size_t ch = static_cast<size_t>(chunks) * heads, dkp = gla_tiles(key_dim) * 16;
  a.qd = static_cast<float *>(workspace);
  a.kd = a.qd + ch * dkp * kGC;
  a.am = a.kd + ch * dkp * kGC;
  a.dec = a.am + ch * kGC * kGC;
  a.o = a.dec + ch * dkp;
  hipStream_t s = static_cast<hipStream_t>(stream);
  return dtype == TLF_DT_BF16 ? launch_gla_portions<unsigned short>(a, first_seq, s)
                              : launch_gla_portions<float>(a, first_seq, s);
}
