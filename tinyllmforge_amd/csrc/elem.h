// Element access for kernels that exist for bf16 (uint16 bits) and fp32 tensors alike: all arithmetic is fp32,
// only loads and stores differ.
#pragma once
#include "common.h"

namespace tlf {

template <typename T>
struct Elem;

template <>
struct Elem<unsigned short> {
  static __device__ __forceinline__ float ld(const unsigned short *p) { return bf16_bits_to_float(*p); }
  static __device__ __forceinline__ void st(unsigned short *p, float v) { *p = float_to_bf16_bits(v); }
  static __device__ __forceinline__ float rnd(float v) { return bf16_bits_to_float(float_to_bf16_bits(v)); }
  static __device__ __forceinline__ void ld8(const unsigned short *p, float (&f)[8]) {
    unpack8(*reinterpret_cast<const uint4 *>(p), f);
  }
  static __device__ __forceinline__ void st8(unsigned short *p, const float (&f)[8]) {
    *reinterpret_cast<uint4 *>(p) = pack8(f);
  }
  struct Raw8 {
    uint4 a;
  };
  static __device__ __forceinline__ void raw8(const unsigned short *p, Raw8 &r) {
    r.a = *reinterpret_cast<const uint4 *>(p);
  }
  static __device__ __forceinline__ void zero8(Raw8 &r) { r.a = make_uint4(0, 0, 0, 0); }
  static __device__ __forceinline__ void cvt8(const Raw8 &r, float (&f)[8]) { unpack8(r.a, f); }
};

template <>
struct Elem<float> {
  static __device__ __forceinline__ float ld(const float *p) { return *p; }
  static __device__ __forceinline__ void st(float *p, float v) { *p = v; }
  static __device__ __forceinline__ float rnd(float v) { return v; }
  static __device__ __forceinline__ void ld8(const float *p, float (&f)[8]) {
    const float4 a = reinterpret_cast<const float4 *>(p)[0], b = reinterpret_cast<const float4 *>(p)[1];
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
    f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
  }
  static __device__ __forceinline__ void st8(float *p, const float (&f)[8]) {
    reinterpret_cast<float4 *>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
    reinterpret_cast<float4 *>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
  }
  struct Raw8 {
    float4 a, b;
  };
  static __device__ __forceinline__ void raw8(const float *p, Raw8 &r) {
    r.a = reinterpret_cast<const float4 *>(p)[0];
    r.b = reinterpret_cast<const float4 *>(p)[1];
  }
  static __device__ __forceinline__ void zero8(Raw8 &r) { r.a = r.b = make_float4(0.f, 0.f, 0.f, 0.f); }
  static __device__ __forceinline__ void cvt8(const Raw8 &r, float (&f)[8]) {
    f[0] = r.a.x; f[1] = r.a.y; f[2] = r.a.z; f[3] = r.a.w;
    f[4] = r.b.x; f[5] = r.b.y; f[6] = r.b.z; f[7] = r.b.w;
  }
};

// A bf16 projection [rows, n] that exists as fp32 partial sums [splits, rows, n] (times a scale per column where the
// weight is int8): the value is their sum, rounded to bf16 as the projection's own kernel would.
struct Partials {
  const float *p;
  const float *scale;
  int64_t plane;      // rows * n
  int32_t n, splits;
  __device__ __forceinline__ float ld(int64_t row, int col) const {
    const float *s = p + row * n + col;
    float v = 0.f;
#pragma unroll 4
    for (int k = 0; k < splits; ++k) v += s[k * plane];
    return Elem<unsigned short>::rnd(scale ? v * scale[col] : v);
  }
  __device__ __forceinline__ void ld8(int64_t row, int col, float (&f)[8]) const {
    const float *s = p + row * n + col;
    float4 a = make_float4(0.f, 0.f, 0.f, 0.f), b = a;
#pragma unroll 4
    for (int k = 0; k < splits; ++k) {
      const float4 x = reinterpret_cast<const float4 *>(s + k * plane)[0], y = reinterpret_cast<const float4 *>(s + k * plane)[1];
      a.x += x.x; a.y += x.y; a.z += x.z; a.w += x.w;
      b.x += y.x; b.y += y.y; b.z += y.z; b.w += y.w;
    }
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = Elem<unsigned short>::rnd(scale ? f[e] * scale[col + e] : f[e]);
  }
};
inline int partials_check(const void *partials, const float *scale, int32_t splits, int32_t dtype) {
  if (splits < 0 || splits > 64) return TLF_E_SHAPE;
  if (splits > 1 && dtype != TLF_DT_BF16) return TLF_E_UNSUPPORTED;
  if (splits > 1 && !partials) return TLF_E_NULL;
  return splits > 1 && (!aligned16(partials) || !aligned16(scale)) ? TLF_E_ALIGN : TLF_OK;
}

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }

// xIELU: a z^2 + z / 2 above zero, b (e^z - 1 - z) + z / 2 below; a = softplus(p), b = 1/2 + softplus(q).
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// e^z - 1 - z without cancellation: five terms of the series near zero (relative error below 2^-24 for |z| < 1/16).
__device__ __forceinline__ float exp_rest(float z) {
  if (z > -0.0625f) {
    float r = fmaf(z, 1.0f / 720.0f, 1.0f / 120.0f);
    r = fmaf(z, r, 1.0f / 24.0f);
    r = fmaf(z, r, 1.0f / 6.0f);
    r = fmaf(z, r, 0.5f);
    return z * z * r;
  }
  return __builtin_amdgcn_exp2f(z * 1.4426950408889634f) - 1.0f - z;
}
__device__ __forceinline__ float xielu_f32(float z, float a, float b) {
  return fmaf(z > 0.f ? a * z * z : b * exp_rest(fminf(z, 0.f)), 1.0f, 0.5f * z);
}

// Sum over aligned groups of N lanes (4, 8, 16, 32 or 64), on the vector ALU (DPP) up to a row of 16 lanes.
template <int CTRL>
__device__ __forceinline__ float dpp_move(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false));
}
template <int N>
__device__ __forceinline__ float group_sum(float v) {
  static_assert(N == 4 || N == 8 || N == 16 || N == 32 || N == 64, "lanes per group");
  v += dpp_move<0xB1>(v);                   // quad_perm [1, 0, 3, 2]
  v += dpp_move<0x4E>(v);                   // quad_perm [2, 3, 0, 1]
  if (N >= 8) v += dpp_move<0x141>(v);      // row_half_mirror
  if (N >= 16) v += dpp_move<0x140>(v);     // row_mirror
  if (N >= 32) v += __shfl_xor(v, 16, 64);
  if (N >= 64) v += __shfl_xor(v, 32, 64);
  return v;
}

}  // namespace tlf
