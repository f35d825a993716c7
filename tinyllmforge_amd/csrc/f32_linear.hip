// The few dense operations a model needs in 32-bit mode: y = x . W^T with v_mfma_f32_16x16x4_f32 (true fp32 products
// and sums), SiLU-and-mul and the greedy argmax on fp32 rows.  32-bit mode is for checking numerics, so these favour
// generality (any M, N, K) over speed: a 64 x 64 tile per workgroup, K staged 16 at a time.
#include "elem.h"

namespace tlf {

constexpr int kFT = 64, kFK = 16, kFPad = kFK + 4;

__global__ __launch_bounds__(256) void f32_gemm_kernel(const float *__restrict__ x, int64_t ldx,
                                                       const float *__restrict__ w, float *__restrict__ y, int32_t M,
                                                       int32_t N, int32_t K) {
  __shared__ __attribute__((aligned(16))) float Xs[kFT][kFPad], Ws[kFT][kFPad];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = lane & 15, g = lane >> 4;
  const int m0 = blockIdx.y * kFT, n0 = blockIdx.x * kFT;
  floatx4 acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = floatx4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < K; k0 += kFK) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = i * 16 + tid / 16, c = tid % 16;
      const bool kin = k0 + c < K;
      Xs[r][c] = kin && m0 + r < M ? x[static_cast<int64_t>(m0 + r) * ldx + k0 + c] : 0.f;
      Ws[r][c] = kin && n0 + r < N ? w[static_cast<int64_t>(n0 + r) * K + k0 + c] : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < kFK / 4; ++s) {
      const float a = Xs[wave * 16 + n][s * 4 + g];
#pragma unroll
      for (int i = 0; i < 4; ++i)
        acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, Ws[i * 16 + n][s * 4 + g], acc[i], 0, 0, 0);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int m = m0 + wave * 16 + g * 4 + r, c = n0 + i * 16 + n;
      if (m < M && c < N) y[static_cast<int64_t>(m) * N + c] = acc[i][r];
    }
}

__global__ __launch_bounds__(256) void f32_silu_mul_kernel(const float *__restrict__ x, float *__restrict__ y,
                                                           int64_t rows, int32_t inter) {
  const int64_t i = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (i >= rows * inter) return;
  const int64_t r = i / inter;
  const float *p = x + r * 2 * inter + (i - r * inter);
  y[i] = silu_f32(p[0]) * p[inter];
}

__global__ __launch_bounds__(256) void f32_argmax_kernel(const float *__restrict__ logits, int64_t stride,
                                                         int64_t *__restrict__ out, int32_t vocab) {
  __shared__ unsigned long long part[4];
  const float *lr = logits + static_cast<int64_t>(blockIdx.x) * stride;
  unsigned long long best = 0;
  for (int i = threadIdx.x; i < vocab; i += 256) {
    unsigned int b = __float_as_uint(lr[i] + 0.0f);  // -0 + 0 = +0
    b = (b & 0x80000000u) ? ~b : (b | 0x80000000u);
    const unsigned long long key = (static_cast<unsigned long long>(b) << 32) | (0xffffffffu - static_cast<unsigned>(i));
    best = key > best ? key : best;
  }
  best = wave_max_u64(best);
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = best;
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 4; ++w) best = part[w] > best ? part[w] : best;
    out[blockIdx.x] = static_cast<int64_t>(0xffffffffu - static_cast<unsigned>(best & 0xffffffffu));
  }
}

}  // namespace tlf

extern "C" int tlf_f32_gemm(const float *x, int64_t x_stride, const float *w, float *y, int32_t M, int32_t N, int32_t K,
                            void *stream) {
  if (M < 0 || N <= 0 || K <= 0 || x_stride < K) return TLF_E_SHAPE;
  if (M == 0) return TLF_OK;
  if (!x || !w || !y) return TLF_E_NULL;
  if ((M + tlf::kFT - 1) / tlf::kFT > 65535) return TLF_E_SHAPE;
  TLF_LAUNCH(tlf::f32_gemm_kernel, dim3((N + tlf::kFT - 1) / tlf::kFT, (M + tlf::kFT - 1) / tlf::kFT), dim3(256), 0,
             static_cast<hipStream_t>(stream), x, x_stride, w, y, M, N, K);
  return tlf::launch_status();
}

extern "C" int tlf_f32_silu_and_mul(const float *x, float *y, int32_t rows, int32_t inter, void *stream) {
  if (rows < 0 || inter <= 0) return TLF_E_SHAPE;
  if (rows == 0) return TLF_OK;
  if (!x || !y) return TLF_E_NULL;
  const int64_t total = static_cast<int64_t>(rows) * inter;
  TLF_LAUNCH(tlf::f32_silu_mul_kernel, dim3(static_cast<unsigned>((total + 255) / 256)), dim3(256), 0,
             static_cast<hipStream_t>(stream), x, y, static_cast<int64_t>(rows), inter);
  return tlf::launch_status();
}

extern "C" int tlf_f32_argmax(const float *logits, int64_t row_stride, int64_t *out, int32_t rows, int32_t vocab,
                              void *stream) {
  if (rows < 0 || vocab <= 0 || row_stride < vocab) return TLF_E_SHAPE;
  if (rows == 0) return TLF_OK;
  if (!logits || !out) return TLF_E_NULL;
  TLF_LAUNCH(tlf::f32_argmax_kernel, dim3(rows), dim3(256), 0, static_cast<hipStream_t>(stream), logits, row_stride,
             out, vocab);
  return tlf::launch_status();
}
