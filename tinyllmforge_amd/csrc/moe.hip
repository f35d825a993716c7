// Mixture of experts: router, grouping of the rows by expert, the grouped products, and the xIELU activation of dense
// layers.
//
//   router     z = W_router h (bf16 or fp32 factors, fp32 sums), the `top` largest of each row and their sigmoids
//   group      rows (token, k) in expert order, an index each way, tiles of `tile_rows` rows of one expert
//   products   gemm_dlds_kernel<GROUPED> (gemm.hip) in bf16; a plain fp32 kernel here
// No host value depends on the routing: grids are sized for the worst case and tiles past the list's end leave at once,
// so a captured graph replays with any routing.
#include "gemm_shared.h"
#include "elem.h"

namespace tlf {

int launch_grouped(GemmParams p, int bm, hipStream_t stream);

constexpr int kMaxExperts = 512;

struct RouterArgs {
  const void *h;          // [n, ldh]
  const void *w;          // [E16, K], E rounded up to 16
  int64_t ldh;
  int32_t *ids;           // [n, top]
  float *weights;         // [n, top]
  int32_t n, E, E16, K, top;
};

// One wave picks the `top` largest of logits z[0 .. E): key order is value, then the smaller index.
__device__ __forceinline__ void pick_top(const RouterArgs &a, const float *z, int64_t tok) {
  const int lane = threadIdx.x & 63;
  float v[kMaxExperts / 64];
  unsigned long long key[kMaxExperts / 64];
#pragma unroll
  for (int i = 0; i < kMaxExperts / 64; ++i) {
    const int e = i * 64 + lane;
    v[i] = e < a.E ? z[e] : 0.f;
    unsigned int b = __float_as_uint(v[i] + 0.0f);
    b = (b & 0x80000000u) ? ~b : (b | 0x80000000u);
    key[i] = e < a.E ? (static_cast<unsigned long long>(b) << 32) | (0xffffffffu - static_cast<unsigned>(e)) : 0ull;
  }
  for (int k = 0; k < a.top; ++k) {
    unsigned long long best = 0;
#pragma unroll
    for (int i = 0; i < kMaxExperts / 64; ++i) best = key[i] > best ? key[i] : best;
    best = wave_max_u64(best);
    const int e = static_cast<int>(0xffffffffu - static_cast<unsigned>(best & 0xffffffffu));
#pragma unroll
    for (int i = 0; i < kMaxExperts / 64; ++i)
      if (key[i] == best) {
        a.ids[tok * a.top + k] = e;
        a.weights[tok * a.top + k] = sigmoid_f32(v[i]);
        key[i] = 0;
      }
  }
}

// bf16: 16 tokens per workgroup, eight waves split K, experts 64 at a time
__global__ __launch_bounds__(512) void router_kernel(const RouterArgs a) {
  extern __shared__ __attribute__((aligned(16))) float logits[];    // [16][E16 + 4]
  __shared__ __attribute__((aligned(16))) float red[8][16][68];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int tok0 = blockIdx.x * 16, ldz = a.E16 + 4;
  const unsigned short *hp = static_cast<const unsigned short *>(a.h) + min(tok0 + n, a.n - 1) * a.ldh + g * 8;
  const int steps = a.K / 32, lo = steps * wave / 8, hi = steps * (wave + 1) / 8;
  for (int e0 = 0; e0 < a.E16; e0 += 64) {
    const int tiles = min(4, (a.E16 - e0) / 16);
    const unsigned short *wp[4];
    floatx4 acc[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      wp[t] = static_cast<const unsigned short *>(a.w) + static_cast<int64_t>(e0 + min(t, tiles - 1) * 16 + n) * a.K + g * 8;
      acc[t] = floatx4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll 2
    for (int k = lo; k < hi; ++k) {
      Pack16 x, w[4];
      x.u = *reinterpret_cast<const uint4 *>(hp + k * 32);
#pragma unroll
      for (int t = 0; t < 4; ++t) w[t].u = *reinterpret_cast<const uint4 *>(wp[t] + k * 32);
#pragma unroll
      for (int t = 0; t < 4; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[t].v, x.v, acc[t], 0, 0, 0);
    }
#pragma unroll
    for (int t = 0; t < 4; ++t)
      *reinterpret_cast<float4 *>(&red[wave][n][t * 16 + g * 4]) = make_float4(acc[t][0], acc[t][1], acc[t][2], acc[t][3]);
    __syncthreads();
    for (int i = tid; i < 16 * tiles * 16; i += 512) {
      const int r = i / (tiles * 16), e = i - r * (tiles * 16);
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < 8; ++w) s += red[w][r][e];
      logits[r * ldz + e0 + e] = s;
    }
    __syncthreads();
  }
  for (int r = wave; r < 16 && tok0 + r < a.n; r += 8) pick_top(a, logits + r * ldz, tok0 + r);
}

// fp32: a workgroup per token, a wave per expert
__global__ __launch_bounds__(256) void router_f32_kernel(const RouterArgs a) {
  __shared__ float logits[kMaxExperts];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int64_t tok = blockIdx.x;
  const float *h = static_cast<const float *>(a.h) + tok * a.ldh;
  for (int e = wave; e < a.E; e += 4) {
    const float *w = static_cast<const float *>(a.w) + static_cast<int64_t>(e) * a.K;
    float s = 0.f;
    for (int k = lane; k < a.K; k += 64) s = fmaf(h[k], w[k], s);
    s = wave_sum(s);
    if (lane == 0) logits[e] = s;
  }
  __syncthreads();
  if (wave == 0) pick_top(a, logits, tok);
}

// ---------------------------------------------------------------------------------------------------------------
struct GroupArgs {
  const int32_t *ids;       // [entries]
  const float *weights;     // [entries]
  int32_t *row_of;          // [entries] row of an entry in expert order
  int32_t *src;             // [entries] token of a row
  float *row_weight;        // [entries] weight of a row
  int4 *tiles;
  int32_t *num_tiles;
  int32_t entries, E, top, tile_rows;
};

// One workgroup: counts, prefix sums, tile list, placement.  The order of rows inside an expert is arbitrary (it does not
// enter any value).
__global__ __launch_bounds__(1024) void moe_group_kernel(const GroupArgs a) {
  __shared__ int count[kMaxExperts], start[kMaxExperts], cursor[kMaxExperts], tstart[kMaxExperts];
  const int tid = threadIdx.x;
  for (int e = tid; e < a.E; e += 1024) count[e] = 0;
  __syncthreads();
  for (int i = tid; i < a.entries; i += 1024) atomicAdd(&count[a.ids[i]], 1);
  __syncthreads();
  if (tid < 64) {
    constexpr int kEach = kMaxExperts / 64;
    int rows = 0, tiles = 0;
#pragma unroll
    for (int k = 0; k < kEach; ++k) {
      const int e = tid * kEach + k, c = e < a.E ? count[e] : 0;
      rows += c;
      tiles += (c + a.tile_rows - 1) / a.tile_rows;
    }
    int r = rows, t = tiles;
    for (int o = 1; o < 64; o <<= 1) {
      const int r2 = __shfl_up(r, o, 64), t2 = __shfl_up(t, o, 64);
      if (tid >= o) { r += r2; t += t2; }
    }
    if (tid == 63) *a.num_tiles = t;
    r -= rows;
    t -= tiles;
#pragma unroll
    for (int k = 0; k < kEach; ++k) {
      const int e = tid * kEach + k;
      if (e < a.E) {
        start[e] = cursor[e] = r;
        tstart[e] = t;
        r += count[e];
        t += (count[e] + a.tile_rows - 1) / a.tile_rows;
      }
    }
  }
  __syncthreads();
  for (int e = tid; e < a.E; e += 1024)
    for (int k = 0, left = count[e]; left > 0; ++k, left -= a.tile_rows)
      a.tiles[tstart[e] + k] = make_int4(e, start[e] + k * a.tile_rows, min(left, a.tile_rows), 0);
  for (int i = tid; i < a.entries; i += 1024) {
    const int r = atomicAdd(&cursor[a.ids[i]], 1);
    a.row_of[i] = r;
    a.src[r] = i / a.top;
    a.row_weight[r] = a.weights[i];
  }
}

// ---------------------------------------------------------------------------------------------------------------
// fp32: 64 x 64 tiles of y = x W^T per expert (see f32_linear.hip), any K
constexpr int kGT = 64, kGK = 16;
struct GroupedF32Args {
  const float *x, *w;
  float *y;
  int64_t ldx;
  GroupedRows g;
  int32_t N, K, act;
};
__global__ __launch_bounds__(256) void grouped_f32_kernel(const GroupedF32Args a) {
  __shared__ __attribute__((aligned(16))) float Xs[kGT][kGK + 4], Ws[kGT][kGK + 4];
  if (static_cast<int>(blockIdx.y) >= *a.g.num_tiles) return;
  const int4 tile = a.g.tiles[blockIdx.y];
  const float *w = a.w + static_cast<int64_t>(tile.x) * a.N * a.K;
  const int m0 = tile.y, rows = tile.z, n0 = blockIdx.x * kGT;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, n = lane & 15, g = lane >> 4;
  floatx4 acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = floatx4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < a.K; k0 += kGK) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = i * 16 + tid / 16, c = tid % 16;
      const bool kin = k0 + c < a.K;
      const int64_t xr = r < rows ? (a.g.x_rows ? a.g.x_rows[m0 + r] : m0 + r) : 0;
      Xs[r][c] = kin && r < rows ? a.x[xr * a.ldx + k0 + c] : 0.f;
      Ws[r][c] = kin && n0 + r < a.N ? w[static_cast<int64_t>(n0 + r) * a.K + k0 + c] : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < kGK / 4; ++s) {
      const float v = Xs[wave * 16 + n][s * 4 + g];
#pragma unroll
      for (int i = 0; i < 4; ++i)
        acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(v, Ws[i * 16 + n][s * 4 + g], acc[i], 0, 0, 0);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int m = wave * 16 + g * 4 + r, c = n0 + i * 16 + n;
      const float up = __shfl(acc[i][r], (lane & ~15) | ((n & 7) + 8), 64);   // channels: 8 gate, then the 8 matching up
      if (m >= rows || c >= a.N) continue;
      const int64_t row = m0 + m;
      if (a.act == 0) a.y[row * a.N + c] = acc[i][r];
      else if (n < 8)
        a.y[row * (a.N / 2) + (c >> 4) * 8 + n] = clipped_glu(acc[i][r], up, a.g.row_scale ? a.g.row_scale[row] : 1.0f, a.g.limit);
    }
}

// ---------------------------------------------------------------------------------------------------------------
struct XieluArgs {
  const void *x;
  Partials part;
  int64_t ldx;
  int32_t col;            // first column of the activation's input in a row
  const void *pq;         // [2]
  void *out;
  int64_t ldo;
  int32_t rows, cols, padded;   // columns cols .. padded - 1 of `out` become zeros
};
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float xielu_f32(float z, float a, float b) {
  return z > 0.f ? fmaf(a * z, z, 0.5f * z) : fmaf(b, expm1f(z) - z, 0.5f * z);
}
template <typename T, int VEC, bool PART>
__global__ __launch_bounds__(256) void xielu_kernel(const XieluArgs a) {
  const int nch = a.padded / VEC;
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (item >= static_cast<int64_t>(a.rows) * nch) return;
  const int64_t row = item / nch;
  const int c = static_cast<int>(item - row * nch) * VEC;
  const float sa = softplus_f32(Elem<T>::ld(static_cast<const T *>(a.pq)));
  const float sb = 0.5f + softplus_f32(Elem<T>::ld(static_cast<const T *>(a.pq) + 1));
  const T *x = static_cast<const T *>(a.x) + row * a.ldx + a.col + c;
  T *o = static_cast<T *>(a.out) + row * a.ldo + c;
  if constexpr (VEC == 8) {
    float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (c < a.cols) {
      if constexpr (PART) a.part.ld8(row, a.col + c, f);
      else Elem<T>::ld8(x, f);
#pragma unroll
      for (int e = 0; e < 8; ++e) f[e] = xielu_f32(f[e], sa, sb);
    }
    Elem<T>::st8(o, f);
  } else {
    Elem<T>::st(o, c < a.cols ? xielu_f32(PART ? a.part.ld(row, a.col + c) : Elem<T>::ld(x), sa, sb) : 0.f);
  }
}

}  // namespace tlf

extern "C" int tlf_moe_route(const void *h, int64_t h_stride, const void *router, int32_t *ids, float *weights, int32_t n,
                             int32_t experts, int32_t K, int32_t top, int32_t dtype, void *stream) {
  using namespace tlf;
  if (n < 0 || experts <= 0 || experts > kMaxExperts || top <= 0 || top > experts || K <= 0 || K % 64 || h_stride < K) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (n == 0) return TLF_OK;
  if (!h || !router || !ids || !weights) return TLF_E_NULL;
  if (!aligned16(h) || !aligned16(router) || h_stride % 8) return TLF_E_ALIGN;
  const RouterArgs a{h, router, h_stride, ids, weights, n, experts, (experts + 15) / 16 * 16, K, top};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == TLF_DT_BF16)
    TLF_LAUNCH(router_kernel, dim3((n + 15) / 16), dim3(512), 16 * (a.E16 + 4) * 4, s, a);
  else
    TLF_LAUNCH(router_f32_kernel, dim3(n), dim3(256), 0, s, a);
  return launch_status();
}

extern "C" int tlf_moe_group(const int32_t *ids, const float *weights, int32_t *row_of, int32_t *src, float *row_weight,
                             int32_t *tiles, int32_t *num_tiles, int32_t max_tiles, int32_t n, int32_t top, int32_t experts,
                             int32_t tile_rows, void *stream) {
  using namespace tlf;
  if (n < 0 || top <= 0 || experts <= 0 || experts > kMaxExperts || tile_rows <= 0) return TLF_E_SHAPE;
  const int64_t entries = static_cast<int64_t>(n) * top;
  if (entries > (1 << 28) || max_tiles < entries / tile_rows + (entries < experts ? entries : experts)) return TLF_E_SHAPE;
  if (n == 0) return TLF_OK;
  if (!ids || !weights || !row_of || !src || !row_weight || !tiles || !num_tiles) return TLF_E_NULL;
  if (!aligned16(tiles)) return TLF_E_ALIGN;
  const GroupArgs a{ids, weights, row_of, src, row_weight, reinterpret_cast<int4 *>(tiles), num_tiles,
                    static_cast<int32_t>(entries), experts, top, tile_rows};
  TLF_LAUNCH(moe_group_kernel, dim3(1), dim3(1024), 0, static_cast<hipStream_t>(stream), a);
  return launch_status();
}

extern "C" int tlf_moe_gemm(const void *x, int64_t x_stride, int32_t x_count, const void *w, void *y, const int32_t *tiles,
                            const int32_t *num_tiles, int32_t max_tiles, int32_t tile_rows, const int32_t *x_rows,
                            const float *row_scale, int32_t rows, int32_t N, int32_t K, int32_t clipped_glu, float limit,
                            int32_t dtype, void *stream) {
  using namespace tlf;
  if (rows < 0 || N <= 0 || K <= 0 || N % 16 || max_tiles <= 0 || max_tiles > 65535 || x_stride < K || x_count < 0) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (rows == 0) return TLF_OK;
  if (!x || !w || !y || !tiles || !num_tiles) return TLF_E_NULL;
  const GroupedRows g{reinterpret_cast<const int4 *>(tiles), num_tiles, x_rows, row_scale,
                      static_cast<int64_t>(N) * K * (dtype == TLF_DT_BF16 ? 2 : 4), limit};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == TLF_DT_F32) {
    if (tile_rows != kGT) return TLF_E_SHAPE;
    const GroupedF32Args a{static_cast<const float *>(x), static_cast<const float *>(w), static_cast<float *>(y), x_stride, g, N, K, clipped_glu};
    TLF_LAUNCH(grouped_f32_kernel, dim3((N + kGT - 1) / kGT, max_tiles), dim3(256), 0, s, a);
    return launch_status();
  }
  if (tile_rows != 32 && tile_rows != 128) return TLF_E_SHAPE;
  if (!aligned16(x) || !aligned16(w) || !aligned16(y) || x_stride % 8) return TLF_E_ALIGN;
  if (static_cast<int64_t>(x_count) * x_stride * 2 > 0xffffffffll) return TLF_E_TOO_LARGE;   // x rows are 32-bit byte offsets
  GemmParams p{};
  p.x = static_cast<const unsigned char *>(x);
  p.ldx_bytes = x_stride * 2;
  p.w = static_cast<const unsigned char *>(w);
  p.y = static_cast<unsigned short *>(y);
  p.M = rows; p.N = N; p.K = K;
  p.m_tiles = max_tiles;
  p.act = clipped_glu ? 3 : 0;
  p.g = g;
  return launch_grouped(p, tile_rows, s);
}

extern "C" int tlf_xielu(const void *x, int64_t x_stride, const float *partials, int32_t splits, const float *scale,
                         int32_t col, const void *pq, void *out, int64_t out_stride, int32_t rows, int32_t cols,
                         int32_t padded_cols, int32_t dtype, void *stream) {
  using namespace tlf;
  if (rows < 0 || cols <= 0 || padded_cols < cols || col < 0 || x_stride < col + cols || out_stride < padded_cols) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (rows == 0) return TLF_OK;
  if (int rc = partials_check(partials, scale, splits, dtype)) return rc;
  if ((!x && splits <= 1) || !pq || !out) return TLF_E_NULL;
  XieluArgs a{x, Partials{partials, scale, rows * x_stride, static_cast<int32_t>(x_stride), splits}, x_stride, col, pq, out, out_stride, rows, cols, padded_cols};
  const bool vec = cols % 8 == 0 && padded_cols % 8 == 0 && col % 8 == 0 && x_stride % 8 == 0 && out_stride % 8 == 0 &&
                   aligned16(out) && (splits > 1 || aligned16(x));
  const int64_t items = static_cast<int64_t>(rows) * (padded_cols / (vec ? 8 : 1));
  const dim3 grid(static_cast<unsigned>((items + 255) / 256));
  hipStream_t s = static_cast<hipStream_t>(stream);
#define TLF_XI(T, PART)                                                                   \
  do {                                                                                    \
    if (vec) TLF_LAUNCH((xielu_kernel<T, 8, PART>), grid, dim3(256), 0, s, a);            \
    else TLF_LAUNCH((xielu_kernel<T, 1, PART>), grid, dim3(256), 0, s, a);                \
  } while (0)
  if (splits > 1) TLF_XI(unsigned short, true);
  else if (dtype == TLF_DT_BF16) TLF_XI(unsigned short, false);
  else TLF_XI(float, false);
#undef TLF_XI
  return launch_status();
}
