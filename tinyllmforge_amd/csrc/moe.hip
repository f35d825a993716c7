// Mixture of experts: router, grouping of the rows by expert, the grouped products, and the xIELU activation of dense
// layers.
//
//   router     z = W_router h (tlf_gemm_f32_sums or the fp32 product)
//   group      each row's experts and their weights, either the `top` largest logits and their sigmoids, or the `top` largest
//              of softmax + correction with their softmax values, normalised to a sum of 1; rows (token, k) in expert order, an
//              index each way, tiles of `tile_rows` rows of one expert.  Experts from E on (identity experts) have no rows
//   products   gemm_dlds_kernel<GROUPED> (gemm.hip) in bf16; a plain fp32 kernel here
// No host value depends on the routing: grids are sized for the worst case and tiles past the list's end leave at once,
// so a captured graph replays with any routing.
#include "gemm_shared.h"
#include "elem.h"

namespace tlf {

int launch_grouped(GemmParams p, int bm, hipStream_t stream);

constexpr int kMaxExperts = 512;

struct GroupArgs {
  const float *sums;        // [splits, n, E16] partial router logits
  int64_t plane;            // n * E16
  const void *correction;   // [choices] or NULL: sigmoid scores
  int32_t choices;          // E and the identity experts
  int32_t *ids;             // [entries] expert of entry (token, k)
  float *weights;           // [entries] its score
  int32_t *row_of;          // [entries] row of an entry in expert order
  int32_t *src;             // [entries] token of a row
  float *row_weight;        // [entries] weight of a row
  int4 *tiles;
  int32_t *num_tiles;
  int32_t *hist;            // [blocks, E]
  int32_t n, splits, E, E16, top, entries, tile_rows, blocks, f32;
};

__device__ __forceinline__ float wave_max(float v) {
  v = fmaxf(v, dpp_move<0xB1>(v));    // quad_perm [1, 0, 3, 2]
  v = fmaxf(v, dpp_move<0x4E>(v));    // quad_perm [2, 3, 0, 1]
  v = fmaxf(v, dpp_move<0x141>(v));   // row_half_mirror
  v = fmaxf(v, dpp_move<0x140>(v));   // row_mirror
  return max_lanes_16_32_48(v);
}

// One wave picks a token's `top` experts: by value, then the smaller index.  logit(e): expert e's.
//   NORM false: the largest logits; weights are their sigmoids
//   NORM true: the largest of softmax + correction; weights are their softmax values over the sum of the chosen ones
template <bool NORM, typename F>
__device__ __forceinline__ void pick_top(const GroupArgs &a, F logit, int32_t *ids, float *weights) {
  const int lane = threadIdx.x & 63;
  constexpr int kEach = kMaxExperts / 64;
  float v[kEach], s[kEach];
  int pick[kEach];
  const int all = a.choices;
#pragma unroll
  for (int i = 0; i < kEach; ++i) {
    v[i] = -INFINITY;
    s[i] = 0.f;
    pick[i] = -1;
    if (i * 64 < all) {            // uniform
      const int e = i * 64 + lane;
      const float z = logit(min(e, all - 1));
      if (e < all) v[i] = z > -3.0e38f ? z : -3.0e38f;     // every pick finds an expert, whatever the input
    }
  }
  if constexpr (NORM) {
    float m = v[0], sum = 0.f;
#pragma unroll
    for (int i = 1; i < kEach; ++i) m = fmaxf(m, v[i]);
    m = wave_max(m);
#pragma unroll
    for (int i = 0; i < kEach; ++i) {
      if (i * 64 >= all) continue;  // uniform
      s[i] = v[i] > -INFINITY ? expf(v[i] - m) : 0.f;
      sum += s[i];
    }
    sum = wave_sum(sum);
#pragma unroll
    for (int i = 0; i < kEach; ++i) {
      const int e = i * 64 + lane;
      s[i] /= sum;
      if (e < all) {
        const float c = a.f32 ? static_cast<const float *>(a.correction)[e] : bf16_bits_to_float(static_cast<const unsigned short *>(a.correction)[e]);
        v[i] = fmaxf(s[i] + c, -3.0e38f);
      }
    }
  }
  float chosen = 0.f;
  for (int k = 0; k < a.top; ++k) {
    float m = v[0];
#pragma unroll
    for (int i = 1; i < kEach; ++i) m = fmaxf(m, v[i]);
    m = wave_max(m);
    bool found = false;
#pragma unroll
    for (int i = 0; i < kEach; ++i) {
      if (found || i * 64 >= all) continue;          // uniform
      const unsigned long long who = __ballot(v[i] == m);
      if (who == 0) continue;
      found = true;
      if (NORM) chosen += __shfl(s[i], __ffsll(who) - 1, 64);
      if (lane == __ffsll(who) - 1) {
        ids[k] = i * 64 + lane;
        if (!NORM) weights[k] = sigmoid_f32(m);
        pick[i] = k;
        v[i] = -INFINITY;
      }
    }
  }
  if constexpr (NORM) {
#pragma unroll
    for (int i = 0; i < kEach; ++i)
      if (pick[i] >= 0) weights[pick[i]] = s[i] / (chosen + 1e-20f);
  }
}

template <bool NORM>
__global__ __launch_bounds__(256) void moe_pick_kernel(const GroupArgs a) {
  const int64_t tok = blockIdx.x * (blockDim.x / 64) + (threadIdx.x >> 6);
  if (tok >= a.n) return;
  const float *z = a.sums + tok * a.E16;
  pick_top<NORM>(a, [&](int e) __attribute__((always_inline)) {
    float v = 0.f;
#pragma unroll 16
    for (int k = 0; k < a.splits; ++k) v += z[k * a.plane + e];
    return v;
  }, a.ids + tok * a.top, a.weights + tok * a.top);
}

// From the experts' row counts: first row and first tile of each, the tile list.  The first wave scans, all threads write.
__device__ __forceinline__ void expert_tiles(const GroupArgs &a, const int *count, int *start, int *tstart) {
  const int tid = threadIdx.x;
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
        start[e] = r;
        tstart[e] = t;
        r += count[e];
        t += (count[e] + a.tile_rows - 1) / a.tile_rows;
      }
    }
  }
  __syncthreads();
  for (int e = tid; e < a.E; e += blockDim.x)
    for (int k = 0, left = count[e]; left > 0; ++k, left -= a.tile_rows)
      a.tiles[tstart[e] + k] = make_int4(e, start[e] + k * a.tile_rows, min(left, a.tile_rows), 0);
}

// The order of rows inside an expert is arbitrary (it enters no value).
__device__ __forceinline__ void place(const GroupArgs &a, int entry, int expert, float weight, int *cursor) {
  if (expert >= a.E) {          // an identity expert: no row
    a.row_of[entry] = -1;
    return;
  }
  const int r = atomicAdd(&cursor[expert], 1);
  a.row_of[entry] = r;
  a.src[r] = entry / a.top;
  a.row_weight[r] = weight;
}

// Few entries: grouped by one workgroup.
constexpr int kSmallEntries = 4096;
__global__ __launch_bounds__(1024) void moe_small_kernel(const GroupArgs a) {
  __shared__ int count[kMaxExperts], start[kMaxExperts], tstart[kMaxExperts];
  const int tid = threadIdx.x;
  int id[kSmallEntries / 1024];
  float weight[kSmallEntries / 1024];
#pragma unroll
  for (int k = 0; k < kSmallEntries / 1024; ++k) {
    const int i = tid + k * 1024;
    if (i < a.entries) {
      id[k] = a.ids[i];
      weight[k] = a.weights[i];
    }
  }
  for (int e = tid; e < a.E; e += 1024) count[e] = 0;
  __syncthreads();
#pragma unroll
  for (int k = 0; k < kSmallEntries / 1024; ++k)
    if (tid + k * 1024 < a.entries && id[k] < a.E) atomicAdd(&count[id[k]], 1);
  __syncthreads();
  expert_tiles(a, count, start, tstart);
  __syncthreads();
#pragma unroll
  for (int k = 0; k < kSmallEntries / 1024; ++k)
    if (tid + k * 1024 < a.entries) place(a, tid + k * 1024, id[k], weight[k], start);
}

// Many tokens: counts per block of entries, a scan over blocks and experts, placement.
constexpr int kBlockEntries = 1024;
__global__ __launch_bounds__(1024) void moe_count_kernel(const GroupArgs a) {
  __shared__ int count[kMaxExperts];
  for (int e = threadIdx.x; e < a.E; e += 1024) count[e] = 0;
  __syncthreads();
  const int i = blockIdx.x * kBlockEntries + threadIdx.x;
  if (i < a.entries && a.ids[i] < a.E) atomicAdd(&count[a.ids[i]], 1);
  __syncthreads();
  for (int e = threadIdx.x; e < a.E; e += 1024) a.hist[blockIdx.x * a.E + e] = count[e];
}
__global__ __launch_bounds__(kMaxExperts) void moe_scan_kernel(const GroupArgs a) {
  __shared__ int count[kMaxExperts], start[kMaxExperts], tstart[kMaxExperts];
  const int e = threadIdx.x;
  int sum = 0;
  if (e < a.E) {
#pragma unroll 8
    for (int b = 0; b < a.blocks; ++b) sum += a.hist[b * a.E + e];
    count[e] = sum;
  }
  __syncthreads();
  expert_tiles(a, count, start, tstart);
  if (e < a.E) {
    int at = start[e];
    for (int b0 = 0; b0 < a.blocks; b0 += 8) {
      int c[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) c[k] = a.hist[min(b0 + k, a.blocks - 1) * a.E + e];
#pragma unroll
      for (int k = 0; k < 8; ++k)
        if (b0 + k < a.blocks) {
          a.hist[(b0 + k) * a.E + e] = at;
          at += c[k];
        }
    }
  }
}
__global__ __launch_bounds__(1024) void moe_place_kernel(const GroupArgs a) {
  __shared__ int cursor[kMaxExperts];
  for (int e = threadIdx.x; e < a.E; e += 1024) cursor[e] = a.hist[blockIdx.x * a.E + e];
  __syncthreads();
  const int i = blockIdx.x * kBlockEntries + threadIdx.x;
  if (i < a.entries) place(a, i, a.ids[i], a.weights[i], cursor);
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
        a.y[row * (a.N / 2) + (c >> 4) * 8 + n] = a.act == 2 ? silu_f32(acc[i][r]) * up
                                                       : clipped_glu(acc[i][r], up, a.g.row_scale ? a.g.row_scale[row] : 1.0f, a.g.limit);
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

extern "C" size_t tlf_moe_group_workspace_bytes(int32_t n, int32_t top, int32_t experts) {
  if (n <= 0 || top <= 0 || experts <= 0) return 0;
  const int64_t entries = static_cast<int64_t>(n) * top;
  return static_cast<size_t>((entries + tlf::kBlockEntries - 1) / tlf::kBlockEntries) * experts * 4;
}

extern "C" int tlf_moe_group(const float *sums, int32_t splits, int32_t *ids, float *weights, int32_t *row_of, int32_t *src,
                             float *row_weight, int32_t *tiles, int32_t *num_tiles, int32_t max_tiles, int32_t n, int32_t top,
                             int32_t experts, int32_t identity, const void *correction, int32_t dtype, int32_t tile_rows,
                             void *workspace, size_t workspace_bytes, void *stream) {
  using namespace tlf;
  if (n < 0 || top <= 0 || experts <= 0 || identity < 0 || experts > kMaxExperts - identity || top > experts + identity || tile_rows <= 0 || splits <= 0 || splits > 64) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  const int64_t entries = static_cast<int64_t>(n) * top;
  if (entries > (1 << 28) || max_tiles < entries / tile_rows + (entries < experts ? entries : experts)) return TLF_E_SHAPE;
  if (n == 0) return TLF_OK;
  if (!sums || !ids || !weights || !row_of || !src || !row_weight || !tiles || !num_tiles) return TLF_E_NULL;
  if (!aligned16(tiles)) return TLF_E_ALIGN;
  GroupArgs a{};
  a.sums = sums; a.ids = ids; a.weights = weights; a.row_of = row_of; a.src = src; a.row_weight = row_weight;
  a.tiles = reinterpret_cast<int4 *>(tiles); a.num_tiles = num_tiles; a.hist = static_cast<int32_t *>(workspace);
  a.n = n; a.splits = splits; a.E = experts; a.E16 = (experts + identity + 15) / 16 * 16; a.top = top;
  a.correction = correction; a.choices = experts + identity; a.f32 = dtype == TLF_DT_F32;
  a.plane = static_cast<int64_t>(n) * a.E16;
  a.entries = static_cast<int32_t>(entries); a.tile_rows = tile_rows;
  a.blocks = static_cast<int32_t>((entries + kBlockEntries - 1) / kBlockEntries);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (entries > kSmallEntries && (!workspace || workspace_bytes < tlf_moe_group_workspace_bytes(n, top, experts))) return TLF_E_WORKSPACE;
  const int waves = n <= 1024 ? 1 : 4;
  if (correction) TLF_LAUNCH((moe_pick_kernel<true>), dim3((n + waves - 1) / waves), dim3(64 * waves), 0, s, a);
  else TLF_LAUNCH((moe_pick_kernel<false>), dim3((n + waves - 1) / waves), dim3(64 * waves), 0, s, a);
  if (entries <= kSmallEntries) {
    TLF_LAUNCH(moe_small_kernel, dim3(1), dim3(1024), 0, s, a);
    return launch_status();
  }
  TLF_LAUNCH(moe_count_kernel, dim3(a.blocks), dim3(1024), 0, s, a);
  TLF_LAUNCH(moe_scan_kernel, dim3(1), dim3(kMaxExperts), 0, s, a);
  TLF_LAUNCH(moe_place_kernel, dim3(a.blocks), dim3(1024), 0, s, a);
  return launch_status();
}

extern "C" int tlf_moe_gemm(const void *x, int64_t x_stride, int32_t x_count, const void *w, void *y, const int32_t *tiles,
                            const int32_t *num_tiles, int32_t max_tiles, int32_t tile_rows, const int32_t *x_rows,
                            const float *row_scale, int32_t rows, int32_t N, int32_t K, int32_t act, float limit,
                            int32_t dtype, void *stream) {
  using namespace tlf;
  if (act < 0 || act > 2) return TLF_E_UNSUPPORTED;
  if (rows < 0 || N <= 0 || K <= 0 || N % 16 || max_tiles <= 0 || max_tiles > 65535 || x_stride < K || x_count < 0) return TLF_E_SHAPE;
  if (dtype != TLF_DT_BF16 && dtype != TLF_DT_F32) return TLF_E_UNSUPPORTED;
  if (rows == 0) return TLF_OK;
  if (!x || !w || !y || !tiles || !num_tiles) return TLF_E_NULL;
  const GroupedRows g{reinterpret_cast<const int4 *>(tiles), num_tiles, x_rows, row_scale,
                      static_cast<int64_t>(N) * K * (dtype == TLF_DT_BF16 ? 2 : 4), limit, act == 2};
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == TLF_DT_F32) {
    if (tile_rows != kGT) return TLF_E_SHAPE;
    const GroupedF32Args a{static_cast<const float *>(x), static_cast<const float *>(w), static_cast<float *>(y), x_stride, g, N, K, act};
    TLF_LAUNCH(grouped_f32_kernel, dim3((N + kGT - 1) / kGT, max_tiles), dim3(256), 0, s, a);
    return launch_status();
  }
  if (tile_rows != 32 && tile_rows != 64 && tile_rows != 128 && tile_rows != 256) return TLF_E_SHAPE;
  if (!aligned16(x) || !aligned16(w) || !aligned16(y) || x_stride % 8) return TLF_E_ALIGN;
  if (static_cast<int64_t>(x_count) * x_stride * 2 > 0xffffffffll) return TLF_E_TOO_LARGE;   // x rows are 32-bit byte offsets
  GemmParams p{};
  p.x = static_cast<const unsigned char *>(x);
  p.ldx_bytes = x_stride * 2;
  p.w = static_cast<const unsigned char *>(w);
  p.y = static_cast<unsigned short *>(y);
  p.M = rows; p.N = N; p.K = K;
  p.m_tiles = max_tiles;
  p.act = act ? 3 : 0;
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
