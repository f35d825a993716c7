/*
 * tlf_hip.h - C ABI of libtlf_hip.so: the per-token hot path of a TinyLLMForge
 * (tinyvllm) engine as hand-written HIP kernels for gfx950 (MI355X).
 *
 * Conventions (all entry points):
 *   - extern "C", plain pointers and sizes; no C++ or torch types.
 *   - Every pointer is a DEVICE pointer owned by the caller (the reference lets
 *     PyTorch own every buffer, so the binding passes tensor.data_ptr()).
 *   - The last argument is a hipStream_t passed as void*; work is only enqueued
 *     on that stream.  No entry point allocates, frees, synchronises or reads
 *     device memory on the host, so every call can be stream-captured into a
 *     hipGraph.  Launch geometry depends only on the integer arguments, never
 *     on device data.
 *   - Return value: 0 = ok, < 0 = rejected argument (TLF_E_*), > 0 = hipError_t
 *     of the failed launch.  Nothing is launched when an argument is rejected.
 *   - "bf16" is bfloat16 stored as uint16; "rows" are tokens unless said otherwise.
 *   - Scratch memory is caller provided: ask tlf_*_workspace_bytes() and pass a
 *     buffer of at least that size (256-byte aligned).
 *
 * Each declaration cites the reference interface (file:line under the
 * reference's tinyvllm/ package) that it replaces.
 */
#ifndef TLF_HIP_H
#define TLF_HIP_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define TLF_ABI_VERSION 1

#define TLF_OK 0
#define TLF_E_NULL (-1)        /* a required pointer is NULL                         */
#define TLF_E_SHAPE (-2)       /* a size is negative, zero where not allowed, or unsupported */
#define TLF_E_ALIGN (-3)       /* a pointer or stride breaks the stated alignment    */
#define TLF_E_WORKSPACE (-4)   /* workspace missing or too small                     */
#define TLF_E_UNSUPPORTED (-5) /* a combination this build has no kernel for          */
#define TLF_E_TOO_LARGE (-6)   /* a size beyond the fixed scratch of a no-allocation entry point */

/* KV-cache element types */
#define TLF_KV_BF16 0
#define TLF_KV_FP8_E4M3 1 /* OCP e4m3fn, per-KV-head fp32 scale */

/* Tensor element types of the entry points that take a `dtype` */
#define TLF_DT_BF16 0
#define TLF_DT_F32 1

/* ABI version of the loaded library (== TLF_ABI_VERSION it was built with). */
int tlf_version(void);
/* Static, human readable text for a return code of this library. */
const char *tlf_error_string(int code);
/* Multiprocessor count and LDS bytes per workgroup of the current device
 * (host query; either out pointer may be NULL). */
int tlf_device_info(int32_t *num_cus, int32_t *lds_bytes);
/* Number of kernels this library has launched in this process so far (host counter, every entry point).
 * A statistic for benchmarks: read it before and after one eager engine step, or around a graph capture,
 * to count the kernels of a step.  No counterpart in the reference. */
int64_t tlf_kernel_launches(void);

/* ---------------------------------------------------------------------------
 * a1  store_kvcache   replaces layers/attention.py:33-48 (Triton kernel 9-30)
 *
 *   cache_row(slot[i]) = key[i] / value[i]  for every token i with slot[i] >= 0
 *
 * key/value: [num_tokens, row_bytes] rows, 16-byte aligned, row strides in
 * BYTES (value is a strided view into the qkv projection in the reference,
 * models/qwen3.py:79).  k_cache/v_cache: [num_slots, row_bytes] contiguous
 * (= [nblk, block_size, Hkv, Dh]).  row_bytes % 16 == 0.  A negative slot is
 * skipped (graph padding rows); slot >= num_slots is also skipped, never
 * written.  Pure byte copy: exact for any element type.
 */
int tlf_store_kvcache(const void *key, int64_t key_stride_bytes,
                      const void *value, int64_t value_stride_bytes,
                      void *k_cache, void *v_cache,
                      const int32_t *slot_mapping, int32_t num_tokens,
                      int32_t row_bytes, int64_t num_slots, void *stream);

/* a13 (build-defined, no reference counterpart): bf16 rows -> e4m3 cache rows,
 * c = e4m3(sat(x / scale[h])).  key/value rows are [Hkv, Dh] bf16 (strides in
 * bytes), cache rows are Hkv*Dh bytes.  k_scale/v_scale: fp32 [Hkv].  Dh % 8 == 0. */
int tlf_store_kvcache_fp8(const void *key, int64_t key_stride_bytes,
                          const void *value, int64_t value_stride_bytes,
                          void *k_cache, void *v_cache,
                          const int32_t *slot_mapping, int32_t num_tokens,
                          int32_t num_kv_heads, int32_t head_dim,
                          const float *k_scale, const float *v_scale,
                          int64_t num_slots, void *stream);

/* ---------------------------------------------------------------------------
 * a5  RMSNorm.rms_forward   replaces layers/layernorm.py:21-31
 *
 *   y = bf16( bf16( x * rsqrt(mean(x^2) + eps) ) * w )      (fp32 math)
 *
 * x is viewed as [outer, inner, cols] bf16 with element strides
 * (x_outer_stride, cols, 1): the q/k-norm call normalises every head of a
 * strided slice of the qkv projection (models/qwen3.py:80-83), the layer norm
 * uses inner = 1.  y is [outer, inner, cols] contiguous.  cols % 8 == 0,
 * cols <= 16384, 16-byte aligned rows.
 */
int tlf_rmsnorm(const void *x, int64_t x_outer_stride, const void *weight, void *y,
                int32_t outer, int32_t inner, int32_t cols, float eps, void *stream);

/* a6  RMSNorm.add_rms_forward   replaces layers/layernorm.py:33-45
 *
 *   s = x + residual (fp32); residual_out = bf16(s);
 *   y = bf16( bf16( s * rsqrt(mean(s^2) + eps) ) * w )
 *
 * All [rows, cols] bf16 contiguous.  y may alias x and residual_out may alias
 * residual (each thread reads its elements before writing them).
 */
int tlf_add_rmsnorm(const void *x, const void *residual, const void *weight,
                    void *y, void *residual_out,
                    int32_t rows, int32_t cols, float eps, void *stream);

/* ---------------------------------------------------------------------------
 * a7  RotaryEmbedding.forward   replaces layers/rotary_embedding.py:41-57 (+5-15)
 *
 *   cs = cos_sin[positions[i]]  (fp32 [max_pos, head_dim] = cos || sin)
 *   per head: y[:d/2] = cos*x[:d/2] - sin*x[d/2:], y[d/2:] = cos*x[d/2:] + sin*x[:d/2]
 *   (neox half split, fp32 products rounded separately, one bf16 rounding)
 *
 * q: [n, num_q_heads*head_dim] bf16 with row stride q_stride (elements), k
 * likewise; outputs contiguous and may alias the inputs.  positions int64 [n],
 * each in [0, max_pos) (a row whose position lies outside the table is copied
 * to the output unrotated; tlf_qknorm_rope_store does the same).  head_dim % 16 == 0.
 */
int tlf_rope(const int64_t *positions, const void *q, int64_t q_stride,
             const void *k, int64_t k_stride, const float *cos_sin,
             void *q_out, void *k_out, int32_t n, int32_t num_q_heads,
             int32_t num_kv_heads, int32_t head_dim, int32_t max_pos, void *stream);

/* Fused form of the reference's op sequence models/qwen3.py:79-94 +
 * layers/attention.py:94-95: q/k RMSNorm over head_dim (a5), RoPE (a7) and the
 * KV-cache store (a1; bf16 or e4m3 by kv_dtype) in one pass over the qkv
 * projection [n, (Hq + 2 Hkv) * head_dim] (row stride qkv_stride elements).
 * Writes q_out [n, Hq*head_dim] contiguous; k/v go only to the caches when
 * slot_mapping is non-NULL, and k_out/v_out (contiguous, may be NULL) receive
 * the rotated K and the V rows for the prefill attention.  Every intermediate
 * rounding of the unfused sequence is kept, so results are bit-identical to
 * running tlf_rmsnorm, tlf_rope and tlf_store_kvcache one after the other.
 * head_dim == 128.
 */
int tlf_qknorm_rope_store(const void *qkv, int64_t qkv_stride,
                          const void *q_norm_weight, const void *k_norm_weight, float eps,
                          const int64_t *positions, const float *cos_sin, int32_t max_pos,
                          void *q_out, void *k_out, void *v_out,
                          void *k_cache, void *v_cache, const int32_t *slot_mapping,
                          int64_t num_slots, int32_t kv_dtype,
                          const float *k_scale, const float *v_scale,
                          int32_t n, int32_t num_q_heads, int32_t num_kv_heads,
                          int32_t head_dim, void *stream);

/* ---------------------------------------------------------------------------
 * a8  SiluAndMul.forward   replaces layers/activation.py:11-14
 *
 *   y = bf16( bf16(silu(x[:, :I])) * x[:, I:] )      x [rows, 2I] -> y [rows, I]
 *
 * bf16, contiguous, I % 8 == 0.
 */
int tlf_silu_and_mul(const void *x, void *y, int32_t rows, int32_t inter, void *stream);

/* ---------------------------------------------------------------------------
 * a9  Sampler.forward, greedy branch   replaces layers/sampler.py:13-14,21
 *
 *   out[b] = first index of max(logits[b, :])       logits bf16 [rows, vocab]
 *
 * (bf16 -> fp32 is monotone, so the argmax over bf16 equals the reference's
 * argmax over the fp32 cast; -0 == +0; NaN logits are not supported.)
 * out: int64 [rows].  logits row stride in elements.  Needs a workspace.
 */
size_t tlf_argmax_workspace_bytes(int32_t rows, int32_t vocab);
int tlf_argmax(const void *logits, int64_t row_stride, int64_t *out,
               int32_t rows, int32_t vocab, void *workspace, size_t workspace_bytes,
               void *stream);

/* tlf_argmax without a workspace argument and without any allocation.  No counterpart in the
 * reference: it is for callers that cannot allocate device memory - code under hipGraph capture, tight
 * serving loops, harnesses that forbid hipMalloc - and so cannot provide (or grow) the workspace that
 * tlf_argmax asks for.  Same kernels and result as tlf_argmax; the partial keys live in a 1 MiB
 * file-scope device array of the library (one copy per GPU, held until the process ends), which
 * bounds rows <= tlf_argmax_noalloc_max_rows() (1024): more rows return TLF_E_TOO_LARGE.  The
 * array's device address is looked up on the first call on each device (a host-side query, no
 * allocation; make that first call outside a stream capture).  Calls on one GPU share the array:
 * calls that may overlap in time (different streams) race; calls on one stream are ordered.
 * Nothing needs clearing between calls (every key read was written by the same call). */
int tlf_argmax_noalloc_max_rows(void);
int tlf_argmax_noalloc(const void *logits, int64_t row_stride, int64_t *out,
                       int32_t rows, int32_t vocab, void *stream);

/* Sampler.forward with temperatures   replaces layers/sampler.py:13-21
 *
 *   T[b] == 0:  out[b] = first index of max(logits[b, :])
 *   T[b]  > 0:  out[b] = argmax_i softmax(logits[b, :] / T[b])_i / (e_i + 1e-10),  e_i ~ Exp(1)
 *               computed as argmax_i logits[b, i] / T[b] - log(e_i + 1e-10)  (same index: the row's
 *               normaliser is common and log is monotone), one pass over the row.
 *
 * The reference takes e from torch's device generator, whose stream no kernel can reproduce; here
 * e_i = -log(u_i) with u from Philox4x32-10: key = seed, counter = (i / 4, b, offset) gives the
 * uniforms of elements 4 (i / 4) .. + 3, u = (x >> 8) * 2^-24 + 2^-25.  Same distribution, its
 * own stream; the caller advances offset once per call.
 * logits bf16 [rows, vocab] (row stride in elements), temperatures fp32 [rows] >= 0, out int64
 * [rows].  workspace: tlf_argmax_workspace_bytes(rows, vocab). */
int tlf_sample(const void *logits, int64_t row_stride, const float *temperatures, int64_t *out,
               int32_t rows, int32_t vocab, uint64_t seed, uint64_t offset,
               void *workspace, size_t workspace_bytes, void *stream);

/* ---------------------------------------------------------------------------
 * a10  weight-only int8 linear (build-defined; the reference has bf16 F.linear
 * only: layers/linear.py:48-49, 82-83, 180-181; same [N, K] weight layout)
 *
 *   y[m, n] = bf16( (sum_k x[m, k] * float(wq[n, k])) * scale[n] )   fp32 accumulate
 *
 * x: bf16 [M, K] row stride x_stride (elements); wq: the int8 weight IN TILE ORDER, i.e. the output
 * of tlf_w8a16_pack_weight for the row-major [N, K] weight (same bytes, re-ordered so that every wave
 * reads contiguous runs: the 16-byte piece W[n, 16 a .. 16 a + 15] sits at byte
 * ((n / 32) * (K / 32) + a / 2) * 1024 + (a % 2) * 512 + (n % 32) * 16; rows are padded to a multiple of
 * 32); scale: fp32 [N]; y: bf16 [M, N] contiguous.  K % 64 == 0, N % 16 == 0.  Every W8A16 entry point
 * below takes the weight in this order.
 * workspace: fp32 partial sums when the kernel plan for (M, N, K) splits K across workgroups
 * (few output tiles, long K); tlf_w8a16_gemm_workspace_bytes gives the size for this and for
 * tlf_bf16_gemm (0 when neither plan splits), 16-byte aligned.
 */
size_t tlf_w8a16_packed_bytes(int32_t N, int32_t K);   /* = round_up(N, 32) * K */
int tlf_w8a16_pack_weight(const void *wq_rowmajor, void *packed, int32_t N, int32_t K, void *stream);
size_t tlf_w8a16_gemm_workspace_bytes(int32_t M, int32_t N, int32_t K);
int tlf_w8a16_gemm(const void *x, int64_t x_stride, const void *wq, const float *scale,
                   void *y, int32_t M, int32_t N, int32_t K,
                   void *workspace, size_t workspace_bytes, void *stream);

/* a10 / f1  bf16 linear   replaces layers/linear.py:48-49, 82-83, 180-181 and the
 * logits product layers/embed_head.py:63
 *
 *   y[m, n] = bf16( sum_k x[m, k] * w[n, k] )      fp32 accumulate
 *
 * Same shapes and constraints as tlf_w8a16_gemm with w bf16 [N, K].
 */
int tlf_bf16_gemm(const void *x, int64_t x_stride, const void *w, void *y,
                  int32_t M, int32_t N, int32_t K,
                  void *workspace, size_t workspace_bytes, void *stream);

/* gate_up projection fused with the activation: replaces MergedColumnParallelLinear.forward
 * (layers/linear.py:82-83) followed by SiluAndMul.forward (layers/activation.py:11-14) in
 * Qwen3MLP.forward (models/qwen3.py:123-130).
 *
 *   g = bf16(scale[..] * sum_k x[m,k] wq[.., k]),  u likewise
 *   y[m, c] = bf16( bf16(silu(g[m, c])) * u[m, c] )          y: bf16 [M, N/2] contiguous
 *
 * wq / scale rows are INTERLEAVED (before tlf_w8a16_pack_weight): rows 16 j .. 16 j + 7 are gate channels 8 j .. 8 j + 7 and rows
 * 16 j + 8 .. 16 j + 15 the matching up channels (N = 2 x intermediate size, N % 16 == 0), so that
 * both halves of a product sit in one lane's accumulators.  Bit-identical to tlf_w8a16_gemm on
 * the same interleaved weight followed by tlf_silu_and_mul on the de-interleaved result.
 * Needs no workspace (K is never split across workgroups).  Other constraints as tlf_w8a16_gemm. */
int tlf_w8a16_gemm_silu_mul(const void *x, int64_t x_stride, const void *wq, const float *scale,
                            void *y, int32_t M, int32_t N, int32_t K, void *stream);
/* The same with bf16 weights: w bf16 [N, K] row-major with its rows interleaved the same way (no scale). */
int tlf_bf16_gemm_silu_mul(const void *x, int64_t x_stride, const void *w, void *y,
                           int32_t M, int32_t N, int32_t K, void *stream);

/* Row-parallel projection fused with what follows it in a decoder layer: replaces
 * RowParallelLinear.forward (layers/linear.py:181-183; o_proj, down_proj) followed by
 * RMSNorm.add_rms_forward (layers/layernorm.py:33-45) of post_attention_layernorm, of the next
 * layer's input_layernorm, or of the final norm (models/qwen3.py:163-166, 188-190).
 *
 *   h = bf16(scale[n] * sum_k x[m,k] wq[n,k])          (tlf_bf16_gemm_add_rmsnorm: no scale, w bf16)
 *   s = h + residual (fp32);  residual_out = bf16(s)
 *   y = bf16( bf16( s * rsqrt(mean(s^2) + eps) ) * norm_weight )
 *
 * residual, y, residual_out: bf16 [M, N] contiguous; norm_weight bf16 [N]; N <= 16384;
 * residual_out may alias residual.  Bit-identical to the GEMM entry point followed by
 * tlf_add_rmsnorm.  When the plan for (M, N, K) splits K across workgroups, the
 * sum of the partial products, the residual add and the norm are one kernel (h never goes to
 * memory); otherwise h is staged in the workspace and the two kernels run back to back.
 * workspace: tlf_gemm_add_rmsnorm_workspace_bytes(M, N, K) bytes, 256-byte aligned.
 * Other constraints as tlf_w8a16_gemm. */
size_t tlf_gemm_add_rmsnorm_workspace_bytes(int32_t M, int32_t N, int32_t K);
int tlf_w8a16_gemm_add_rmsnorm(const void *x, int64_t x_stride, const void *wq, const float *scale,
                               const void *residual, const void *norm_weight, void *y,
                               void *residual_out, int32_t M, int32_t N, int32_t K, float eps,
                               void *workspace, size_t workspace_bytes, void *stream);
int tlf_bf16_gemm_add_rmsnorm(const void *x, int64_t x_stride, const void *w, const void *residual,
                              const void *norm_weight, void *y, void *residual_out, int32_t M,
                              int32_t N, int32_t K, float eps, void *workspace,
                              size_t workspace_bytes, void *stream);

/* qkv projection fused with what follows it in the attention block: replaces
 * QKVParallelLinear.forward (layers/linear.py:82-83 through models/qwen3.py:78) followed by the
 * q/k RMSNorm, RoPE and KV-cache store that tlf_qknorm_rope_store performs (models/qwen3.py:79-94,
 * layers/attention.py:94-95).
 *
 *   qkv = bf16(scale[c] * sum_k x[t,k] wq[c,k])   [n, (Hq + 2 Hkv) * head_dim]   (bf16 entry: no scale, w bf16)
 *   then exactly tlf_qknorm_rope_store(qkv, ...): same arguments, same outputs, same bits.
 *
 * When the plan for (n, (Hq + 2 Hkv) * head_dim, K) splits K across workgroups, the sum of the partial
 * products, the norms, the rotation and the store are one kernel (qkv never goes to memory); otherwise qkv
 * is staged in the workspace and the two kernels run back to back.
 * workspace: tlf_gemm_qknorm_rope_store_workspace_bytes(n, (Hq + 2 Hkv) * head_dim, K) bytes, 256-byte
 * aligned.  Other constraints as tlf_w8a16_gemm / tlf_bf16_gemm and tlf_qknorm_rope_store. */
size_t tlf_gemm_qknorm_rope_store_workspace_bytes(int32_t M, int32_t N, int32_t K);
int tlf_w8a16_gemm_qknorm_rope_store(const void *x, int64_t x_stride, const void *wq, const float *scale,
                                     const void *q_norm_weight, const void *k_norm_weight, float eps,
                                     const int64_t *positions, const float *cos_sin, int32_t max_pos,
                                     void *q_out, void *k_out, void *v_out,
                                     void *k_cache, void *v_cache, const int32_t *slot_mapping,
                                     int64_t num_slots, int32_t kv_dtype,
                                     const float *k_scale, const float *v_scale,
                                     int32_t n, int32_t num_q_heads, int32_t num_kv_heads,
                                     int32_t head_dim, int32_t K,
                                     void *workspace, size_t workspace_bytes, void *stream);
int tlf_bf16_gemm_qknorm_rope_store(const void *x, int64_t x_stride, const void *w,
                                    const void *q_norm_weight, const void *k_norm_weight, float eps,
                                    const int64_t *positions, const float *cos_sin, int32_t max_pos,
                                    void *q_out, void *k_out, void *v_out,
                                    void *k_cache, void *v_cache, const int32_t *slot_mapping,
                                    int64_t num_slots, int32_t kv_dtype,
                                    const float *k_scale, const float *v_scale,
                                    int32_t n, int32_t num_q_heads, int32_t num_kv_heads,
                                    int32_t head_dim, int32_t K,
                                    void *workspace, size_t workspace_bytes, void *stream);

/* LM head fused with the greedy sample: replaces ParallelLMHead.forward's product
 * (layers/embed_head.py:63) followed by Sampler.forward's greedy branch (layers/sampler.py:13-14,21)
 * when every temperature of the batch is 0.
 *
 *   token_ids[m] = argmax_n bf16( sum_k x[m,k] * w[n,k] ),  first index among ties      int64 [M]
 *
 * The [M, N] logits are never stored (more than 16 tokens; a smaller batch stages them in the
 * workspace): the GEMM epilogue keeps one (value, index) key per token, N-tile and wave, and a
 * second small kernel takes their maximum.  Identical to tlf_bf16_gemm followed by tlf_argmax.
 * workspace: tlf_gemm_argmax_workspace_bytes(M, N, K) bytes, 256-byte aligned.
 * Other constraints as tlf_bf16_gemm. */
size_t tlf_gemm_argmax_workspace_bytes(int32_t M, int32_t N, int32_t K);
int tlf_bf16_gemm_argmax(const void *x, int64_t x_stride, const void *w, int64_t *token_ids,
                         int32_t M, int32_t N, int32_t K,
                         void *workspace, size_t workspace_bytes, void *stream);

/* Diagnostic, no counterpart in the reference, touches no GPU: the kernel plan the two GEMM entry
 * points would use for a shape.  plan8 = {tile channels, tile tokens, LDS stages, waves/SIMD budget,
 * K-groups per workgroup, split-K factor, K per split, N-tile columns per XCD patch}; tile 0 x 0
 * means the skinny kernel.  Returns TLF_OK when a kernel instance exists for the plan,
 * TLF_E_UNSUPPORTED otherwise (the GEMM call would return the same). */
int tlf_gemm_plan(int32_t M, int32_t N, int32_t K, int32_t w8, int32_t *plan8);

/* ---------------------------------------------------------------------------
 * a3  paged decode attention   replaces the decode branch layers/attention.py:106-109
 *     (flash_attn_with_kvcache, one query token per sequence)
 *
 *   out[b, h] = softmax(scale * q[b, h] . K_b^T) V_b    over rows 0..context_lens[b]-1,
 *   row t of sequence b = cache[block_tables[b, t / block_size], t % block_size, h / (Hq/Hkv), :]
 *
 * q: bf16 [batch, Hq, Dh] with row stride q_stride (elements); caches
 * [num_cache_blocks, block_size, Hkv, Dh] contiguous, bf16 or e4m3 (kv_dtype;
 * e4m3 rows are dequantised as float(c) * scale[kvh], k_scale/v_scale fp32 [Hkv],
 * NULL for bf16); block_tables int32 [batch, max_blocks] with row stride
 * block_table_stride; entries at or beyond ceil(context_len / block_size) are
 * never dereferenced (the reference pads them with -1 or 0); entries outside
 * [0, num_cache_blocks) inside that range make the kernel skip the block.
 * context_lens int32 [batch]; a sequence with context_len <= 0 gets zeros.
 * out: bf16 [batch, Hq*Dh] contiguous.  fp32 softmax and accumulation; the
 * probabilities enter the P.V product as a bf16 hi + lo pair (about 16 significant bits;
 * flash-attn rounds them to one bf16).
 * Dh == 128, Hq % Hkv == 0, Hq/Hkv <= 16, Hkv in {1,2,4,8,16}, block_size % 16 == 0,
 * batch <= 1024.
 * Calls that share a workspace must not overlap in time.
 */
size_t tlf_paged_decode_attn_workspace_bytes(int32_t batch, int32_t num_q_heads,
                                             int32_t head_dim, int32_t max_blocks,
                                             int32_t block_size);
int tlf_paged_decode_attn(const void *q, int64_t q_stride,
                          const void *k_cache, const void *v_cache, int32_t kv_dtype,
                          const float *k_scale, const float *v_scale,
                          const int32_t *block_tables, int64_t block_table_stride,
                          const int32_t *context_lens, void *out,
                          int32_t batch, int32_t num_q_heads, int32_t num_kv_heads,
                          int32_t head_dim, int32_t block_size, int32_t max_blocks,
                          int64_t num_cache_blocks, float scale,
                          void *workspace, size_t workspace_bytes, void *stream);

/* a3 with the split of the work made once per decode step instead of once per layer (build-defined; the reference
 * calls flash_attn_with_kvcache per layer, layers/attention.py:106-109, and every layer of a step passes the same
 * context_lens and block_tables).  tlf_paged_decode_plan scans the lengths, finds every workgroup's first sequence
 * and copies the block-table entries it needs first into plan (tlf_paged_decode_plan_bytes() bytes, 16-byte
 * aligned); tlf_paged_decode_attn_planned is tlf_paged_decode_attn reading that plan: same arguments (the lengths
 * and tables must be the ones the plan was made from, with the same batch, block_size and max_blocks), same
 * results bit for bit, and its first cache rows are requested one memory round trip after the kernel starts
 * instead of three.  The plan is read-only to the attention calls: one plan serves all layers of the step.  A plan
 * made for another batch size (or for a grid another max_blocks / block_size gives) is recognised by its header
 * and turns every output row into NaN; one made from other lengths of the same batch cannot be told apart and gives
 * what those lengths would give. */
size_t tlf_paged_decode_plan_bytes(void);
int tlf_paged_decode_plan(const int32_t *context_lens, const int32_t *block_tables,
                          int64_t block_table_stride, int32_t batch, int32_t block_size,
                          int32_t max_blocks, void *plan, size_t plan_bytes, void *stream);
int tlf_paged_decode_attn_planned(const void *q, int64_t q_stride,
                                  const void *k_cache, const void *v_cache, int32_t kv_dtype,
                                  const float *k_scale, const float *v_scale,
                                  const int32_t *block_tables, int64_t block_table_stride,
                                  const int32_t *context_lens, void *out,
                                  int32_t batch, int32_t num_q_heads, int32_t num_kv_heads,
                                  int32_t head_dim, int32_t block_size, int32_t max_blocks,
                                  int64_t num_cache_blocks, float scale,
                                  void *workspace, size_t workspace_bytes, const void *plan, void *stream);

/* ---------------------------------------------------------------------------
 * a4  varlen causal prefill attention   replaces the prefill branch
 *     layers/attention.py:96-105 (flash_attn_varlen_func, causal=True)
 *
 * q: bf16 [total_q, Hq, Dh] row stride q_stride (elements).  Sequence s owns
 * query rows cu_seqlens_q[s]..cu_seqlens_q[s+1]-1 and keys
 * 0..len_k-1 with len_k = cu_seqlens_k[s+1] - cu_seqlens_k[s].  The causal mask
 * is bottom-right aligned: query i sees keys 0..(len_k - len_q) + i.
 *   block_tables == NULL: k/v are packed rows [total_k, Hkv, Dh] with row
 *     strides k_stride/v_stride (elements; v is a strided view in the reference).
 *   block_tables != NULL: k/v are the paged caches (layout and kv_dtype as in
 *     tlf_paged_decode_attn) and EVERY sequence reads its keys from them
 *     (layers/attention.py:99-100).
 * out: bf16 [total_q, Hq*Dh] contiguous.  max_seqlen_q bounds the grid.
 * fp32 softmax and accumulation.  The P.V product runs in fp16: P with 11 significant bits (flash-attn rounds
 * it to one bf16, 8 bits), carried as 2^15 p so that weights down to 2^-29 of the row maximum are normal fp16
 * numbers (the factor cancels in O / l), and V converted to fp16 when its tile is staged (exact for e4m3 rows).
 * The input domain stays that of bf16 operands: a 64-token tile of bf16 V rows that fp16 cannot hold (some
 * |v| >= 65536, or no element as large as 2^-9) makes the workgroup leave a marker in its first output element,
 * and a second launch inside this call recomputes exactly those row tiles with both products in bf16 (P as a
 * bf16 hi + lo pair).  So the call is two launches for bf16 rows and one for e4m3 rows; out is complete when
 * the call's work on the stream is.
 * Dh == 128, Hq % Hkv == 0.
 */
int tlf_varlen_prefill_attn(const void *q, int64_t q_stride,
                            const void *k, int64_t k_stride,
                            const void *v, int64_t v_stride, int32_t kv_dtype,
                            const float *k_scale, const float *v_scale,
                            const int32_t *cu_seqlens_q, const int32_t *cu_seqlens_k,
                            const int32_t *block_tables, int64_t block_table_stride,
                            void *out, int32_t num_seqs, int32_t max_seqlen_q,
                            int32_t num_q_heads, int32_t num_kv_heads, int32_t head_dim,
                            int32_t block_size, int64_t num_cache_blocks, float scale,
                            void *stream);

/* ---------------------------------------------------------------------------
 * K9  embedding row gather   replaces layers/embed_head.py:38 (F.embedding)
 *   y[i] = weight[ids[i]]   ids int64 [n], weight bf16 [vocab, cols], cols % 8 == 0.
 *   Rows with an id outside [0, vocab) are zero filled.
 */
int tlf_embedding(const int64_t *ids, const void *weight, void *y,
                  int32_t n, int32_t vocab, int32_t cols, void *stream);

/* ---------------------------------------------------------------------------
 * Bandwidth probes (no reference counterpart): plain streaming kernels that
 * bench.py uses to measure the HBM rate a read-only / copy kernel reaches on
 * the box and to scale the profiler's traffic counters.  bytes % 16 == 0,
 * 16-byte aligned pointers; sink is a 4-byte device word that is never
 * actually written for ordinary data.
 */
int tlf_probe_read(const void *src, size_t bytes, void *sink, void *stream);
int tlf_probe_copy(const void *src, void *dst, size_t bytes, void *stream);

/* Two more probes for the GEMM's rooflines (no reference counterpart).
 * tlf_probe_mfma: 512 workgroups x 4 waves each issue 16 * iters v_mfma_f32_32x32x16_bf16 from registers:
 *   2 * 32*32*16 * 16 * iters * 2048 flop per launch.  mode 0: small-integer operands, mode 1: pseudo-random
 *   bf16 values times int8-valued weights (the clock a kernel sees on real data); mode 2 / 3: the same two with
 *   idle cycles after every MFMA (a duty of about 0.9: how the clock answers to the load).  out: 512 * 256 floats.
 * tlf_probe_mix: 256 workgroups of 8 waves; waves 0..3 stream big (read once: floor(big_bytes / 16 MiB) * 16 KiB
 *   per wave, from HBM), waves 4..7 re-read small_region (L2 resident: at least 16 KiB, a multiple of 1 KiB)
 *   l2_eighths / 8 times as many bytes.  Shows what a CU's vector-memory path does with both at once. */
int tlf_probe_mfma(void *out, int32_t iters, int32_t mode, void *stream);
int tlf_probe_mix(const void *big, size_t big_bytes, const void *small_region, size_t small_bytes,
                  int32_t l2_eighths, void *sink, void *stream);

/* ===========================================================================
 * Mechanisms of hybrid (attention + recurrent) decoders.  No counterpart in the reference.  `dtype` is the
 * element type of activations, weights and caches (TLF_DT_BF16 or TLF_DT_F32); the residual stream, norms,
 * rotations, scores, attention weights, decays and recurrent states are fp32 in both.
 *
 * A step is a batch of sequences: sequence s owns the rows cu_seqlens_q[s] .. cu_seqlens_q[s + 1] - 1 of the step's
 * tensors and has seq_starts[s] tokens before them in the caches.
 *
 * Deferred projections.  tlf_gemm_deferred is tlf_w8a16_gemm (scale given) or tlf_bf16_gemm (scale NULL) without the
 * last step of a plan that splits K across workgroups: *splits (host memory, set before the call returns; it depends on
 * M, N and K only) says how many partial sums [splits, M, N] fp32 stand at the head of the workspace, 1: y is complete.
 * The entry points with the arguments (partials, splits, scale) read such a projection: with splits > 1 its value is
 * bf16(sum * scale), what the reduce kernel would store, and the row stride is N (bf16 only, partials 16-byte aligned,
 * the row pointer is not read); with splits <= 1 they read the rows.
 *
 * Grouped RMSNorm around an fp32 residual.  A row of `width` values is split into `groups` equal parts, each
 * divided by its own sqrt(mean(part^2) + eps); the whole is multiplied by a weight.
 *
 *   tlf_group_rmsnorm_add:    x += norm(y + y_bias) * w_post;  h = norm(x) * w_next
 *   tlf_embed_group_rmsnorm:  x  = table[id];                  h = norm(x) * (w_next + w_offset)
 *
 * x fp32 [rows, width] contiguous; y, h, table, weights: dtype; y_bias may be NULL; w_next NULL: no h.
 * width / groups <= 16384.  An id outside [0, vocab) embeds as zeros. */
int tlf_gemm_deferred(const void *x, int64_t x_stride, const void *w, const float *scale, void *y, int32_t M, int32_t N,
                      int32_t K, void *workspace, size_t workspace_bytes, int32_t *splits, void *stream);
int tlf_group_rmsnorm_add(const void *y, int64_t y_stride, const float *partials, int32_t splits, const float *scale,
                          const void *y_bias, const void *w_post, float *x, const void *w_next, void *h, int32_t rows, int32_t width, int32_t groups, float eps,
                          int32_t dtype, void *stream);
int tlf_embed_group_rmsnorm(const int64_t *ids, const void *table, int32_t vocab, float *x, const void *w_next,
                            float w_offset, void *h, int32_t rows, int32_t width, int32_t groups, float eps,
                            int32_t dtype, void *stream);

/* Dense operations of 32-bit mode (fp32 products and sums; any M, N, K): y = x . w^T, y = silu(x[:, :I]) * x[:, I:],
 * greedy argmax (first index among ties). */
int tlf_f32_gemm(const float *x, int64_t x_stride, const float *w, float *y, int32_t M, int32_t N, int32_t K,
                 void *stream);
int tlf_f32_silu_and_mul(const float *x, float *y, int32_t rows, int32_t inter, void *stream);
int tlf_f32_argmax(const float *logits, int64_t row_stride, int64_t *out, int32_t rows, int32_t vocab, void *stream);

/* Attention with unnormalised sigmoid weights over a sliding window and pooled blocks.
 *
 * Position i sees the tokens j with 0 <= i - j < window, and for every block b of `pool` tokens with
 * b * pool + pool - 1 <= i - window one key (the mean of the block's cached keys) and one value (the mean of its
 * values).  weight = sigmoid(q . k * scale + score_bias[head]);  out = sum(weight * value) * gate[row, head].
 *
 * Caches: k_cache / v_cache [num_pages, block_size, Hkv, Dp], pk_cache / pv_cache [num_pages, ceil(block_size / pool),
 * Hkv, Dp] with the same page numbers: block b is row b - (page * block_size) / pool of the page that holds its last
 * token (page = index in the sequence).  Dp = head_dim rounded up to a multiple of 32, pads are zeros.
 * block_size % 64 == 0, head_dim <= 256, rot_dims even.
 *
 * tlf_attn_prep: projection rows [q heads | k heads | one gate value per q head] -> biases (may be NULL) added;
 *   v row = the key so far; first rot_dims dimensions of q and k rotated pairwise (2 i, 2 i + 1) with
 *   cos_sin[pos] = cos of the rot_dims / 2 angles, then their sines (a position outside the table is not rotated);
 *   q and k divided by their root mean square; k / v rows stored at slot_mapping (negative: not stored),
 *   q_out [n, Hq, Dp], gate [n, Hq] = sigmoid, fp32.  Partial sums: head_dim and rot_dims multiples of 8 only.
 * tlf_pool_blocks: pooled rows of the blocks that sequences first_seq .. first_seq + num_seqs - 1 complete in this step
 *   (max_tokens: the most tokens one of them has in the step).
 * tlf_pooled_attn_rows: any rows; row_seq[r] is the block-table row (NULL: r).  slot_mapping[r] < 0: a padding row,
 *   out = 0.  pool_new: also write the pooled row of a block that a row's own token completes (decode).
 *   max_len bounds the positions.  out rows: Hq * head_dim values.
 * tlf_pooled_attn_prefill: bf16 matrix-core kernel for the portions of sequences first_seq .. + num_seqs - 1 (all other
 *   arguments as above; q, gate and out are indexed by the step's rows). */
int tlf_attn_prep(const void *proj, int64_t proj_stride, const float *partials, int32_t splits, const float *scale,
                  const void *q_bias, const void *k_bias,
                  const int64_t *positions, const float *cos_sin, int32_t max_pos, int32_t rot_dims,
                  const int32_t *slot_mapping, int64_t num_slots, void *q_out, void *k_cache, void *v_cache,
                  float *gate, int32_t n, int32_t num_q_heads, int32_t num_kv_heads, int32_t head_dim,
                  int32_t padded_dim, float eps, int32_t dtype, void *stream);
int tlf_pool_blocks(const void *k_cache, const void *v_cache, void *pk_cache, void *pv_cache,
                    const int32_t *block_tables, int64_t bt_stride, const int32_t *cu_seqlens_q,
                    const int32_t *seq_starts, int32_t first_seq, int32_t num_seqs, int32_t max_tokens,
                    int32_t num_kv_heads, int32_t head_dim, int32_t block_size, int32_t pool, int32_t window,
                    int64_t num_pages, int32_t dtype, void *stream);
size_t tlf_pooled_attn_rows_workspace_bytes(int32_t rows, int32_t num_q_heads, int32_t num_kv_heads, int32_t head_dim,
                                            int32_t pool, int32_t window, int32_t max_len);
int tlf_pooled_attn_rows(const void *q, const void *score_bias, const float *gate, const void *k_cache,
                         const void *v_cache, void *pk_cache, void *pv_cache, const int32_t *block_tables,
                         int64_t bt_stride, const int64_t *positions, const int32_t *slot_mapping,
                         const int32_t *row_seq, void *out, int64_t out_stride, int32_t rows, int32_t num_q_heads,
                         int32_t num_kv_heads, int32_t head_dim, int32_t block_size, int32_t pool, int32_t window,
                         int32_t max_len, int64_t num_pages, float scale, int32_t pool_new, int32_t dtype,
                         void *workspace, size_t workspace_bytes, void *stream);
int tlf_pooled_attn_prefill(const void *q, const void *score_bias, const float *gate, const void *k_cache,
                            const void *v_cache, const void *pk_cache, const void *pv_cache,
                            const int32_t *block_tables, int64_t bt_stride, const int32_t *cu_seqlens_q,
                            const int32_t *seq_starts, int32_t first_seq, int32_t num_seqs, int32_t max_tokens,
                            void *out, int64_t out_stride, int32_t num_q_heads, int32_t num_kv_heads, int32_t head_dim,
                            int32_t block_size, int32_t pool, int32_t window, int64_t num_pages, float scale,
                            void *stream);

/* Gated linear attention with a decay per key channel.  Projection rows are [q | k | v | g | r] (heads * key_dim twice,
 * heads * value_dim twice, rank values).  Per head, state S [key_dim, value_dim] fp32 at state[slot, head]:
 *   alpha = sigmoid(a2 . r + a2_bias)^(1 / tau);  S = diag(alpha) S + k v^T;  o = S^T (q * q_scale)
 *   out = o / sqrt(mean(o^2) + eps) * norm_weight * silu(g)
 * a2 [heads * key_dim, rank].  key_dim <= 256, value_dim <= 512, rank <= 256.
 *
 * tlf_gla_decode: one token per row; position 0 starts from a zero state, a slot outside [0, num_slots) is a padding
 *   row (out = 0).
 * tlf_gla_portions: sequences first_seq .. + num_seqs - 1 of the step (state_slots and seq_starts are indexed by the
 *   step's sequences, a start of 0 begins with a zero state).  Their tokens are cut into chunks of 16 that do not cross a
 *   sequence (a sequence's last chunk may be shorter) and follow each other: chunk c holds the chunk_lens[c] rows from chunk_rows[c] on, counted from the row `proj` and
 *   `out` point to; sequence first_seq + s owns the chunks cu_chunks[s] .. cu_chunks[s + 1] - 1.  `rows` rows in all. */
int tlf_gla_decode(const void *proj, int64_t proj_stride, const float *partials, int32_t splits,
                   const float *scale, const void *a2, const void *a2_bias,
                   const void *norm_weight, float *state, const int32_t *state_slots, int32_t num_slots,
                   const int64_t *positions, void *out, int64_t out_stride, int32_t rows, int32_t heads,
                   int32_t key_dim, int32_t value_dim, int32_t rank, float tau, float q_scale, float eps,
                   int32_t dtype, void *stream);
size_t tlf_gla_portions_workspace_bytes(int32_t rows, int32_t chunks, int32_t num_seqs, int32_t heads,
                                        int32_t key_dim, int32_t value_dim);
int tlf_gla_portions(const void *proj, int64_t proj_stride, const void *a2, const void *a2_bias,
                     const void *norm_weight, float *state, const int32_t *state_slots, int32_t num_slots,
                     const int32_t *seq_starts, const int32_t *chunk_rows, const int32_t *chunk_lens,
                     const int32_t *cu_chunks, int32_t chunks, int32_t first_seq, int32_t num_seqs, void *out,
                     int64_t out_stride, int32_t rows, int32_t heads, int32_t key_dim, int32_t value_dim,
                     int32_t rank, float tau, float q_scale, float eps, int32_t dtype, void *workspace,
                     size_t workspace_bytes, void *stream);

/* Residual add with a multiplier and the next RMSNorm, for layers whose sublayers share one norm:
 *   x += mult * (y + sum_k extra[extra_rows[row * top + k]], k < top);   h = x / rms(x) * (w_next + w_offset)
 * (w_offset 1: a weight stored around zero; w_next NULL: no h.  y may be partial sums as above.) */
int tlf_residual_rmsnorm(const void *y, int64_t y_stride, const float *partials, int32_t splits, const float *scale,
                         const void *extra, int64_t extra_stride, const int32_t *extra_rows, int32_t top, float mult,
                         float *x, const void *w_next, float w_offset, void *h, int32_t rows, int32_t width, float
                         eps, int32_t dtype, void *stream);

/* Latent attention: per token one cache row [latent: Ra | rotated key: Ta | 0] of Lp values for all heads, Ra and Ta being
 * rank and rot_dim rounded up to 8 and Lp their sum rounded up to 64; head h's key is [Uk_h c | rotated part], its value
 * Uv_h c.  Softmax over the `window` keys up to a position.  Query rows: [own part: Da | rotated: Ta | 0] of Dq values, Da =
 * dim rounded up to 8, Dq the sum rounded up to 32.  rank <= 1536, dim, rot_dim, vdim <= 1024, Lp <= 2048.
 *
 * tlf_latent_prep: projection rows [q: heads * (dim + rot_dim), own part first in a head | ... | latent at latent_col: rank |
 *   rot_dim] -> q_out [n, heads, Dq] with the rotated part turned pairwise (2 i, 2 i + 1) by cos_sin[pos] (cos of the pairs,
 *   then sin; with `halves` pairs (i, i + rot_dim / 2)), latent / rms * norm_weight and the turned key into the cache row
 *   slot_mapping[token] (negative: not stored).  q_out or cache NULL: without the queries or the latents (latent_col then counts
 *   from the row's first column, queries may lie in another tensor).  cq_norm: the cq_rank columns from cq_col on, / rms * cq_norm,
 *   to cq_out [n, cq_stride] (zeros behind).  gate_out [n, heads] (with cache): sigmoid of the columns from gate_col on.
 * tlf_head_gemm: y[row, head] = W[head] x[row, head], W [heads, N, K]; N a multiple of 16, K of 32.  In rows below n_main
 *   only the first k_main columns hold weights (n_main 0: all).
 * tlf_latent_rows: absorbed attention, any rows in either dtype: q [rows, heads, Lp] = [Uk_h^T q_own | q_rot | 0]; writes
 *   part [rows, heads, Rp] (Rp = Ra rounded up to 32), the unnormalised mix of latents, and ml [rows, heads, 2], maximum
 *   (of score * log2 e) and denominator.  row_seq[r]: block-table row (NULL: r).
 * tlf_latent_attn: the same on the matrix cores, bf16, Lp <= 576 (tlf_latent_attn_supported).  With cu_seqlens_q NULL
 *   sequence s is the single row s at positions[s] (slot_mapping[s] < 0: a padding row, no keys; max_tokens 1), otherwise
 *   rows cu_seqlens_q[s] - first_row .. of q, sequences first_seq .. + num_seqs - 1 of at most max_tokens rows, after
 *   seq_starts[s] cached tokens.  The work is cut into pieces by a plan (tlf_latent_attn_plan, once per step and window:
 *   the same arguments, row_size = Lp; it depends on no layer), written to part [pieces, units, Rp] and ml [pieces, units,
 *   2].  tlf_latent_attn_layout gives (host memory) layout[3] = int32 values of a plan, pieces, units.
 * tlf_latent_values: out[row, head] = Uv_h (sum of the pieces / denominator); uv [heads, vdim rounded up to 16, Rp]; plan
 *   NULL: part as from tlf_latent_rows, otherwise the plan and its arguments (with cu_seqlens_q, row_seq[r] is the sequence
 *   of row r of `out`).  gate [rows, heads] (NULL: none) multiplies a head's result.  Rows without keys give 0.
 * tlf_latent_gather: for the expanded form: cache rows of the keys that sequence first_seq + s sees in this step (from
 *   position max(0, start - window + 1) on) as rows kv_offsets[s] .. kv_offsets[s + 1] - 1 of `out`; max_rows bounds them.
 * tlf_latent_prefill: portions from expanded keys and values (rows [heads * Da | heads * Va], Va = vdim rounded up to 8) and
 *   the gathered rows; gate as above, by the step's rows; bf16, Dq <= 256, vdim <= 128 (tlf_latent_prefill_supported). */
int tlf_latent_prep(const void *proj, int64_t proj_stride, const float *partials, int32_t splits, const float *scale,
                    int32_t latent_col, const void *norm_weight, const int64_t *positions, const float *cos_sin,
                    int32_t max_pos, int32_t halves, const int32_t *slot_mapping, int64_t num_slots, void *q_out, void *cache,
                    int32_t cq_col, int32_t cq_rank, const void *cq_norm, void *cq_out, int32_t cq_stride,
                    int32_t gate_col, float *gate_out, int32_t n, int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim, float eps,
                    int32_t dtype, void *stream);
int tlf_head_gemm(const void *x, const void *w, void *y, int32_t rows, int32_t heads, int32_t N, int32_t K, int32_t
                  n_main, int32_t k_main, int32_t dtype, void *stream);
int tlf_latent_rows(const void *q, const void *cache, const int32_t *block_tables, int64_t bt_stride, const int64_t
                    *positions, const int32_t *slot_mapping, const int32_t *row_seq, float *part, float *ml, int32_t
                    rows, int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim, int32_t
                    block_size, int32_t window, int64_t num_pages, float scale, int32_t dtype, void *stream);
int tlf_latent_attn_layout(int32_t num_seqs, int32_t max_tokens, int32_t heads, int32_t row_size, int32_t *layout);
int tlf_latent_attn_plan(const int64_t *positions, const int32_t *slot_mapping, const int32_t *cu_seqlens_q, const
                         int32_t *seq_starts, int32_t first_seq, int32_t first_row, int32_t num_seqs, int32_t
                         max_tokens, int32_t heads, int32_t row_size, int32_t window, int32_t *plan, void *stream);
int tlf_latent_attn(const void *q, const void *cache, const int32_t *block_tables, int64_t bt_stride, const int64_t
                    *positions, const int32_t *slot_mapping, const int32_t *cu_seqlens_q, const int32_t *seq_starts,
                    int32_t first_seq, int32_t first_row, int32_t num_seqs, int32_t max_tokens, const int32_t *plan,
                    float *part, float *ml, int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim,
                    int32_t block_size, int32_t window, int64_t num_pages, float scale, void *stream);
int tlf_latent_values(const float *part, const float *ml, const int32_t *plan, const int32_t *cu_seqlens_q, const
                      int32_t *row_seq, int32_t first_seq, int32_t first_row, int32_t num_seqs, int32_t max_tokens,
                      const void *uv, const float *gate, void *out, int64_t out_stride, int32_t rows, int32_t heads, int32_t dim,
                      int32_t rot_dim, int32_t rank, int32_t vdim, int32_t dtype, void *stream);
int tlf_latent_attn_supported(int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim);
int tlf_latent_gather(const void *cache, const int32_t *block_tables, int64_t bt_stride, const int32_t *cu_seqlens_q,
                      const int32_t *seq_starts, const int32_t *kv_offsets, int32_t first_seq, int32_t num_seqs,
                      int32_t max_rows, void *out, int32_t row_size, int32_t block_size, int32_t window, int64_t
                      num_pages, void *stream);
int tlf_latent_prefill_supported(int32_t heads, int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim);
int tlf_latent_prefill(const void *q, const void *expanded, int64_t expanded_stride, const void *latents, const
                       int32_t *cu_seqlens_q, const int32_t *seq_starts, const int32_t *kv_offsets, int32_t
                       first_seq, int32_t num_seqs, int32_t max_tokens, const float *gate, void *out, int64_t out_stride, int32_t heads,
                       int32_t dim, int32_t rot_dim, int32_t rank, int32_t vdim, int32_t window, float scale, void
                       *stream);

/* Mixture of experts.  Rows (token, k) are put in expert order; nothing on the host depends on the routing.
 *
 * tlf_gemm_f32_sums: y = x . w^T with bf16 factors as fp32 sums [*splits, M, N] to be added up (*splits in host memory);
 *   for the router's logits, N = experts rounded up to 16.
 * tlf_moe_group: from the logits' sums (experts + identity of them), with correction NULL ids[token, k] the `top` largest
 *   (ties: the smaller index) and weights[token, k] = sigmoid; otherwise the `top` largest of softmax + correction (of `dtype`)
 *   and weights = softmax values, normalised to a sum of 1.  Experts from `experts` on have no rows: row_of = -1; row_of[token * top + k] = the entry's row in expert order, src[row] its token, row_weight[row] its weight;
 *   tiles (int32 x 4: expert, first row, rows, 0) cut the rows into at most tile_rows of one expert each, *num_tiles <=
 *   max_tiles of them; max_tiles >= n * top / tile_rows + min(experts, n * top).  experts + identity <= 512.
 * tlf_moe_gemm: y[row] = W[expert] x[x_rows ? x_rows[row] : row]; w [experts, N, K].  act 1 and 2: channels are interleaved
 *   as for the SiLU-and-mul products (8 gate, then the 8 matching up), y [rows, N / 2]; act 1, clipped GLU: with f =
 *   row_scale[row] (NULL: 1), g = min(f gate, limit), u = clamp(f up, +-limit): y = g sigmoid(1.702 g) (u + 1); act 2: y =
 *   silu(gate) up in fp32.  bf16: tile_rows 32, 64, 128 or 256, K a
 *   multiple of 64; fp32: tile_rows 64.  x_count bounds the x rows.
 * tlf_xielu: with a = softplus(pq[0]), b = 1/2 + softplus(pq[1]), out = a z^2 + z / 2 for z > 0, b (e^z - 1 - z) + z / 2
 *   otherwise, z = columns col .. col + cols - 1 of x (or of partial sums); columns cols .. padded_cols - 1 become 0.
 * tlf_bf16_gemm_xielu: y = x . w^T with that activation on the columns from act_col on (a multiple of 8), which go to `out`
 *   (its columns 0 .. out_cols - 1, as far as N reaches) instead of y; for many rows. */
size_t tlf_gemm_f32_sums_bytes(int32_t M, int32_t N, int32_t K);
int tlf_gemm_f32_sums(const void *x, int64_t x_stride, const void *w, float *sums, size_t sums_bytes, int32_t M,
                      int32_t N, int32_t K, int32_t *splits, void *stream);
size_t tlf_moe_group_workspace_bytes(int32_t n, int32_t top, int32_t experts);
int tlf_moe_group(const float *sums, int32_t splits, int32_t *ids, float *weights, int32_t *row_of, int32_t *src,
                  float *row_weight, int32_t *tiles, int32_t *num_tiles, int32_t max_tiles, int32_t n, int32_t top,
                  int32_t experts, int32_t identity, const void *correction, int32_t dtype, int32_t tile_rows,
                  void *workspace, size_t workspace_bytes, void *stream);
int tlf_moe_gemm(const void *x, int64_t x_stride, int32_t x_count, const void *w, void *y, const int32_t *tiles,
                 const int32_t *num_tiles, int32_t max_tiles, int32_t tile_rows, const int32_t *x_rows, const float
                 *row_scale, int32_t rows, int32_t N, int32_t K, int32_t act, float limit, int32_t dtype,
                 void *stream);
int tlf_bf16_gemm_xielu(const void *x, int64_t x_stride, const void *w, void *y, int32_t M, int32_t N, int32_t K,
                        int32_t act_col, const void *pq, void *out, int64_t out_stride, int32_t out_cols, void
                        *stream);
int tlf_xielu(const void *x, int64_t x_stride, const float *partials, int32_t splits, const float *scale, int32_t
              col, const void *pq, void *out, int64_t out_stride, int32_t rows, int32_t cols, int32_t padded_cols,
              int32_t dtype, void *stream);

/* Layer norm around an fp32 residual stream: with t = x[row] after the step, h = ((t - mean) / sqrt(variance + eps) * w_next +
 * b_next) * out_scale, the variance being the mean of the squared deviations.
 *
 * tlf_embed_layernorm: x = table[id].
 * tlf_residual_layernorm: x += y (NULL and splits <= 1: none; or its partial sums) + the sum over k < top of extra_weights[row,
 *   k] (NULL: 1) times extra[extra_rows[row, k]], a negative index standing for self[row]. */
int tlf_embed_layernorm(const int64_t *ids, const void *table, int32_t vocab, float *x, const void *w_next, const void
                        *b_next, float out_scale, void *h, int32_t rows, int32_t width, float eps, int32_t dtype,
                        void *stream);
int tlf_residual_layernorm(const void *y, int64_t y_stride, const float *partials, int32_t splits, const float *scale,
                           const void *extra, int64_t extra_stride, const int32_t *extra_rows, const float
                           *extra_weights, int32_t top, const void *self, int64_t self_stride, float *x, const void
                           *w_next, const void *b_next, float out_scale, void *h, int32_t rows, int32_t width, float
                           eps, int32_t dtype, void *stream);

/* Causal grouped-query attention with a sink, a score cap and an output gate on paged, head-major caches k_cache [pages,
 * kv_heads, block, Dp], v_cache [pages, kv_heads, block, Vp] (Dp, Vp: dim and vdim rounded up to 32, pads are zeros).
 *   score = scale (q . k), cap > 0: cap tanh(score / cap);  out = sigmoid(gate) * sum exp(score) v / (sum exp(score) + exp(sink))
 * sink [heads] and gate [rows, heads * vdim] may be NULL (no such term).  dim, vdim <= 512, block a multiple of 64.
 *
 * tlf_sink_prep: projection rows [q: heads * dim | k: kv_heads * dim | v: kv_heads * vdim | gate: heads * vdim] -> + bias (NULL:
 *   none; of the channels of q, k and v) -> with conv [taps, channels] y_p = sum_j conv[j] u_(p - taps + 1 + j), zeros before the
 *   sequence -> q, k / rms over the head * q_norm / k_norm (NULL: 1) -> q times q_mult[pos] (NULL: 1) -> the first rot_dims
 *   dimensions of q and k turned by cos_sin[pos] (cos of the pairs, then sin), i with i + rot_dims / 2 -> q times score_scale
 *   log2(e), with a cap also times 2 / cap (what the kernels below expect in q) -> q_out [n, heads, Dp]
 *   and the cache rows slot_mapping[token] (negative: not stored).  ring [state slots, taps, channels] holds the projected rows
 *   (without bias) of a sequence's last positions, p in row p mod taps: rows of one-token sequences (row_seq NULL, or
 *   cu_seqlens_q of row_seq[row]) are written here, those of portions by tlf_conv_tail afterwards.  gate_out [n, heads * vdim]
 *   (NULL: not copied) gets the gate's columns; with splits > 1 it must be there and row_seq NULL.
 * tlf_conv_tail: last taps - 1 projected rows of sequences first_seq .. (proj: the step's rows) into the ring.
 * tlf_sink_attn_rows: row r of q [rows, heads, Dp] attends to positions 0 .. positions[r] of sequence row_seq[r] (NULL: r);
 *   slot_mapping[r] < 0: a padding row (zeros).  max_len bounds the positions.  bf16 up to 256 dimensions on the matrix cores.
 * tlf_sink_attn_prefill: portions of sequences first_seq .., rows as in the step; bf16, dim, vdim <= 256. */
int tlf_sink_prep(const void *proj, int64_t proj_stride, const float *partials, int32_t splits, const float *scale,
                  const void *bias, const void *conv, int32_t taps, void *ring, const int32_t *state_slots, int64_t
                  num_state_slots, const int32_t *row_seq, const int32_t *cu_seqlens_q, const void *q_norm, const void
                  *k_norm, const int64_t *positions, const float *cos_sin, const float *q_mult, int32_t max_pos,
                  int32_t rot_dims, const int32_t *slot_mapping, void *q_out, void *k_cache, void *v_cache, void
                  *gate_out, int32_t n, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t
                  block_size, int64_t num_pages, float eps, float score_scale, float cap, int32_t dtype, void
                  *stream);
int tlf_conv_tail(const void *proj, int64_t proj_stride, void *ring, const int32_t *state_slots, int64_t
                  num_state_slots, const int32_t *cu_seqlens_q, const int32_t *seq_starts, int32_t first_seq, int32_t
                  num_seqs, int32_t taps, int32_t channels, int32_t dtype, void *stream);
size_t tlf_sink_attn_rows_workspace_bytes(int32_t rows, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim,
                                          int32_t max_len, int32_t dtype);
int tlf_sink_attn_rows(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables, int64_t
                       bt_stride, const int64_t *positions, const int32_t *slot_mapping, const int32_t *row_seq, const
                       void *sink, const void *gate, int64_t gate_stride, void *out, int64_t out_stride, int32_t rows,
                       int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size, int32_t
                       max_len, int64_t num_pages, float cap, int32_t dtype, void *workspace, size_t workspace_bytes, void *stream);
int tlf_sink_attn_prefill_supported(int32_t dim, int32_t vdim);
int tlf_sink_attn_prefill(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables, int64_t
                          bt_stride, const int32_t *cu_seqlens_q, const int32_t *seq_starts, int32_t first_seq,
                          int32_t num_seqs, int32_t max_tokens, const void *sink, const void *gate, int64_t
                          gate_stride, void *out, int64_t out_stride, int32_t heads, int32_t kv_heads, int32_t dim,
                          int32_t vdim, int32_t block_size, int64_t num_pages, float cap, void *stream);

/* Norm behind the sum, with what follows it:
 *   x_out = rms_norm(alpha * x + layer_scale * y) * w   (tlf_post_rmsnorm; y or its partial sums as above)
 *   x_out = embed_scale * table[id]                      (tlf_embed_shift; an id outside [0, vocab) embeds as zeros)
 *   h = x_out, or with w_next (no mix) rms_norm(x_out) * w_next, or with mix  v + (v_before - v) * mix  for v = x_out's row and v_before
 *       the row of the token before (zeros at position 0)
 * x, x_out fp32 [rows, width]; h, table, weights: dtype; h may be NULL without mix and w_next.  ring fp32 [num_slots, 2, width] holds the
 * rows before, position p in row p mod 2: a sequence's first row of the step reads it, single rows write it (portions:
 * tlf_conv_tail with taps 2 on x_out).  row_seq NULL: row r is the one row of sequence r; otherwise rows cu_seqlens_q[s] .. belong to
 * sequence s and x_out must not be x.  A state slot outside [0, num_slots) reads zeros and is not written.  width <= 16384.
 * tlf_rows_rmsnorm: rows of x in `groups` equal parts, each / its rms, * w, to out [rows, out_stride] (zeros from cols on). */
int tlf_post_rmsnorm(const void *y, int64_t y_stride, const float *partials, int32_t splits, const float *scale, const void
                     *layer_scale, float alpha, const float *x, const void *w, float eps, float *x_out, const void *mix,
                     float *ring, int64_t num_slots, const int32_t *state_slots, const int32_t *row_seq, const int32_t
                     *cu_seqlens_q, const int64_t *positions, const void *w_next, void *h, int32_t rows, int32_t width,
                     int32_t dtype, void *stream);
int tlf_embed_shift(const int64_t *ids, const void *table, int32_t vocab, float embed_scale, float *x_out, const void *mix,
                    float *ring, int64_t num_slots, const int32_t *state_slots, const int32_t *row_seq, const int32_t
                    *cu_seqlens_q, const int64_t *positions, void *h, int32_t rows, int32_t width, int32_t dtype, void
                    *stream);
int tlf_rows_rmsnorm(const void *x, int64_t x_stride, const void *w, void *out, int64_t out_stride, int32_t rows, int32_t
                     cols, int32_t groups, float eps, int32_t dtype, void *stream);

/* Causal grouped-query attention whose heads mix their weights after the softmax, on the caches of the sink attention:
 *   w_h = softmax(score_scale temp_h (q_h . k));  out_h = sum_j (sum_g talk[h, g] w_g(j)) v(j) of head h's KV head
 *
 * tlf_talk_prep: projection rows [q: heads * dim | k: kv_heads * dim | v: kv_heads * vdim] -> q and k / rms over all of q, all of k
 *   * q_norm, k_norm -> the first rot_dims dimensions of every head turned pairwise (2 i, 2 i + 1) by cos_sin[pos] (cos of the pairs,
 *   then sin) -> q times temp[head] (NULL: 1) score_scale log2(e) -> q_out [n, heads, Dp] and the cache rows
 *   slot_mapping[token] (negative: not stored).  heads * Dp <= 32768.
 * tlf_talk_attn_rows: row r of q attends to positions 0 .. positions[r] of sequence row_seq[r] (NULL: r); slot_mapping[r] < 0: a
 *   padding row (zeros).  max_len bounds the positions.  talk [heads, heads].  heads <= 1024; bf16 up to 128 heads and 256
 *   dimensions on the matrix cores.  The workspace holds the scores (4 bytes per row, head and key).
 * tlf_talk_attn_prefill: portions of sequences first_seq .., rows as in the step; bf16, heads <= 32, dim, vdim <= 128 and a limit
 *   on kv_heads * vdim (tlf_talk_attn_prefill_supported).  stats: scratch, [rows of the step, heads]. */
int tlf_talk_prep(const void *proj, int64_t proj_stride, const float *partials, int32_t splits, const float *scale, const void
                  *q_norm, const void *k_norm, const void *temp, const int64_t *positions, const float *cos_sin, int32_t
                  max_pos, int32_t rot_dims, const int32_t *slot_mapping, void *q_out, void *k_cache, void *v_cache,
                  int32_t n, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size, int64_t
                  num_pages, float eps, float score_scale, int32_t dtype, void *stream);
size_t tlf_talk_attn_rows_workspace_bytes(int32_t rows, int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim,
                                          int32_t max_len, int32_t dtype);
int tlf_talk_attn_rows(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables, int64_t
                       bt_stride, const int64_t *positions, const int32_t *slot_mapping, const int32_t *row_seq, const
                       void *talk, void *out, int64_t out_stride, int32_t rows, int32_t heads, int32_t kv_heads, int32_t
                       dim, int32_t vdim, int32_t block_size, int32_t max_len, int64_t num_pages, int32_t dtype, void
                       *workspace, size_t workspace_bytes, void *stream);
int tlf_talk_attn_prefill_supported(int32_t heads, int32_t kv_heads, int32_t dim, int32_t vdim);
int tlf_talk_attn_prefill(const void *q, const void *k_cache, const void *v_cache, const int32_t *block_tables, int64_t
                          bt_stride, const int32_t *cu_seqlens_q, const int32_t *seq_starts, int32_t first_seq, int32_t
                          num_seqs, int32_t max_tokens, const void *talk, float *stats, void *out, int64_t out_stride, int32_t heads,
                          int32_t kv_heads, int32_t dim, int32_t vdim, int32_t block_size, int64_t num_pages, void
                          *stream);

/* State-space layer with a scalar decay per head (Mamba-2).  Projection rows [z: inner | x: inner | B: groups * state_dim | C: groups *
 * state_dim | dt: heads], inner = heads * vdim; head h uses group h / (heads / groups).
 *   [x | B | C] = silu(conv_bias + sum_j conv[j] u_(p - taps + 1 + j)), zeros before the sequence;  dt = softplus(dt + dt_bias)
 *   S = exp(-exp(A_log) dt) S + dt B x^T;  out = (S^T C + D x) * silu(z)          state fp32 [slots, heads, state_dim, vdim]
 * conv [taps, channels of x, B, C]; ring [slots, taps, channels]: projected rows of a sequence's last positions, p in row p mod taps.
 * Position 0 starts from a zero state.  state_dim, vdim <= 512.
 *
 * tlf_ssd_decode: one token per row, ring and state updated; a slot outside [0, num_slots) is a padding row (out = 0).
 * tlf_ssd_portions: sequences first_seq .. + num_seqs - 1 of at most max_tokens rows, whose rows are the last `rows` of the step,
 *   from first_row on (positions, row_seq, cu_seqlens_q, proj, out: of the whole step).  The ring is read, not written
 *   (tlf_conv_tail).  bf16 with state_dim <= 256 on the matrix cores, otherwise token by token. */
int tlf_ssd_decode(const void *proj, int64_t proj_stride, const float *partials, int32_t splits, const float *scale, const
                   void *conv, const void *conv_bias, int32_t taps, const void *dt_bias, const void *A_log, const void *D,
                   void *ring, float *state, const int32_t *state_slots, int32_t num_slots, const int64_t *positions, void
                   *out, int64_t out_stride, int32_t rows, int32_t heads, int32_t vdim, int32_t state_dim, int32_t groups,
                   int32_t dtype, void *stream);
size_t tlf_ssd_portions_workspace_bytes(int32_t rows, int32_t num_seqs, int32_t max_tokens, int32_t heads, int32_t vdim,
                                        int32_t state_dim, int32_t groups, int32_t dtype);
int tlf_ssd_portions(const void *proj, int64_t proj_stride, const void *conv, const void *conv_bias, int32_t taps, const void
                     *dt_bias, const void *A_log, const void *D, void *ring, float *state, const int32_t *state_slots,
                     int32_t num_slots, const int64_t *positions, const int32_t *row_seq, const int32_t *cu_seqlens_q,
                     const int32_t *seq_starts, int32_t first_seq, int32_t num_seqs, int32_t first_row, int32_t max_tokens,
                     void *out, int64_t out_stride, int32_t rows, int32_t heads, int32_t vdim, int32_t state_dim, int32_t
                     groups, int32_t dtype, void *workspace, size_t workspace_bytes, void *stream);

#ifdef __cplusplus
}
#endif
#endif /* TLF_HIP_H */
