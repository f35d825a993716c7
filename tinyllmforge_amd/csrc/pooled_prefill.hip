#include "pooled_attn.h"
extern "C" int tlf_pooled_attn_prefill(const void *q, const void *score_bias, const float *gate, const void *k_cache,
                            const void *v_cache, const void *pk_cache, const void *pv_cache,
                            const int32_t *block_tables, int64_t bt_stride, const int32_t *cu_seqlens_q,
                            const int32_t *seq_starts, int32_t first_seq, int32_t num_seqs, int32_t max_tokens,
                            void *out, int64_t out_stride, int32_t num_q_heads, int32_t num_kv_heads, int32_t head_dim,
                            int32_t block_size, int32_t pool, int32_t window, int64_t num_pages, float scale,
                            void *stream) { return TLF_E_UNSUPPORTED; }
