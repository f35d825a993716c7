"""Sigmoid attention over a sliding window and pooled blocks, on paged caches.

Position ``i`` sees the ``window`` tokens up to itself and one mean key / value per block of ``pool`` tokens that lies
wholly before them.  The layer owns two paged caches with common page numbers: token rows and block means."""
import torch
from torch import nn

from .. import ops
from ..utils.context import get_context


class PooledWindowAttention(nn.Module):
    def __init__(self, num_heads: int, num_kv_heads: int, head_dim: int, scale: float, window: int, pool: int,
                 rot_dims: int, rope: torch.Tensor, eps: float, dtype: torch.dtype):
        super().__init__()
        self.num_heads, self.num_kv_heads, self.head_dim = num_heads, num_kv_heads, head_dim
        self.scale, self.window, self.pool, self.rot_dims, self.eps = scale, window, pool, rot_dims, eps
        self.dtype = dtype
        self.register_buffer("cos_sin", rope, persistent=False)
        self.score_bias = nn.Parameter(torch.zeros(num_heads))
        self.takes_partials = head_dim % 8 == 0 and rot_dims % 8 == 0    # the preparation may add up split projections
        self.kv = None                      # ops.PooledKV, bound by the model runner

    # -- what the model runner asks a layer with a paged cache
    def page_bytes(self, block_size: int) -> int:
        return ops.PooledKV.page_bytes(block_size, self.num_kv_heads, self.head_dim, self.pool,
                                       torch.empty(0, dtype=self.dtype).element_size())

    def bind_pages(self, pages: int, block_size: int, device):
        self.kv = ops.PooledKV(pages, block_size, self.num_kv_heads, self.head_dim, self.pool, self.window,
                               self.dtype, device) if pages else None

    def forward(self, proj: torch.Tensor, q_bias, k_bias, positions: torch.Tensor) -> torch.Tensor:
        """``proj``: rows ``[q | k | gate]`` -> ``[N, heads * head_dim]``, gated."""
        ctx, kv = get_context(), self.kv
        q, gate = ops.attn_prep(proj, q_bias, k_bias, positions, self.cos_sin, self.rot_dims, ctx.slot_mapping, kv.k,
                                kv.v, self.num_heads, self.head_dim, self.eps)
        n = proj.shape[0]
        out = torch.empty(n, self.num_heads * self.head_dim, dtype=proj.dtype, device=proj.device)
        single = ctx.num_single
        bias = self.score_bias.data
        if single:
            ops.pooled_attention_rows(q[:single], bias, gate[:single], kv, ctx.block_tables, positions[:single],
                                      ctx.slot_mapping[:single], self.scale, ctx.max_len, out[:single], pool_new=True)
        if single < n:
            portions = ctx.cu_seqlens_q.numel() - 1 - single
            ops.pool_blocks(kv, ctx.block_tables, ctx.cu_seqlens_q, ctx.seq_starts, single, portions, ctx.max_portion)
            if proj.dtype == torch.bfloat16:
                ops.pooled_attention_prefill(q, bias, gate, kv, ctx.block_tables, ctx.cu_seqlens_q, ctx.seq_starts,
                                             single, portions, ctx.max_portion, self.scale, out)
            else:
                ops.pooled_attention_rows(q[single:], bias, gate[single:], kv, ctx.block_tables, positions[single:],
                                          ctx.slot_mapping[single:], self.scale, ctx.max_len, out[single:],
                                          row_seq=ctx.row_seq[single:])
        return out
