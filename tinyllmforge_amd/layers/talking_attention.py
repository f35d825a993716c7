"""Causal grouped-query attention whose heads mix their weights after the softmax, on paged head-major caches.

In front of it: RMS norm over the whole query and the whole key projection, rotation of neighbouring dimensions, a temperature
per head."""
import torch
from torch import nn

from .. import ops
from ..utils.context import get_context


class TalkingHeadsAttention(nn.Module):
    def __init__(self, num_heads: int, num_kv_heads: int, dim: int, value_dim: int, scale: float, eps: float, dtype: torch.dtype,
                 rot_dims: int = 0, rope=None):
        super().__init__()
        self.num_heads, self.num_kv_heads, self.dim, self.value_dim = num_heads, num_kv_heads, dim, value_dim
        self.scale, self.eps, self.dtype, self.rot_dims = scale, eps, dtype, rot_dims
        self.register_buffer("cos_sin", rope, persistent=False)
        self.parts = {"q": num_heads * dim, "k": num_kv_heads * dim, "v": num_kv_heads * value_dim}
        self.q_norm, self.k_norm = nn.Module(), nn.Module()
        self.q_norm.weight, self.k_norm.weight = nn.Parameter(torch.ones(self.parts["q"])), nn.Parameter(torch.ones(self.parts["k"]))
        self.temp = nn.Parameter(torch.ones(num_heads))
        self.talk = nn.Parameter(torch.eye(num_heads))
        self.kv = None                      # ops.SinkKV, bound by the model runner

    # -- what the model runner asks a layer with a paged cache
    def page_bytes(self, block_size: int) -> int:
        return ops.SinkKV.page_bytes(block_size, self.num_kv_heads, self.dim, self.value_dim, self.dtype.itemsize)

    def bind_pages(self, pages: int, block_size: int, device):
        self.kv = ops.SinkKV(pages, block_size, self.num_kv_heads, self.dim, self.value_dim, self.dtype, device) if pages else None

    def forward(self, proj, positions: torch.Tensor) -> torch.Tensor:
        """``proj``: rows ``[q | k | v]`` -> ``[N, heads * value_dim]``."""
        ctx, kv, n = get_context(), self.kv, proj.shape[0]
        q = ops.talk_prep(proj, kv, self.num_heads, positions, ctx.slot_mapping, self.q_norm.weight.data, self.k_norm.weight.data,
                          self.temp.data, self.cos_sin, self.rot_dims, self.eps, self.scale)
        out = torch.empty(n, self.num_heads * self.value_dim, dtype=self.dtype, device=q.device)
        tiles = self.dtype == torch.bfloat16 and ops.talk_prefill_supported(self.num_heads, self.num_kv_heads, self.dim, self.value_dim)
        rows = ctx.num_short_rows if tiles else n
        if rows:
            ops.talk_attention_rows(q[:rows], kv, ctx.block_tables, positions[:rows], ctx.slot_mapping[:rows], self.talk.data, ctx.max_len,
                                    out[:rows], ctx.row_seq[:rows] if ctx.num_single < rows else None)
        if rows < n:
            first = ctx.num_single + ctx.num_short
            ops.talk_attention_prefill(q, kv, ctx.block_tables, ctx.cu_seqlens_q, ctx.seq_starts, first,
                                       ctx.cu_seqlens_q.numel() - 1 - first, ctx.max_portion, self.talk.data, out)
        return out
