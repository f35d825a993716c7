"""Gated linear attention with a decay per key channel: an fp32 state per sequence and head instead of a KV cache."""
import torch
from torch import nn

from .. import ops
from ..utils.context import get_context


class GatedLinearAttention(nn.Module):
    def __init__(self, num_heads: int, key_dim: int, value_dim: int, rank: int, tau: float, eps: float):
        super().__init__()
        self.num_heads, self.key_dim, self.value_dim = num_heads, key_dim, value_dim
        self.tau, self.eps = tau, eps
        self.decay_weight = nn.Parameter(torch.zeros(num_heads * key_dim, rank))
        self.decay_bias = nn.Parameter(torch.zeros(num_heads * key_dim))
        self.norm = nn.Module()
        self.norm.weight = nn.Parameter(torch.ones(value_dim))
        self.state = None                   # fp32 [slots, heads, key_dim, value_dim], bound by the model runner

    # -- what the model runner asks a layer with a recurrent state
    def slot_bytes(self) -> int:
        return 4 * self.num_heads * self.key_dim * self.value_dim

    def bind_slots(self, slots: int, device):
        self.state = torch.zeros(slots, self.num_heads, self.key_dim, self.value_dim, dtype=torch.float32,
                                 device=device) if slots else None

    def forward(self, proj: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """``proj``: rows ``[q | k | v | g | r]`` -> ``[N, heads * value_dim]``, normed and gated."""
        ctx = get_context()
        n = proj.shape[0]
        out = torch.empty(n, self.num_heads * self.value_dim, dtype=proj.dtype, device=proj.device)
        single = ctx.num_single
        weights = (self.decay_weight.data, self.decay_bias.data, self.norm.weight.data)
        if single:
            ops.gla_decode(proj if single == n else proj[:single], *weights, self.state, ctx.state_slots, positions[:single], self.tau, self.eps,
                           out[:single])
        if single < n:
            ops.gla_portions(proj[single:], *weights, self.state, ctx.state_slots, ctx.seq_starts, ctx.chunk_rows,
                             ctx.chunk_lens, ctx.cu_chunks, single, ctx.cu_chunks.numel() - 1, self.tau, self.eps,
                             out[single:])
        return out
