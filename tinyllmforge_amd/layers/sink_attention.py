"""Causal grouped-query attention with a learned sink, an optional score cap and an elementwise output gate, on paged
head-major caches.

In front of it, each where the layer has it: biases, a short causal convolution over time per channel of q, k and v, RMS norm
per head of q and k, a temperature per position on q, rotation in halves.  A layer that runs several times in a row has caches
and convolution states of its own for every run."""
import math

import torch
from torch import nn

from .. import ops
from ..utils.context import get_context


def query_temperatures(coef: float, every: float, max_position: int) -> torch.Tensor:
    """fp32 ``[max_position]``: ``1 + coef ln(floor((p + 1) / every) + 1)``; double precision, CPU."""
    steps = torch.tensor([math.floor((p + 1) / every) for p in range(max_position)], dtype=torch.float64, device="cpu")
    return (1 + coef * torch.log(steps + 1)).float()


class SinkAttention(nn.Module):
    def __init__(self, num_heads: int, num_kv_heads: int, dim: int, value_dim: int, scale: float, eps: float, dtype: torch.dtype,
                 cap: float | None = None, bias: bool = False, taps: int = 0, weighted_norm: bool = False, rot_dims: int = 0,
                 rope=None, temperatures=None, runs: int = 1, short_rows: bool = True):
        super().__init__()
        self.num_heads, self.num_kv_heads, self.dim, self.value_dim = num_heads, num_kv_heads, dim, value_dim
        self.scale, self.eps, self.dtype, self.cap, self.rot_dims, self.runs = scale, eps, dtype, cap, rot_dims, runs
        self.short_rows = short_rows        # portions below the design's long_portion run row by row
        self.register_buffer("cos_sin", rope, persistent=False)
        self.register_buffer("temperatures", temperatures, persistent=False)
        self.parts = {"q": num_heads * dim, "k": num_kv_heads * dim, "v": num_kv_heads * value_dim, "g": num_heads * value_dim}
        self.channels = sum(self.parts[p] for p in "qkv")
        self.sink = nn.Parameter(torch.zeros(num_heads))
        self.bias = self.conv = self.q_norm = self.k_norm = None
        if bias:
            self.bias = nn.Parameter(torch.zeros(self.channels))
            self.bias.weight_loader = self.load_channels
        if taps:
            self.conv = nn.Parameter(torch.zeros(taps, self.channels))
            self.conv.weight_loader = self.load_channels
        if weighted_norm:
            self.q_norm, self.k_norm = nn.Module(), nn.Module()
            self.q_norm.weight, self.k_norm.weight = nn.Parameter(torch.ones(dim)), nn.Parameter(torch.ones(dim))
        # the preparation may add up split projections of single rows
        self.takes_partials = dim % 8 == 0 and value_dim % 8 == 0 and max(dim, value_dim) <= 256
        self.kv, self.rings = [None] * runs, [None] * runs      # bound by the model runner

    def load_channels(self, param: nn.Parameter, tensor: torch.Tensor, part: str):
        """Bias ``[channels]`` or convolution ``[channels, taps]`` of one projection."""
        at = 0
        for name in "qkv":
            if name == part:
                break
            at += self.parts[name]
        expected = (self.parts[part],) if param.dim() == 1 else (self.parts[part], param.shape[0])
        assert tuple(tensor.shape) == expected, (part, tuple(tensor.shape))
        param.data[..., at:at + self.parts[part]].copy_(tensor.T if tensor.dim() == 2 else tensor)

    # -- what the model runner asks a layer with a paged cache and a state
    def page_bytes(self, block_size: int) -> int:
        return self.runs * ops.SinkKV.page_bytes(block_size, self.num_kv_heads, self.dim, self.value_dim, self.dtype.itemsize)

    def bind_pages(self, pages: int, block_size: int, device):
        self.kv = [ops.SinkKV(pages, block_size, self.num_kv_heads, self.dim, self.value_dim, self.dtype, device) if pages else None
                   for _ in range(self.runs)]

    def slot_bytes(self) -> int:
        return 0 if self.conv is None else self.runs * self.conv.numel() * self.dtype.itemsize

    def bind_slots(self, slots: int, device):
        if self.conv is not None:
            self.rings = [torch.zeros(slots, *self.conv.shape, dtype=self.dtype, device=device) if slots else None
                          for _ in range(self.runs)]

    def takes_deferred(self, rows: int) -> bool:
        """Whether ``forward`` reads a step's projection as partial sums."""
        return self.takes_partials and get_context().num_single == rows

    def forward(self, proj, positions: torch.Tensor, run: int = 0) -> torch.Tensor:
        """``proj``: rows ``[q | k | v | gate]`` -> ``[N, heads * value_dim]``, gated."""
        ctx, kv, ring = get_context(), self.kv[run], self.rings[run]
        n, single = proj.shape[0], ctx.num_single
        data = lambda p: p.data if p is not None else None
        weight = lambda m: m.weight.data if m is not None else None
        q, gate = ops.sink_prep(proj, kv, self.num_heads, positions, ctx.slot_mapping, self.eps, self.scale, self.cap,
                                data(self.bias), data(self.conv),
                                ring, ctx.state_slots, ctx.row_seq if single < n else None, ctx.cu_seqlens_q, weight(self.q_norm),
                                weight(self.k_norm), self.cos_sin, self.rot_dims, self.temperatures)
        if ring is not None and single < n:
            ops.conv_tail(proj, ring, ctx.state_slots, ctx.cu_seqlens_q, ctx.seq_starts, single, ctx.cu_seqlens_q.numel() - 1 - single)
        out = torch.empty(n, self.num_heads * self.value_dim, dtype=self.dtype, device=q.device)
        tiles = self.dtype == torch.bfloat16 and ops.sink_prefill_supported(self.dim, self.value_dim)
        rows = n if not tiles else ctx.num_short_rows if self.short_rows else single
        if rows:
            ops.sink_attention_rows(q[:rows], kv, ctx.block_tables, positions[:rows], ctx.slot_mapping[:rows], self.sink.data,
                                    gate[:rows], self.cap, ctx.max_len, out[:rows],
                                    ctx.row_seq[:rows] if single < rows else None)
        if rows < n:
            first = single + (ctx.num_short if self.short_rows else 0)
            ops.sink_attention_prefill(q, kv, ctx.block_tables, ctx.cu_seqlens_q, ctx.seq_starts, first,
                                       ctx.cu_seqlens_q.numel() - 1 - first, ctx.max_portion, self.sink.data, gate, self.cap, out)
        return out
