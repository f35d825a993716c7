"""Mixture of experts: a router with sigmoid scores and small clipped-GLU feed-forwards, run as grouped products."""
import torch
from torch import nn

from .. import ops
from .linear import _round_up, pad_2d, pad_columns


class ClippedGLUExperts(nn.Module):
    """``experts`` feed-forwards of which each token takes the ``top`` with the largest scores; an expert gets its input
    times the token's score.  The result stays in expert order: rows to be added up through an index."""

    def __init__(self, width: int, experts: int, top: int, ff: int, limit: float):
        super().__init__()
        self.width, self.experts, self.top, self.ff, self.limit = width, experts, top, ff, limit
        self.columns, self.inter = _round_up(width, 64), _round_up(ff, 64)
        self.router = nn.Parameter(torch.zeros(_round_up(experts, 16), self.columns))
        self.gate_up = nn.Parameter(torch.zeros(experts, 2 * self.inter, self.columns))     # 8 gate rows, then the 8 up rows
        self.down = nn.Parameter(torch.zeros(experts, _round_up(width, 16), self.inter))
        for name in ("router", "gate_up", "down"):
            getattr(self, name).weight_loader = self.weight_loader

    def _channels(self, param, expert: int, which: int):
        """Gate (0) or up (1) rows of an expert: a view ``[inter / 8, 8, columns]``."""
        return param.data[expert].view(self.inter // 8, 2, 8, self.columns)[:, which]

    def weight_loader(self, param: nn.Parameter, tensor: torch.Tensor, shard):
        """``shard``: 'router' or (expert, 'gate' | 'up' | 'down')."""
        if shard == "router":
            assert tuple(tensor.shape) == (self.experts, self.width), tuple(tensor.shape)
            param.data[:self.experts, :self.width].copy_(tensor)
            return
        expert, kind = shard
        if kind == "down":
            assert tuple(tensor.shape) == (self.width, self.ff), tuple(tensor.shape)
            param.data[expert, :self.width, :self.ff].copy_(tensor)
        else:
            assert tuple(tensor.shape) == (self.ff, self.width), tuple(tensor.shape)
            self._channels(param, expert, int(kind == "up")).copy_(pad_2d(tensor, self.inter, self.columns).view(self.inter // 8, 8, -1))

    def zero_pads_(self):
        """After a random fill: the pads are zeros again."""
        self.router.data[self.experts:].zero_()
        for param in (self.router, self.gate_up):
            param.data[..., self.width:].zero_()
        if self.inter != self.ff:
            for expert in range(self.experts):
                for which in (0, 1):
                    rows = self._channels(self.gate_up, expert, which)
                    rows[-(-self.ff // 8):].zero_()
                    if self.ff % 8:
                        rows[self.ff // 8, self.ff % 8:].zero_()
        self.down.data[:, self.width:].zero_()
        self.down.data[..., self.ff:].zero_()

    def tile_rows(self, tokens: int) -> int:
        """Rows of a tile of the grouped products: rows per expert decide between streaming the weights and reusing them."""
        if self.router.dtype == torch.float32:
            return 64
        rows = tokens * self.top / self.experts
        return 32 if rows <= 8 else 64 if rows <= 32 else 128 if rows < 512 else 256

    def forward(self, h: torch.Tensor):
        """``(rows, index)``: the result for token t is the sum of ``rows[index[t]]``."""
        h = pad_columns(h, self.columns)
        rows = ops.moe_group(ops.moe_logits(h, self.router.data), self.experts, self.top, self.tile_rows(h.shape[0]))
        a = ops.moe_gemm(h, self.gate_up.data, rows, gather=True, clipped_glu=True, limit=self.limit)
        return ops.moe_gemm(a, self.down.data, rows, gather=False), rows.row_of
