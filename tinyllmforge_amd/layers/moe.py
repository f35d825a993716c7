"""Mixtures of experts: a router and small gated feed-forwards, run as grouped products."""
import torch
from torch import nn

from .. import ops
from .linear import _round_up, pad_2d, pad_columns


class GroupedExperts(nn.Module):
    """Weights of ``experts`` gated feed-forwards of which each token takes ``top``.  A router output beyond the experts stands
    for an ``identity`` expert, which has no weights."""

    def __init__(self, width: int, experts: int, top: int, ff: int, identity: int = 0):
        super().__init__()
        self.width, self.experts, self.top, self.ff, self.identity = width, experts, top, ff, identity
        self.columns, self.inter = _round_up(width, 64), _round_up(ff, 64)
        self.router = nn.Parameter(torch.zeros(_round_up(experts + identity, 16), self.columns))
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
            assert tuple(tensor.shape) == (self.experts + self.identity, self.width), tuple(tensor.shape)
            param.data[:self.experts + self.identity, :self.width].copy_(tensor)
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
        self.router.data[self.experts + self.identity:].zero_()
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

    def routes(self) -> dict:
        """Checkpoint names -> (parameter, part of it)."""
        out = {"router": ("router", "router")}
        for e in range(self.experts):
            for kind, target in (("gate", "gate_up"), ("up", "gate_up"), ("down", "down")):
                out[f"e{e}.{kind}"] = (target, (e, kind))
        return out


class ClippedGLUExperts(GroupedExperts):
    """Sigmoid scores of the ``top`` largest logits, clipped-GLU experts; an expert gets its input times the token's score.
    The result stays in expert order: rows to be added up through an index."""

    def __init__(self, width: int, experts: int, top: int, ff: int, limit: float):
        super().__init__(width, experts, top, ff)
        self.limit = limit

    def forward(self, h: torch.Tensor):
        """``(rows, index)``: the result for token t is the sum of ``rows[index[t]]``."""
        h = pad_columns(h, self.columns)
        rows = ops.moe_group(ops.moe_logits(h, self.router.data), self.experts, self.top, self.tile_rows(h.shape[0]))
        a = ops.moe_gemm(h, self.gate_up.data, rows, gather=True, clipped_glu=True, limit=self.limit)
        return ops.moe_gemm(a, self.down.data, rows, gather=False), rows.row_of


class SwiGLUExperts(GroupedExperts):
    """Softmax scores over all router outputs; the ``top`` largest of score plus correction are taken, weighted by their scores
    over the sum of them.  SwiGLU experts, and identity experts that hand the input through."""

    def __init__(self, width: int, experts: int, top: int, ff: int, identity: int = 0):
        super().__init__(width, experts, top, ff, identity)
        self.correction = nn.Parameter(torch.zeros(experts + identity))

    def forward(self, h: torch.Tensor):
        """``(rows, index, weights, h)``: the result for token t is the sum of ``weights[t] * rows[index[t]]``, an index below
        zero standing for ``h[t]``."""
        own = h
        h = pad_columns(h, self.columns)
        rows = ops.moe_group(ops.moe_logits(h, self.router.data), self.experts, self.top, self.tile_rows(h.shape[0]),
                             self.correction.data, self.identity)
        a = ops.moe_gemm(h, self.gate_up.data, rows, gather=True, swiglu=True)
        return ops.moe_gemm(a, self.down.data, rows, gather=False), rows.row_of, rows.scores, own

    def routes(self) -> dict:
        return super().routes() | {"correction": ("correction", None)}
