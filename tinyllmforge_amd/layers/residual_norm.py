"""Norms in front of sublayers, around an fp32 residual stream: weights and the two fused steps."""
import torch
from torch import nn

from .. import ops


class ResidualRMSNorm(nn.Module):
    """``x / rms(x) * (offset + weight)``; ``offset`` 1: the weight is stored around zero."""

    def __init__(self, size: int, eps: float, offset: float = 0.0):
        super().__init__()
        self.eps, self.offset = eps, offset
        self.weight = nn.Parameter(torch.full((size,), 1.0 - offset))
        self.weight.identity = 1.0 - offset

    def after_embedding(self, ids: torch.Tensor, table: torch.Tensor):
        """``(x, self(x))`` with ``x`` the fp32 embedding rows."""
        return ops.embed_group_rms_norm(ids, table, self.weight.data, 1, self.eps, self.offset)

    def after_adding(self, y, x: torch.Tensor, mult: float, extra=None, extra_rows=None) -> torch.Tensor:
        """``x += mult * (y + extra rows)`` in place, then ``self(x)``: one kernel."""
        return ops.residual_rms_norm(y, x, mult, self.weight.data, self.offset, self.eps, extra, extra_rows)


class ResidualLayerNorm(nn.Module):
    """``((x - mean) / sqrt(variance + eps) * weight + bias) * out_scale``."""

    def __init__(self, size: int, eps: float, out_scale: float = 1.0):
        super().__init__()
        self.eps, self.out_scale = eps, out_scale
        self.weight, self.bias = nn.Parameter(torch.ones(size)), nn.Parameter(torch.zeros(size))
        self.bias.identity = 0.0

    def after_embedding(self, ids: torch.Tensor, table: torch.Tensor):
        """``(x, self(x))`` with ``x`` the fp32 embedding rows."""
        return ops.embed_layer_norm(ids, table, self.weight.data, self.bias.data, self.eps, self.out_scale)

    def after_adding(self, y, x: torch.Tensor, extra=None, extra_rows=None, extra_weights=None, own=None) -> torch.Tensor:
        """``x += y + weighted extra rows`` in place, then ``self(x)``: one kernel."""
        return ops.residual_layer_norm(y, x, self.weight.data, self.bias.data, self.eps, self.out_scale, extra, extra_rows,
                                       extra_weights, own)
