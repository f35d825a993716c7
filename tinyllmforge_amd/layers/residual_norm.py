"""RMSNorm in front of sublayers that share it, around an fp32 residual stream: weights and the two fused steps."""
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
