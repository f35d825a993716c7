"""SwiGLU gate (reference: tinyvllm/layers/activation.py:5-14)."""
import torch
from torch import nn

from .. import ops


class SiluAndMul(nn.Module):
    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return ops.silu_and_mul(x)


class XIELU(nn.Module):
    """``a z^2 + z/2`` above zero, ``b (e^z - 1 - z) + z/2`` below, with ``a = softplus(p)`` and ``b = 1/2 + softplus(q)``."""

    def __init__(self):
        super().__init__()
        self.pq = nn.Parameter(torch.zeros(2))

    def forward(self, x, col: int, cols: int, out: torch.Tensor) -> torch.Tensor:
        """Columns ``col ..`` of ``x`` (rows or ``ops.Deferred``) into ``out``."""
        return ops.xielu(x, col, cols, self.pq.data, out)
