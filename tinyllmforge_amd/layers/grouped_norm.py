"""RMSNorm in groups around an fp32 residual stream: weights and the two fused steps."""
import torch
from torch import nn

from .. import ops


class GroupedRMSNorm(nn.Module):
    def __init__(self, size: int, groups: int, eps: float):
        super().__init__()
        self.groups, self.eps = groups, eps
        self.weight = nn.Parameter(torch.ones(size))

    def after_embedding(self, ids: torch.Tensor, table: torch.Tensor, positions=None):
        """``(x, self(x))`` with ``x`` the fp32 embedding rows."""
        return ops.embed_group_rms_norm(ids, table, self.weight.data, self.groups, self.eps)

    def add_then(self, y: torch.Tensor, bias, x: torch.Tensor, following: "GroupedRMSNorm") -> torch.Tensor:
        """``x += self(y + bias)`` in place, then ``following(x)``: one kernel."""
        return ops.group_rms_norm_add(y, bias, self.weight.data, x, following.weight.data, self.groups, self.eps)
