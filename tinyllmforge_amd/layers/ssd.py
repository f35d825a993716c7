"""State-space layer with a scalar decay per head (Mamba-2): short convolution, fp32 state per sequence and head, output gate
and grouped norm."""
import torch
from torch import nn

from .. import ops
from ..utils.context import get_context


class StateSpace(nn.Module):
    def __init__(self, num_heads: int, value_dim: int, state_dim: int, groups: int, taps: int, norm_groups: int, eps: float,
                 dtype: torch.dtype):
        super().__init__()
        self.num_heads, self.value_dim, self.state_dim, self.groups = num_heads, value_dim, state_dim, groups
        self.taps, self.norm_groups, self.eps, self.dtype = taps, norm_groups, eps, dtype
        self.inner = num_heads * value_dim
        self.channels = self.inner + 2 * groups * state_dim
        self.conv = nn.Parameter(torch.zeros(taps, self.channels))
        self.conv.weight_loader = self.load_conv
        self.conv_bias = nn.Parameter(torch.zeros(self.channels))
        self.dt_bias, self.A_log, self.D = (nn.Parameter(torch.zeros(num_heads)) for _ in range(3))
        self.norm = nn.Module()
        self.norm.weight = nn.Parameter(torch.ones(self.inner))
        self.state = self.ring = None       # fp32 [slots, heads, state, value], [slots, taps, channels]; bound by the model runner

    @property
    def columns(self) -> int:
        """Of a projection row ``[z | x | B | C | dt]``."""
        return self.inner + self.channels + self.num_heads

    def load_conv(self, param: nn.Parameter, tensor: torch.Tensor, part: str):
        assert tuple(tensor.shape) == (self.channels, self.taps), tuple(tensor.shape)
        param.data.copy_(tensor.T)

    # -- what the model runner asks a layer with a recurrent state
    def slot_bytes(self) -> int:
        return 4 * self.num_heads * self.state_dim * self.value_dim + self.taps * self.channels * self.dtype.itemsize

    def bind_slots(self, slots: int, device):
        self.state = self.ring = None
        if slots:
            self.state = torch.zeros(slots, self.num_heads, self.state_dim, self.value_dim, dtype=torch.float32, device=device)
            self.ring = torch.zeros(slots, self.taps, self.channels, dtype=self.dtype, device=device)

    def weights(self) -> ops.SsdWeights:
        return ops.SsdWeights(self.conv.data, self.conv_bias.data, self.dt_bias.data, self.A_log.data, self.D.data)

    def forward(self, proj, positions: torch.Tensor) -> torch.Tensor:
        """``proj``: rows ``[z | x | B | C | dt]`` -> ``[N, heads * value_dim padded to 64]``, gated and normed."""
        ctx, n = get_context(), proj.shape[0]
        single, w = ctx.num_single, self.weights()
        out = torch.empty(n, self.inner, dtype=self.dtype, device=self.state.device)
        if single:
            ops.ssd_decode(proj if single == n else proj[:single], w, self.ring, self.state, ctx.state_slots, positions[:single], self.groups,
                           out[:single])
        if single < n:
            portions = ctx.cu_seqlens_q.numel() - 1 - single
            ops.ssd_portions(proj, w, self.ring, self.state, ctx.state_slots, positions, ctx.row_seq, ctx.cu_seqlens_q, ctx.seq_starts, single,
                             portions, single, ctx.max_portion, self.groups, out)
            ops.conv_tail(proj[:, self.inner:], self.ring, ctx.state_slots, ctx.cu_seqlens_q, ctx.seq_starts, single, portions)
        return ops.rows_rms_norm(out, self.norm.weight.data, self.norm_groups, self.eps, 64)
