"""Norms in front of sublayers or behind the sum, around an fp32 residual stream: weights and the fused steps."""
import torch
from torch import nn

from .. import ops
from ..utils.context import get_context


class ResidualRMSNorm(nn.Module):
    """``x / rms(x) * (offset + weight)``; ``offset`` 1: the weight is stored around zero."""

    def __init__(self, size: int, eps: float, offset: float = 0.0):
        super().__init__()
        self.eps, self.offset = eps, offset
        self.weight = nn.Parameter(torch.full((size,), 1.0 - offset))
        self.weight.identity = 1.0 - offset

    def after_embedding(self, ids: torch.Tensor, table: torch.Tensor, positions=None):
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

    def after_embedding(self, ids: torch.Tensor, table: torch.Tensor, positions=None):
        """``(x, self(x))`` with ``x`` the fp32 embedding rows."""
        return ops.embed_layer_norm(ids, table, self.weight.data, self.bias.data, self.eps, self.out_scale)

    def after_adding(self, y, x: torch.Tensor, extra=None, extra_rows=None, extra_weights=None, own=None) -> torch.Tensor:
        """``x += y + weighted extra rows`` in place, then ``self(x)``: one kernel."""
        return ops.residual_layer_norm(y, x, self.weight.data, self.bias.data, self.eps, self.out_scale, extra, extra_rows,
                                       extra_weights, own)


class TokenShift(nn.Module):
    """What a sublayer reads: the stream's row ``v`` moved towards the row before it, ``v + (before - v) * weight`` (zeros before
    a sequence's first).  The last row of every sequence is part of its state."""

    def __init__(self, size: int, embed_scale: float = 1.0):
        super().__init__()
        self.size, self.embed_scale = size, embed_scale
        self.weight = nn.Parameter(torch.zeros(size))
        self.ring = None                    # fp32 [slots, 2, size], position p in row p mod 2; bound by the model runner

    # -- what the model runner asks a layer with a recurrent state
    def slot_bytes(self) -> int:
        return 4 * 2 * self.size

    def bind_slots(self, slots: int, device):
        self.ring = torch.zeros(slots, 2, self.size, dtype=torch.float32, device=device) if slots else None

    def arguments(self, rows: int, positions) -> ops.ShiftArguments:
        ctx = get_context()
        portions = ctx.num_single < rows
        return ops.ShiftArguments(self.weight.data, self.ring, ctx.state_slots, positions, ctx.row_seq if portions else None,
                                  ctx.cu_seqlens_q if portions else None)

    def keep_last_rows(self, x: torch.Tensor):
        """Portions: their last rows into the state, once every row has been read."""
        ctx = get_context()
        if ctx.num_single < x.shape[0]:
            ops.conv_tail(x, self.ring, ctx.state_slots, ctx.cu_seqlens_q, ctx.seq_starts, ctx.num_single,
                          ctx.cu_seqlens_q.numel() - 1 - ctx.num_single)

    def after_embedding(self, ids: torch.Tensor, table: torch.Tensor, positions):
        """``(stream, shifted rows)`` with the stream's rows ``embed_scale`` times the embedding."""
        x, h = ops.embed_shift(ids, table, self.embed_scale, self.arguments(ids.numel(), positions))
        self.keep_last_rows(x)
        return Stream(x), h


class Stream:
    """The fp32 residual rows.  A step that reads its neighbours' rows again puts new ones in their place."""
    __slots__ = ("x",)

    def __init__(self, x: torch.Tensor):
        self.x = x


class ResidualPostNorm(nn.Module):
    """Norm behind the sum: ``x = rms_norm(alpha x + layer_scale * y) * weight``."""

    def __init__(self, size: int, eps: float, alpha: float):
        super().__init__()
        self.eps, self.alpha = eps, alpha
        self.weight, self.layer_scale = nn.Parameter(torch.ones(size)), nn.Parameter(torch.ones(size))

    def after_adding(self, y, stream: Stream, positions=None, following=None) -> torch.Tensor:
        """Updates the stream and returns its rows as they are (``following`` None), shifted (a ``TokenShift``) or normed (a
        ``ResidualRMSNorm``): one kernel."""
        x, shift = stream.x, following if isinstance(following, TokenShift) else None
        args = shift.arguments(x.shape[0], positions) if shift is not None else None
        stream.x, h = ops.post_rms_norm(y, x, self.alpha, self.layer_scale.data, self.weight.data, self.eps, args,
                                        following.weight.data if following is not None and shift is None else None)
        if shift is not None:
            shift.keep_last_rows(stream.x)
        return h
