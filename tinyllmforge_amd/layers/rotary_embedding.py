"""Rotary position embedding (reference: tinyvllm/layers/rotary_embedding.py:21-70).

The cos/sin table is computed on the host in fp32 with the reference's formula and uploaded,
so its bits are the same as a CPU restatement's; the rotation runs in the HIP kernel.
"""
import math
from functools import lru_cache

import torch
from torch import nn

from .. import ops


def build_cos_sin_cache(rotary_dim: int, max_position: int, base: float) -> torch.Tensor:
    """fp32 ``[max_position, rotary_dim]`` = cos || sin (rotary_embedding.py:31-36), on the CPU."""
    inv_freq = 1.0 / (base ** (torch.arange(0, rotary_dim, 2, dtype=torch.float32, device="cpu") / rotary_dim))
    t = torch.arange(max_position, dtype=torch.float32, device="cpu")
    freqs = torch.einsum("i,j -> ij", t, inv_freq)
    return torch.cat((freqs.cos(), freqs.sin()), dim=-1)


def yarn_frequencies(f: torch.Tensor, dims: int, base: float, factor: float, original: float, fast: float, slow: float):
    """YaRN: pairs that turn more than ``fast`` times over ``original`` positions keep their frequency, those that turn less
    than ``slow`` times have it divided by ``factor``, with a ramp over the pair index between.  Returns the frequencies and the
    factor of cos and sin."""
    pair = lambda turns: dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(pair(fast)), 0), min(math.ceil(pair(slow)), dims - 1)
    ramp = ((torch.arange(f.numel(), dtype=f.dtype, device=f.device) - lo) / max(hi - lo, 0.001)).clamp(0, 1)
    return f / factor * ramp + f * (1 - ramp), 0.1 * math.log(factor) + 1


def rotation_table(dims: int, max_position: int, base: float, **scaling) -> torch.Tensor:
    """fp32 ``[max_position, dims]`` = cos || sin of ``p * base^(-2 i / dims)``, or of scaled frequencies (``yarn_frequencies``);
    angles in double precision, CPU."""
    f = torch.tensor(base, dtype=torch.float64, device="cpu") ** (-torch.arange(0, dims, 2, dtype=torch.float64, device="cpu") / max(dims, 1))
    mult = 1.0
    if scaling:
        f, mult = yarn_frequencies(f, dims, base, **scaling)
    a = torch.arange(max_position, dtype=torch.float64, device="cpu")[:, None] * f
    return (torch.cat((a.cos(), a.sin()), dim=-1) * mult).float()


class RotaryEmbedding(nn.Module):
    def __init__(self, head_size: int, rotary_dim: int, max_position_embedding: int, base: float):
        super().__init__()
        assert rotary_dim == head_size
        self.head_size = head_size
        cache = build_cos_sin_cache(rotary_dim, max_position_embedding, base)
        self.register_buffer("cos_sin_cache", cache, persistent=False)

    def forward(self, positions: torch.Tensor, query: torch.Tensor, key: torch.Tensor):
        return ops.rope(positions, query, key, self.cos_sin_cache, self.head_size)


@lru_cache(1)
def get_rope(head_size: int, rotary_dim: int, max_position: int, base: float, rope_scaling=None):
    assert rope_scaling is None
    return RotaryEmbedding(head_size, rotary_dim, max_position, base)
