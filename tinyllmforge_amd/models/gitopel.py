"""Gitopel: a decoder whose layers are sigmoid attention over a window with pooled blocks, or gated linear attention,
each with an optional gated MLP, between grouped RMSNorms on both sides of every sublayer.

The residual stream is fp32.  Every sublayer ends in one kernel that applies its closing norm, adds to the residual and
applies the opening norm of whatever follows; all projections of a sublayer's input are one matrix product."""
import torch
from torch import nn

from ..config import GitopelConfig
from ..layers.embed_head import PaddedLMHead
from ..layers.gla import GatedLinearAttention
from ..layers.grouped_norm import GroupedRMSNorm
from ..layers.linear import GatedUpLinear, StackedLinear
from ..layers.pooled_attention import PooledWindowAttention
from ..utils.context import get_context
from .layered import LayeredForCausalLM, prefixed

DEFAULT_RANK = 16     # rows of a gla layer's first decay factor when no checkpoint fixes them


class GitopelAttention(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, dtype, rope):
        super().__init__()
        heads, kv, dim = m["heads"], m["kv_heads"], m["dim"]
        self.qkg = StackedLinear(width, {"q": heads * dim, "k": kv * dim, "g": heads})
        self.q_bias = nn.Parameter(torch.zeros(heads * dim))
        self.k_bias = nn.Parameter(torch.zeros(kv * dim))
        self.attn = PooledWindowAttention(heads, kv, dim, m["scale"], m["mask"]["size"], m["mask"]["pool"],
                                          m["rot"]["dims"], rope, eps, dtype)
        self.o = StackedLinear(heads * dim, {"o": width})
        self.o_bias = nn.Parameter(torch.zeros(width))

    def forward(self, h, positions):
        """The output projection without its bias (the norm that follows adds it), and that bias."""
        project = self.qkg.forward_deferred if self.attn.takes_partials else self.qkg
        o = self.attn(project(h), self.q_bias.data, self.k_bias.data, positions)
        return self.o.forward_deferred(o), self.o_bias.data

    routes = {"q": ("qkg.weight", "q"), "k": ("qkg.weight", "k"), "g": ("qkg.weight", "g"), "o": ("o.weight", "o"),
              "q.b": ("q_bias", None), "k.b": ("k_bias", None), "o.b": ("o_bias", None), "pb": ("attn.score_bias", None)}


class GitopelGLA(nn.Module):
    def __init__(self, width: int, m: dict, eps: float):
        super().__init__()
        heads, dk, dv, rank = m["heads"], m["dim"], m["vdim"], m.get("rank", DEFAULT_RANK)
        self.qkvgr = StackedLinear(width, {"q": heads * dk, "k": heads * dk, "v": heads * dv, "g": heads * dv, "a1": rank})
        self.gla = GatedLinearAttention(heads, dk, dv, rank, m["tau"], eps)
        self.o = StackedLinear(heads * dv, {"o": width})

    def forward(self, h, positions):
        single = get_context().num_single == h.shape[0]      # the prompt kernels read rows, the decode kernel partial sums
        proj = self.qkvgr.forward_deferred(h) if single else self.qkvgr(h)
        return self.o.forward_deferred(self.gla(proj, positions)), None

    routes = {**{p: ("qkvgr.weight", p) for p in ("q", "k", "v", "g", "a1")}, "o": ("o.weight", "o"),
              "a2": ("gla.decay_weight", None), "a2.b": ("gla.decay_bias", None), "norm": ("gla.norm.weight", None)}


class GitopelMLP(nn.Module):
    def __init__(self, width: int, ff: int):
        super().__init__()
        self.gate_up = GatedUpLinear(width, ff)
        self.down = StackedLinear(ff, {"down": width})

    def forward(self, h):
        return self.down.forward_deferred(self.gate_up.forward_silu_mul(h))

    routes = {"gate": ("gate_up.weight", 0), "up": ("gate_up.weight", 1), "down": ("down.weight", "down")}


class GitopelLayer(nn.Module):
    def __init__(self, cfg: GitopelConfig, layer: dict, rope):
        super().__init__()
        norm = lambda: GroupedRMSNorm(cfg.width, cfg.norm["groups"], cfg.norm["eps"])
        if layer["type"] == "attention":
            self.mix = GitopelAttention(cfg.width, layer["mixer"], cfg.norm["eps"], cfg.torch_dtype, rope)
        else:
            self.mix = GitopelGLA(cfg.width, layer["mixer"], cfg.norm["eps"])
        self.norm1, self.norm1b = norm(), norm()
        self.mlp = None
        if layer.get("mlp"):
            self.mlp = GitopelMLP(cfg.width, layer["mlp"]["ff"])
            self.norm2, self.norm2b = norm(), norm()

    def forward(self, positions, h, x, following: GroupedRMSNorm):
        """``h``: the residual ``x`` after ``norm1``; ``x`` is updated in place and returned normed by ``following``."""
        y, bias = self.mix(h, positions)
        h = self.norm1b.add_then(y, bias, x, self.norm2 if self.mlp is not None else following)
        if self.mlp is not None:
            h = self.norm2b.add_then(self.mlp(h), None, x, following)
        return h

    def routes(self) -> dict:
        norms = ["norm1", "norm1b"] + (["norm2", "norm2b"] if self.mlp is not None else [])
        out = {n: (n + ".weight", None) for n in norms} | prefixed("mix.", self.mix.routes)
        return out | prefixed("mlp.", self.mlp.routes) if self.mlp is not None else out


class GitopelForCausalLM(LayeredForCausalLM):
    fixed_tensors = LayeredForCausalLM.fixed_tensors | {"head": ("head.weight", "head")}

    def __init__(self, config: GitopelConfig):
        super().__init__(config)
        rope = lambda layer: self.rope_table(layer["mixer"]["rot"]) if layer["type"] == "attention" else None
        self.layers = nn.ModuleList([GitopelLayer(config, layer, rope(layer)) for layer in config.layers])
        self.norm = GroupedRMSNorm(config.width, config.norm["groups"], config.norm["eps"])
        self.head = PaddedLMHead(config.vocab, config.width)
