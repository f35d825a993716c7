"""Gitopel: a decoder whose layers are sigmoid attention over a window with pooled blocks, or gated linear attention,
each with an optional gated MLP, between grouped RMSNorms on both sides of every sublayer.

The residual stream is fp32.  Every sublayer ends in one kernel that applies its closing norm, adds to the residual and
applies the opening norm of whatever follows; all projections of a sublayer's input are one matrix product."""
import re

import torch
from torch import nn

from .. import ops
from ..config import GitopelConfig
from ..layers.embed_head import PaddedLMHead
from ..layers.gla import GatedLinearAttention
from ..layers.grouped_norm import GroupedRMSNorm
from ..layers.linear import GatedUpLinear, StackedLinear
from ..layers.pooled_attention import PooledWindowAttention, interleaved_cos_sin
from ..utils.context import get_context

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


class GitopelForCausalLM(nn.Module):
    def __init__(self, config: GitopelConfig):
        super().__init__()
        self.config = config
        self.embed = nn.Parameter(torch.empty(config.vocab, config.width))
        tables = {}                          # layers with the same rotation share a table

        def rope(layer):
            if layer["type"] != "attention":
                return None
            key = (layer["mixer"]["rot"]["dims"], layer["mixer"]["rot"]["base"])
            if key not in tables:
                tables[key] = interleaved_cos_sin(key[0], config.max_position_embeddings, key[1]).to(self.embed.device)
            return tables[key]

        self.layers = nn.ModuleList([GitopelLayer(config, layer, rope(layer)) for layer in config.layers])
        self.norm = GroupedRMSNorm(config.width, config.norm["groups"], config.norm["eps"])
        self.head = PaddedLMHead(config.vocab, config.width)
        self.loaded_tensors: set[str] = set()

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        norms = [layer.norm1 for layer in self.layers] + [self.norm]
        x, h = norms[0].after_embedding(input_ids, self.embed.data)
        for layer, following in zip(self.layers, norms[1:]):
            h = layer(positions, h, x, following)
        return h

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        return self.head(hidden_states)

    def compute_greedy_ids(self, hidden_states: torch.Tensor) -> torch.Tensor:
        return self.head.forward_greedy(hidden_states)

    # -- checkpoint names
    def route_tensor(self, name: str):
        """Checkpoint tensor -> (parameter, part of it or None)."""
        fixed = {"embed": ("embed", None), "final.norm": ("norm.weight", None), "head": ("head.weight", "head")}
        if name in fixed:
            return fixed[name]
        m = re.fullmatch(r"l(\d+)\.(.+)", name)
        if m is None or int(m[1]) >= len(self.layers):
            raise KeyError(f"unknown tensor {name!r}")
        prefix, rest, layer = f"layers.{m[1]}.", m[2], self.layers[int(m[1])]
        if re.fullmatch(r"norm[12]b?", rest):
            return prefix + rest + ".weight", None
        group, _, short = rest.partition(".")
        module = {"mix": layer.mix, "mlp": layer.mlp}[group]
        target, part = module.routes[short]
        return f"{prefix}{group}.{target}", part

    def expected_tensors(self) -> set[str]:
        out = {"embed", "final.norm", "head"}
        for i, layer in enumerate(self.layers):
            names = ["norm1", "norm1b"] + ["mix." + k for k in layer.mix.routes]
            if layer.mlp is not None:
                names += ["norm2", "norm2b"] + ["mlp." + k for k in layer.mlp.routes]
            out |= {f"l{i}.{n}" for n in names}
        return out

    # -- what the engine does with the weights after loading
    def _linears(self):
        for layer in self.layers:
            yield from (m for m in layer.modules() if isinstance(m, (StackedLinear, GatedUpLinear)))

    def quantize_linears_(self):
        """Weight-only int8 for the projections of every layer (embedding and head stay as they are)."""
        for lin in self._linears():
            lin.zero_pads_()
            lin.quantize_()
        return self

    def pack_linears_(self):
        """Once after loading, on the GPU: pads back to zero, then the row and tile orders the fused kernels read."""
        for lin in [*self._linears(), self.head]:
            if not getattr(lin, "interleaved", False):
                lin.zero_pads_()
            if lin.is_quantized:
                lin.pack_()
            elif isinstance(lin, GatedUpLinear) and lin.weight.dtype == torch.bfloat16:
                lin.interleave_()
        return self
