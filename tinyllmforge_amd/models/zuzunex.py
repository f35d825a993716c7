"""Zuzunex: a pre-norm decoder of grouped-query attention with sinks and output gates and of SwiGLU feed-forwards or mixtures
of experts with a shared expert, some of whose layers run several times in a row.

The residual stream is fp32.  Each sublayer ends in one kernel that adds to it and applies the layer norm of whatever follows;
queries, keys, values and the output gate are one product."""
from torch import nn

from ..config import ZuzunexConfig
from ..layers.embed_head import PaddedLMHead
from ..layers.linear import GatedUpLinear, StackedLinear
from ..layers.moe import SwiGLUExperts
from ..layers.residual_norm import ResidualLayerNorm
from ..layers.sink_attention import SinkAttention, query_temperatures
from ..utils.side_stream import on_the_side
from .layered import LayeredForCausalLM, prefixed

SIDE_BY_SIDE = 256      # up to this many rows the experts run beside the shared expert, on a stream of their own


class ZuzunexAttention(nn.Module):
    def __init__(self, cfg: ZuzunexConfig, layer: dict, runs: int, rope, temperatures):
        super().__init__()
        m, second = layer["mixer"], layer["type"] == "attention_2"
        rot = m.get("rot")
        self.attn = SinkAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], cfg.norm["eps"], cfg.torch_dtype,
                                  cap=m.get("softcap"), bias=second, taps=(m.get("conv") or 0) if second else 0, weighted_norm=second,
                                  rot_dims=rot["dims"] if rot else 0, rope=rope, temperatures=temperatures, runs=runs)
        self.qkvg = StackedLinear(cfg.width, self.attn.parts)
        self.o = StackedLinear(self.attn.parts["g"], {"o": cfg.width})

    def forward(self, h, positions, run: int):
        proj = self.qkvg.forward_deferred(h) if self.attn.takes_deferred(h.shape[0]) else self.qkvg(h)
        return self.o.forward_deferred(self.attn(proj, positions, run))

    def routes(self) -> dict:
        out = {p: ("qkvg.weight", p) for p in "qkvg"} | {"o": ("o.weight", "o"), "sink": ("attn.sink", None)}
        if self.attn.bias is not None:
            out |= {p + ".b": ("attn.bias", p) for p in "qkv"}
        if self.attn.conv is not None:
            out |= {p + ".conv": ("attn.conv", p) for p in "qkv"}
        if self.attn.q_norm is not None:
            out |= {"q.norm": ("attn.q_norm.weight", None), "k.norm": ("attn.k_norm.weight", None)}
        return out


class ZuzunexMLP(nn.Module):
    def __init__(self, width: int, ff: int):
        super().__init__()
        self.gate_up = GatedUpLinear(width, ff)
        self.down = StackedLinear(ff, {"down": width})

    def forward(self, h):
        """The sublayer's result as arguments of ``ResidualLayerNorm.after_adding``: what to add, extra rows."""
        return self.down.forward_deferred(self.gate_up.forward_silu_mul(h)), ()

    def routes(self) -> dict:
        return {"gate": ("gate_up.weight", 0), "up": ("gate_up.weight", 1), "down": ("down.weight", "down")}


class ZuzunexMoE(nn.Module):
    def __init__(self, width: int, mlp: dict):
        super().__init__()
        r = mlp["router"]
        self.experts = SwiGLUExperts(width, r["experts"], r["top"], mlp["expert"]["ff"], r.get("identity") or 0)
        self.shared = ZuzunexMLP(width, mlp["shared"]["ff"]) if mlp.get("shared") else None

    def forward(self, h):
        if self.shared is None:
            return None, self.experts(h)
        if h.shape[0] > SIDE_BY_SIDE:
            extra = self.experts(h)
            return self.shared(h)[0], extra
        with on_the_side(h.device) as join:
            extra = self.experts(h)
        y, _ = self.shared(h)
        join()
        return y, extra

    def routes(self) -> dict:
        out = prefixed("", {n: ("experts." + target, part) for n, (target, part) in self.experts.routes().items()})
        if self.shared is not None:
            out |= {"shared." + n: ("shared." + target, part) for n, (target, part) in self.shared.routes().items()}
        return out


class ZuzunexLayer(nn.Module):
    def __init__(self, cfg: ZuzunexConfig, layer: dict, runs: int, rope, temperatures):
        super().__init__()
        norm = lambda: ResidualLayerNorm(cfg.width, cfg.norm["eps"])
        self.norm1, self.mix = norm(), ZuzunexAttention(cfg, layer, runs, rope, temperatures)
        self.mlp = self.norm2 = None
        if layer.get("mlp"):
            mlp = layer["mlp"]
            self.norm2 = norm()
            self.mlp = ZuzunexMLP(cfg.width, mlp["ff"]) if mlp["kind"] == "dense" else ZuzunexMoE(cfg.width, mlp)

    def forward(self, positions, h, x, following: ResidualLayerNorm, run: int = 0):
        """``h``: the residual ``x`` after ``norm1``; ``x`` is updated in place and returned normed by ``following``."""
        y = self.mix(h, positions, run)
        if self.mlp is None:
            return following.after_adding(y, x)
        y, extra = self.mlp(self.norm2.after_adding(y, x))
        return following.after_adding(y, x, *extra)

    def routes(self) -> dict:
        norms = ["norm1"] + (["norm2"] if self.mlp is not None else [])
        out = {n: (n + ".weight", None) for n in norms} | {n + ".b": (n + ".bias", None) for n in norms}
        out |= {"mix." + n: ("mix." + target, part) for n, (target, part) in self.mix.routes().items()}
        return out | prefixed("mlp.", self.mlp.routes()) if self.mlp is not None else out


class ZuzunexForCausalLM(LayeredForCausalLM):
    fixed_tensors = LayeredForCausalLM.fixed_tensors | {"final.norm.b": ("norm.bias", None), "head": ("head.weight", "head")}

    def __init__(self, config: ZuzunexConfig):
        super().__init__(config)
        self._temperature_tables = {}
        runs = config.layer_runs()
        self.layers = nn.ModuleList([
            ZuzunexLayer(config, layer, runs.count(i), self.rope_table(layer["mixer"].get("rot")),
                         self.temperature_table(layer["mixer"].get("q_temp"))) for i, layer in enumerate(config.layers)])
        # the factor of the logits goes into what the head reads, before it is rounded
        self.norm = ResidualLayerNorm(config.width, config.norm["eps"], out_scale=config.logit_scale)
        self.head = PaddedLMHead(config.vocab, config.width)

    def temperature_table(self, q_temp: dict | None):
        """Layers with the same temperatures share a table."""
        if not q_temp:
            return None
        key = (q_temp["coef"], q_temp["every"])
        if key not in self._temperature_tables:
            self._temperature_tables[key] = query_temperatures(*key, self.config.max_position_embeddings).to(self.embed.device)
        return self._temperature_tables[key]

    def pack_linears_(self):
        super().pack_linears_()
        for layer in self.layers:
            if isinstance(layer.mlp, ZuzunexMoE):
                layer.mlp.experts.zero_pads_()
        return self
