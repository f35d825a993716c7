"""Tibenex: a post-norm decoder of latent attention, of attention whose heads mix their weights and of state-space layers, each with
an optional SwiGLU feed-forward.

The stream is fp32.  Every sublayer ends in one kernel that scales its result per channel, adds it to the stream, norms the sum
and makes what follows of it: the next mixer's input with the row before mixed in (token shift), or the head's."""
import torch
from torch import nn

from ..config import NO_WINDOW, TibenexConfig
from ..layers.embed_head import PaddedLMHead
from ..layers.latent_attention import LatentAttention
from ..layers.linear import GatedUpLinear, StackedLinear
from ..layers.residual_norm import ResidualPostNorm, ResidualRMSNorm, TokenShift
from ..layers.ssd import StateSpace
from ..layers.talking_attention import TalkingHeadsAttention
from ..utils.context import get_context
from .layered import LayeredForCausalLM, prefixed


class TibenexAttention(nn.Module):
    def __init__(self, cfg: TibenexConfig, m: dict, rope):
        super().__init__()
        rot = m.get("rot")
        self.attn = TalkingHeadsAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], cfg.norm["eps"], cfg.torch_dtype,
                                          rot["dims"] if rot else 0, rope)
        self.qkv = StackedLinear(cfg.width, self.attn.parts)
        self.o = StackedLinear(m["heads"] * m["vdim"], {"o": cfg.width})

    def forward(self, h, positions):
        return self.o.forward_deferred(self.attn(self.qkv.forward_deferred(h), positions))

    routes = {**{p: ("qkv.weight", p) for p in "qkv"}, "o": ("o.weight", "o"), "q.norm": ("attn.q_norm.weight", None),
              "k.norm": ("attn.k_norm.weight", None), "temp": ("attn.temp", None), "talk": ("attn.talk", None)}


class TibenexLatentAttention(nn.Module):
    def __init__(self, cfg: TibenexConfig, m: dict, rope):
        super().__init__()
        self.attn = LatentAttention(m["heads"], m["dim"], m["rot_dim"], m["kv_rank"], m["vdim"], m["scale"], NO_WINDOW,
                                    cfg.windows.index(NO_WINDOW), rope, cfg.norm["eps"], cfg.torch_dtype, halves=True)
        self.down = StackedLinear(cfg.width, {"dq": m["q_rank"], "dkv": m["kv_rank"] + m["rot_dim"], "g": m["heads"]})
        self.q_norm = nn.Module()
        self.q_norm.weight = nn.Parameter(torch.ones(m["q_rank"]))
        self.uq = StackedLinear(m["q_rank"], {"uq": m["heads"] * (m["dim"] + m["rot_dim"])})
        self.o = StackedLinear(m["heads"] * m["vdim"], {"o": cfg.width})

    def forward(self, h, positions):
        cq, gate = self.attn.prepare_down(self.down.forward_deferred(h), self.down.offset("dkv"), positions, self.down.offset("dq"),
                                          self.q_norm.weight.data, self.down.offset("g"))
        q = self.attn.prepare_queries(self.uq.forward_deferred(cq), positions)
        out = torch.empty(h.shape[0], self.o.input_size, dtype=h.dtype, device=h.device)
        self.attn(q, positions, out, gate)
        return self.o.forward_deferred(out)

    routes = {**{p: ("down.weight", p) for p in ("dq", "dkv", "g")}, "dq.norm": ("q_norm.weight", None), "uq": ("uq.weight", "uq"),
              "dkv.norm": ("attn.norm.weight", None), "uk": ("attn.uk", None), "uv": ("attn.uv", None), "o": ("o.weight", "o")}


class TibenexStateSpace(nn.Module):
    def __init__(self, cfg: TibenexConfig, m: dict):
        super().__init__()
        self.ssd = StateSpace(m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"], cfg.norm["eps"], cfg.torch_dtype)
        self.inp = StackedLinear(cfg.width, {"in": self.ssd.columns})
        self.o = StackedLinear(self.ssd.inner, {"o": cfg.width})

    def forward(self, h, positions):
        single = get_context().num_single == h.shape[0]      # the prompt kernels read rows, the decode kernel partial sums
        proj = self.inp.forward_deferred(h) if single else self.inp(h)
        return self.o.forward_deferred(self.ssd(proj, positions))

    routes = {"in": ("inp.weight", "in"), "conv": ("ssd.conv", "conv"), "conv.b": ("ssd.conv_bias", None),
              "dt_bias": ("ssd.dt_bias", None), "A_log": ("ssd.A_log", None), "D": ("ssd.D", None),
              "norm": ("ssd.norm.weight", None), "o": ("o.weight", "o")}


class TibenexMLP(nn.Module):
    def __init__(self, width: int, ff: int):
        super().__init__()
        self.gate_up = GatedUpLinear(width, ff)
        self.down = StackedLinear(ff, {"down": width})

    def forward(self, h):
        return self.down.forward_deferred(self.gate_up.forward_silu_mul(h))

    routes = {"gate": ("gate_up.weight", 0), "up": ("gate_up.weight", 1), "down": ("down.weight", "down")}


class TibenexLayer(nn.Module):
    def __init__(self, cfg: TibenexConfig, layer: dict, rope):
        super().__init__()
        m = layer["mixer"]
        norm = lambda: ResidualPostNorm(cfg.width, cfg.norm["eps"], cfg.postln_alpha)
        self.shift = TokenShift(cfg.width, cfg.embedding_scale)
        self.mix = (TibenexStateSpace(cfg, m) if layer["type"] == "mamba2" else
                    TibenexLatentAttention(cfg, m, rope) if layer["type"] == "latent_attention" else TibenexAttention(cfg, m, rope))
        self.norm1, self.mlp = norm(), None
        if layer.get("mlp"):
            self.mlp, self.norm2 = TibenexMLP(cfg.width, layer["mlp"]["ff"]), norm()

    def forward(self, positions, h, x, following):
        """``h``: the stream ``x`` after ``shift``; ``x`` is updated and returned as ``following`` (a later layer's shift or the
        final norm) makes it."""
        y = self.mix(h, positions)
        if self.mlp is None:
            return self.norm1.after_adding(y, x, positions, following)
        return self.norm2.after_adding(self.mlp(self.norm1.after_adding(y, x)), x, positions, following)

    def routes(self) -> dict:
        out = {"shift": ("shift.weight", None), "norm1": ("norm1.weight", None), "ls1": ("norm1.layer_scale", None)}
        out |= prefixed("mix.", self.mix.routes)
        if self.mlp is not None:
            out |= {"norm2": ("norm2.weight", None), "ls2": ("norm2.layer_scale", None)} | prefixed("mlp.", self.mlp.routes)
        return out


class TibenexForCausalLM(LayeredForCausalLM):
    front = "shift"
    fixed_tensors = LayeredForCausalLM.fixed_tensors | {"head": ("head.weight", "head")}

    def __init__(self, config: TibenexConfig):
        super().__init__(config)
        self.layers = nn.ModuleList([TibenexLayer(config, layer, self.rope_table(layer["mixer"].get("rot"))) for layer in config.layers])
        self.norm = ResidualRMSNorm(config.width, config.norm["eps"])
        self.head = PaddedLMHead(config.vocab, config.width)

    def pack_linears_(self):
        super().pack_linears_()
        for layer in self.layers:
            if isinstance(layer.mix, TibenexLatentAttention):
                layer.mix.attn.pack_()
        return self
