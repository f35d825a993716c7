"""Gigopel: a decoder of parallel layers, windowed latent attention beside a dense xIELU feed-forward or a mixture of experts.

Both sublayers read one norm's output and are added to the fp32 residual together, times a constant.  So a layer is one
product in (queries, latent, rotated key and a dense feed-forward's channels stacked), one product out (attention heads and
those channels side by side), and one kernel that adds and applies the norm of the next layer."""
from torch import nn

from ..config import GigopelConfig
from ..layers.activation import XIELU
from ..layers.embed_head import TiedLMHead
from ..layers.latent_attention import LatentAttention
from ..layers.linear import JoinedLinear, StackedLinear
from ..layers.moe import ClippedGLUExperts
from ..layers.residual_norm import ResidualRMSNorm
from ..utils.side_stream import on_the_side
from .layered import LayeredForCausalLM

SIDE_BY_SIDE = 256      # up to this many rows the experts run beside the attention, on a stream of their own


class GigopelLayer(nn.Module):
    def __init__(self, cfg: GigopelConfig, layer: dict, rope):
        super().__init__()
        m, mlp, eps = layer["mixer"], layer.get("mlp"), cfg.norm["eps"]
        self.mult = cfg.residual_mult
        self.norm1 = ResidualRMSNorm(cfg.width, eps, offset=1.0)
        self.attn = LatentAttention(m["heads"], m["dim"], m["rot_dim"], m["kv_rank"], m["vdim"], m["scale"], m["mask"]["size"],
                                    cfg.windows.index(m["mask"]["size"]), rope, eps, cfg.torch_dtype)
        stacked = {"q": m["heads"] * (m["dim"] + m["rot_dim"]), "dkv": m["kv_rank"] + m["rot_dim"]}
        joined = {"o": m["heads"] * m["vdim"]}
        self.act = self.experts = None
        if mlp and mlp["kind"] == "dense":
            stacked["up"], joined["down"] = mlp["ff"], mlp["ff"]
            self.act = XIELU()
        elif mlp:
            self.experts = ClippedGLUExperts(cfg.width, mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"],
                                             mlp["expert"]["limit"])
        self.inp = StackedLinear(cfg.width, stacked)
        self.out = JoinedLinear(joined, cfg.width)

    def forward(self, positions, h, x, following: ResidualRMSNorm):
        # the projections are read by the kernels that follow at once, before any other product
        rows = self.out.input_rows(h.shape[0], h.dtype, h.device)
        if self.act is not None:
            proj = self.inp.forward_activated(h, "up", self.act, rows[:, self.out.offset("down"):])
        else:
            proj = self.inp.forward_deferred(h)
        q = self.attn.prepare(proj, self.inp.offset("dkv"), positions)
        extra, join = (None, None), None
        if self.experts is not None and h.shape[0] <= SIDE_BY_SIDE:
            with on_the_side(h.device) as join:
                extra = self.experts(h)
        elif self.experts is not None:
            extra = self.experts(h)
        self.attn(q, positions, rows)
        y = self.out.forward_deferred(rows)
        if join is not None:
            join()
        return following.after_adding(y, x, self.mult, *extra)

    def routes(self) -> dict:
        out = {"norm1": ("norm1.weight", None), "mix.q": ("inp.weight", "q"), "mix.dkv": ("inp.weight", "dkv"),
               "mix.dkv.norm": ("attn.norm.weight", None), "mix.uk": ("attn.uk", None), "mix.uv": ("attn.uv", None),
               "mix.o": ("out.weight", "o")}
        if self.act is not None:
            out |= {"mlp.up": ("inp.weight", "up"), "mlp.down": ("out.weight", "down"), "mlp.act": ("act.pq", None)}
        if self.experts is not None:
            out |= {"mlp." + n: ("experts." + target, part) for n, (target, part) in self.experts.routes().items()}
        return out


class GigopelForCausalLM(LayeredForCausalLM):
    def __init__(self, config: GigopelConfig):
        super().__init__(config)
        self.layers = nn.ModuleList([GigopelLayer(config, layer, self.rope_table(layer["mixer"]["rot"])) for layer in config.layers])
        self.norm = ResidualRMSNorm(config.width, config.norm["eps"], offset=1.0)
        self.head = TiedLMHead(config.vocab, config.width)

    def pack_linears_(self):
        super().pack_linears_()
        for layer in self.layers:
            layer.attn.pack_()
            if layer.experts is not None:
                layer.experts.zero_pads_()
        self.head.tie_(self.embed.data)
        return self
