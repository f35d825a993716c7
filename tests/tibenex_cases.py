"""Small Tibenex configurations and random weights for the tests (no files, no fixtures)."""
import torch

from tests.gitopel_cases import logit_error, tokens  # noqa: F401  (the same for every design with a `vocab`)


def dense(ff):
    return dict(kind="dense", ff=ff)


def attention(heads, kv, dim, vdim, rot, mlp=None, base=300.0, scale=None):
    """The weights of ``q.norm`` and ``k.norm`` are around 1: scores spread over several units."""
    return dict(type="attention", mlp=mlp and dense(mlp),
                mixer=dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale or 2.0 / dim ** 0.5, rot=dict(base=base, dims=rot)))


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, mlp=None, base=500.0, scaling=(4.0, 50, 9.0, 0.5), scale=None):
    s = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    return dict(type="latent_attention", mlp=mlp and dense(mlp),
                mixer=dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
                           scale=scale or 2.0 / (dim + rot_dim) ** 0.5, rot=dict(base=base, dims=rot_dim, scaling=s)))


def mamba2(heads, vdim, state, groups, conv=4, norm_groups=1, mlp=None):
    return dict(type="mamba2", mlp=mlp and dense(mlp),
                mixer=dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups))


def config(width, vocab, layers, alpha=1.6, scale=5.0, eps=1e-5):
    return dict(architecture="Tibenex", vocab=vocab, width=width, norm=dict(eps=eps), postln_alpha=alpha, embedding=dict(scale=scale), layers=layers)


# name -> configuration: sizes that divide nothing, powers of two, one of everything, many heads on one key/value head and many
# groups, sizes beyond what the matrix-core kernels take
CONFIGS = {
    "odd": config(90, 203, [mamba2(6, 10, 13, 3, conv=3, norm_groups=4, mlp=50), attention(6, 3, 20, 13, 12, mlp=70), latent(3, 11, 6, 9, 17, 21, mlp=33),
                            attention(2, 1, 26, 34, 26), latent(5, 20, 4, 23, 40, 9)], eps=1e-3),
    "even": config(256, 320, [attention(4, 2, 64, 64, 32, mlp=192), latent(4, 64, 32, 64, 128, 64, mlp=256), mamba2(8, 64, 64, 2, norm_groups=2),
                              attention(16, 4, 32, 64, 32), mamba2(4, 32, 128, 1, norm_groups=4, mlp=128)], alpha=1.0, scale=1.0),
    "ones": config(64, 96, [attention(1, 1, 2, 1, 2, mlp=1), latent(1, 1, 2, 1, 1, 1), mamba2(1, 1, 1, 1, conv=1, mlp=8), mamba2(2, 3, 2, 2, conv=2, norm_groups=2),
                            attention(3, 3, 5, 7, 2, mlp=40)]),
    "wide": config(192, 160, [attention(20, 1, 96, 40, 64, mlp=100), mamba2(12, 24, 40, 12, conv=5, norm_groups=12), latent(9, 128, 64, 128, 200, 96, mlp=64),
                              attention(32, 8, 16, 32, 8), mamba2(10, 48, 96, 5, conv=2, norm_groups=10)], alpha=2.3),
    "beyond": config(128, 150, [attention(40, 2, 24, 16, 8, mlp=64), mamba2(2, 300, 280, 1), latent(2, 260, 64, 150, 70, 300), attention(2, 1, 270, 140, 100),
                                attention(3, 1, 40, 260, 40, mlp=30)]),
}


def shapes(cfg):
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "head": (cfg["vocab"], w)}
    for i, la in enumerate(cfg["layers"]):
        p, m = f"l{i}.", la["mixer"]
        x = p + "mix."
        out |= {p + "shift": (w,), p + "ls1": (w,), p + "norm1": (w,), x + "o": (w, m["heads"] * m["vdim"])}
        if la["type"] == "attention":
            q, k = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            out |= {x + "q": (q, w), x + "k": (k, w), x + "v": (m["kv_heads"] * m["vdim"], w), x + "q.norm": (q,), x + "k.norm": (k,),
                    x + "temp": (m["heads"],), x + "talk": (m["heads"], m["heads"])}
        elif la["type"] == "latent_attention":
            out |= {x + "dq": (m["q_rank"], w), x + "dq.norm": (m["q_rank"],), x + "uq": (m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                    x + "dkv": (m["kv_rank"] + m["rot_dim"], w), x + "dkv.norm": (m["kv_rank"],), x + "uk": (m["heads"] * m["dim"], m["kv_rank"]),
                    x + "uv": (m["heads"] * m["vdim"], m["kv_rank"]), x + "g": (m["heads"], w)}
        else:
            inner, chan = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            out |= {x + "in": (inner + chan + m["heads"], w), x + "conv": (chan, m["conv"]), x + "conv.b": (chan,), x + "dt_bias": (m["heads"],),
                    x + "A_log": (m["heads"],), x + "D": (m["heads"],), x + "norm": (inner,)}
        if la["mlp"]:
            f = la["mlp"]["ff"]
            out |= {p + "ls2": (w,), p + "norm2": (w,), p + "mlp.gate": (f, w), p + "mlp.up": (f, w), p + "mlp.down": (w, f)}
    return out


def weights(cfg, seed=0):
    """bf16 tensors under their checkpoint names.  Scores spread over several units, heads mix with weights far from the
    identity, steps and decays from a few tokens to hundreds, shifts and layer scales that differ from channel to channel."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        x, last = torch.randn(shape, generator=g), name.split(".")[-1]
        if last.startswith("norm"):
            x = 1 + 0.2 * x
        elif last == "shift":
            x = 0.4 + 0.3 * x
        elif last in ("ls1", "ls2"):
            x = 0.8 + 0.3 * x
        elif last == "temp":
            x = 1.3 + 0.4 * x
        elif last == "talk":
            x = torch.eye(shape[0]) * 0.6 + x * 0.5 * shape[0] ** -0.5
        elif last == "A_log":
            x = 0.8 * x
        elif last == "dt_bias":
            x = -2.5 + 1.5 * x
        elif last == "D":
            x = 0.5 + 0.5 * x
        elif last == "b":
            x = 0.3 * x
        elif last == "conv":
            x = x * 0.5
            x[:, -1] += 0.5
        elif name != "embed":
            x = x * shape[-1] ** -0.5
            if last == "g":
                x = 1.5 * x
        out[name] = (0.4 * x if name == "embed" else x).to(torch.bfloat16)
    return out
