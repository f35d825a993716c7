"""Small Gitopel configurations and random weights for the tests (no files, no fixtures)."""
import torch


def attention(heads, kv, dim, rot, size, pool, ff=None, scale=None, base=10000.0):
    return dict(type="attention", mlp=dict(kind="dense", ff=ff) if ff else None,
                mixer=dict(heads=heads, kv_heads=kv, dim=dim, vdim=dim, scale=scale if scale else 4.0 / dim ** 0.5,
                           rot=dict(base=base, dims=rot), mask=dict(size=size, pool=pool)))


def gla(heads, dim, vdim, ff=None, tau=8.0, rank=16):
    return dict(type="gla", mlp=dict(kind="dense", ff=ff) if ff else None,
                mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau, rank=rank))


def config(width, groups, vocab, layers, eps=1e-6):
    return dict(architecture="Gitopel", vocab=vocab, width=width, norm=dict(groups=groups, eps=eps), layers=layers)


# name -> configuration: sizes that divide nothing, one of everything, wide heads, pools beyond a page or a window
CONFIGS = {
    "odd": config(90, 3, 203, [attention(6, 2, 40, 24, 37, 5), gla(3, 24, 20, ff=100, tau=3.0, rank=5),
                               attention(3, 1, 20, 20, 19, 4, ff=50, base=500.0)], eps=1e-5),
    "even": config(256, 4, 320, [gla(2, 64, 64, ff=192), attention(8, 2, 64, 64, 100, 16, ff=192), gla(2, 128, 128)]),
    "ones": config(64, 1, 96, [attention(1, 1, 32, 2, 1, 1, ff=64), gla(1, 16, 16, tau=1.0, rank=1), attention(5, 5, 32, 0, 64, 1)]),
    "wide": config(192, 2, 160, [attention(20, 1, 96, 64, 65, 70, ff=128), gla(1, 160, 272, rank=33), attention(2, 1, 256, 128, 8, 90)]),
}


def shapes(cfg):
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "head": (cfg["vocab"], w)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out |= {p + "norm1": (w,), p + "norm1b": (w,)}
        h, d = m["heads"], m["dim"]
        if layer["type"] == "attention":
            out |= {p + "mix.q": (h * d, w), p + "mix.q.b": (h * d,), p + "mix.k": (m["kv_heads"] * d, w),
                    p + "mix.k.b": (m["kv_heads"] * d,), p + "mix.pb": (h,), p + "mix.g": (h, w),
                    p + "mix.o": (w, h * d), p + "mix.o.b": (w,)}
        else:
            v, r = m["vdim"], m["rank"]
            out |= {p + "mix.q": (h * d, w), p + "mix.k": (h * d, w), p + "mix.v": (h * v, w), p + "mix.g": (h * v, w),
                    p + "mix.a1": (r, w), p + "mix.a2": (h * d, r), p + "mix.a2.b": (h * d,), p + "mix.norm": (v,),
                    p + "mix.o": (w, h * v)}
        if layer["mlp"]:
            f = layer["mlp"]["ff"]
            out |= {p + "norm2": (w,), p + "norm2b": (w,), p + "mlp.gate": (f, w), p + "mlp.up": (f, w), p + "mlp.down": (w, f)}
    return out


def weights(cfg, seed=0):
    """bf16 tensors under their checkpoint names.  Scores spread over several units around a negative bias, so few keys
    carry a position's output and a wrong one shows."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        x = torch.randn(shape, generator=g)
        if "norm" in name.split(".")[-1]:
            x = 1 + 0.2 * x
        elif name.endswith(".pb"):
            x = -3 + 0.5 * x
        elif name.endswith("a2.b"):
            x = 2 + x
        elif name.endswith(".b"):
            x = 0.3 * x
        elif name != "embed":
            x = x * shape[-1] ** -0.5
        out[name] = x.to(torch.bfloat16)
    # a gla head's output is normed, so where q . k of the only tokens it holds nearly cancels, rounding alone decides
    # the output: queries and keys that agree keep that from happening
    for i, layer in enumerate(cfg["layers"]):
        if layer["type"] == "gla":
            q, k = f"l{i}.mix.q", f"l{i}.mix.k"
            out[q] = (0.8 * out[k].float() + 0.6 * out[q].float()).to(torch.bfloat16)
    return out


def tokens(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def logit_error(got, want):
    """Root mean square over the vocabulary of the centred difference, over the spread of the wanted logits; per row."""
    d = got.double() - want.double()
    d = d - d.mean(dim=-1, keepdim=True)
    w = want.double() - want.double().mean(dim=-1, keepdim=True)
    return d.square().mean(dim=-1).sqrt() / w.square().mean().sqrt()
