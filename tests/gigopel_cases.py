"""Small Gigopel configurations and random weights for the tests (no files, no fixtures)."""
import torch

from tests.gitopel_cases import logit_error, tokens  # noqa: F401  (the same for every design with a `vocab`)


def layer(heads, dim, rot, vdim, rank, size, mlp=None, scale=None, base=10000.0):
    return dict(type="latent_attention", mlp=mlp,
                mixer=dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=rank, mask=dict(size=size),
                           scale=scale if scale else 2.5 / (dim + rot) ** 0.5, rot=dict(base=base, dims=rot)))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, limit):
    return dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top))


def config(width, vocab, layers, eps=1e-6, mult=0.7):
    return dict(architecture="Gigopel", vocab=vocab, width=width, norm=dict(eps=eps), residual_mult=mult, layers=layers)


# name -> configuration: sizes that divide nothing, powers of two, one of everything, long cache rows, rows and values beyond
# what the matrix-core kernels take
CONFIGS = {
    "odd": config(90, 203, [layer(3, 20, 6, 13, 27, 37, dense(50)), layer(2, 9, 10, 21, 35, 5, moe(5, 2, 20, 1.5), base=700.0),
                            layer(5, 17, 2, 8, 12, 150)], eps=1e-4),
    "even": config(256, 320, [layer(4, 64, 32, 64, 128, 100, moe(8, 3, 64, 3.0)), layer(4, 64, 32, 64, 128, 100, dense(192)),
                              layer(8, 32, 64, 32, 64, 64, moe(16, 1, 128, 2.5))], mult=1.0),
    "ones": config(64, 96, [layer(1, 1, 2, 1, 1, 1, moe(1, 1, 1, 0.8)), layer(1, 8, 8, 8, 8, 3, dense(1)), layer(2, 3, 2, 5, 4, 2)]),
    "wide": config(192, 160, [layer(20, 96, 64, 128, 512, 130, moe(70, 6, 24, 2.0)), layer(33, 40, 8, 16, 72, 65, dense(100))], mult=0.3),
    "beyond": config(128, 150, [layer(2, 270, 8, 150, 640, 50, dense(64)), layer(3, 16, 16, 200, 1000, 90, moe(3, 2, 40, 1.0))]),
}


def shapes(cfg):
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,)}
    for i, la in enumerate(cfg["layers"]):
        p, m = f"l{i}.", la["mixer"]
        h, r, t = m["heads"], m["kv_rank"], m["rot_dim"]
        out |= {p + "norm1": (w,), p + "mix.q": (h * (m["dim"] + t), w), p + "mix.dkv": (r + t, w), p + "mix.dkv.norm": (r,),
                p + "mix.uk": (h * m["dim"], r), p + "mix.uv": (h * m["vdim"], r), p + "mix.o": (w, h * m["vdim"])}
        mlp = la["mlp"]
        if mlp and mlp["kind"] == "dense":
            out |= {p + "mlp.up": (mlp["ff"], w), p + "mlp.down": (w, mlp["ff"]), p + "mlp.act": (2,)}
        elif mlp:
            f = mlp["expert"]["ff"]
            out[p + "mlp.router"] = (mlp["router"]["experts"], w)
            for e in range(mlp["router"]["experts"]):
                out |= {p + f"mlp.e{e}.gate": (f, w), p + f"mlp.e{e}.up": (f, w), p + f"mlp.e{e}.down": (w, f)}
    return out


CLASS = 6      # leading residual channels that only the embedding writes: a token's class, which the routers read


def weights(cfg, seed=0):
    """bf16 tensors under their checkpoint names.  Softmax scores spread over several units, so that few keys carry a
    position's output.  The routers' choices are far from close calls: the class of a token stands in channels that no layer
    writes, and every class ranks the experts in an order of its own with even steps."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        x = torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if last == "norm" and "dkv" in name:
            x = 1 + 0.2 * x
        elif last.startswith("norm"):
            x = 0.2 * x
        elif name != "embed" and last != "act":
            x = x * shape[-1] ** -0.5
        if name == "embed":
            x[:, :CLASS] = 4.0 * torch.nn.functional.one_hot(torch.arange(shape[0]) % CLASS, CLASS)
        elif last in ("o", "down"):
            x[:CLASS] = 0
        elif last == "router":
            x = 0.02 * x
            steps = torch.linspace(-1, 1, shape[0]) if shape[0] > 1 else torch.ones(1)
            for c in range(CLASS):
                x[:, c] = steps[torch.randperm(shape[0], generator=g)]
        out[name] = x.to(torch.bfloat16)
    return out
