"""Small Zuzunex configurations and random weights for the tests (no files, no fixtures)."""
import torch

from tests.gitopel_cases import logit_error, tokens  # noqa: F401  (the same for every design with a `vocab`)


def attention(heads, kv, dim, vdim, mlp=None, every=16, coef=0.4, cap=6.0, scale=None):
    return dict(type="attention", mlp=mlp,
                mixer=dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale if scale else 2.5 / dim ** 0.5, softcap=cap,
                           q_temp=dict(coef=coef, every=every)))


def attention_2(heads, kv, dim, vdim, rot, mlp=None, conv=3, base=700.0, scaling=(3.0, 48, 8.0, 0.5), scale=None):
    s = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    return dict(type="attention_2", mlp=mlp,
                mixer=dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv, scale=scale if scale else 2.0 / dim ** 0.5,
                           rot=dict(base=base, dims=rot, scaling=s)))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, identity, top, ff, shared):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, identity=identity, top=top), shared=dict(ff=shared))


def config(width, vocab, layers, loop=None, eps=1e-5, logit_scale=0.3):
    return dict(architecture="Zuzunex", vocab=vocab, width=width, norm=dict(eps=eps), logit_scale=logit_scale, layers=layers,
                loop=dict(zip(("start", "stop", "times"), loop)) if loop else None)


# name -> configuration: sizes that divide nothing, powers of two, one of everything, many heads on one key/value head, heads
# beyond what the matrix-core kernels take
CONFIGS = {
    "odd": config(90, 203, [attention_2(3, 1, 20, 13, 12, dense(50)), attention(4, 2, 9, 21, moe(5, 1, 2, 20, 30)),
                            attention_2(5, 5, 17, 8, 6, moe(4, 3, 3, 17, 9), conv=5), attention(2, 1, 26, 34, every=7, cap=2.0)],
                  loop=(1, 3, 3), eps=1e-3),
    "even": config(256, 320, [attention(4, 2, 64, 64, moe(8, 2, 3, 64, 128), every=32), attention_2(4, 4, 64, 128, 64, dense(192), conv=4),
                              attention_2(8, 2, 128, 64, 32, moe(16, 4, 4, 128, 64), conv=2, scaling=None)], loop=(0, 2, 2), logit_scale=1.0),
    "ones": config(64, 96, [attention_2(1, 1, 2, 1, 2, moe(1, 0, 1, 1, 1), conv=1), attention(1, 1, 1, 1, dense(1), every=1),
                            attention(2, 2, 3, 5, moe(1, 1, 2, 8, 8), every=3)], loop=(2, 3, 1)),
    "wide": config(192, 160, [attention(20, 1, 192, 128, moe(70, 6, 6, 24, 40)), attention_2(33, 3, 40, 256, 40, dense(100)),
                              attention_2(4, 2, 96, 160, 16, moe(3, 2, 1, 40, 64))], loop=(1, 2, 2)),
    "beyond": config(128, 150, [attention_2(2, 1, 270, 150, 200, dense(64)), attention(6, 2, 16, 300, moe(3, 1, 2, 40, 24))], loop=(0, 2, 2)),
}


def shapes(cfg):
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "final.norm.b": (w,), "head": (cfg["vocab"], w)}
    for i, la in enumerate(cfg["layers"]):
        p, m = f"l{i}.", la["mixer"]
        parts = dict(q=m["heads"] * m["dim"], k=m["kv_heads"] * m["dim"], v=m["kv_heads"] * m["vdim"])
        out |= {p + "norm1": (w,), p + "norm1.b": (w,), p + "mix.sink": (m["heads"],), p + "mix.g": (m["heads"] * m["vdim"], w),
                p + "mix.o": (w, m["heads"] * m["vdim"])}
        for n, rows in parts.items():
            out[p + "mix." + n] = (rows, w)
            if la["type"] == "attention_2":
                out |= {p + f"mix.{n}.b": (rows,), p + f"mix.{n}.conv": (rows, m["conv"])}
        if la["type"] == "attention_2":
            out |= {p + "mix.q.norm": (m["dim"],), p + "mix.k.norm": (m["dim"],)}
        mlp = la["mlp"]
        if mlp:
            out |= {p + "norm2": (w,), p + "norm2.b": (w,)}
        if mlp and mlp["kind"] == "dense":
            out |= {p + "mlp.gate": (mlp["ff"], w), p + "mlp.up": (mlp["ff"], w), p + "mlp.down": (w, mlp["ff"])}
        elif mlp:
            r = mlp["router"]
            out |= {p + "mlp.router": (r["experts"] + r["identity"], w), p + "mlp.correction": (r["experts"] + r["identity"],)}
            for e in [f"e{k}" for k in range(r["experts"])] + ["shared"]:
                f = mlp["shared"]["ff"] if e == "shared" else mlp["expert"]["ff"]
                out |= {p + f"mlp.{e}.gate": (f, w), p + f"mlp.{e}.up": (f, w), p + f"mlp.{e}.down": (w, f)}
    return out


CLASS = 6      # leading residual channels that only the embedding writes: a token's class, which the routers read


def router_steps(outputs, top, g):
    """Router weights of a class, per output, in a random order: top - 1 large ones, one in the middle, the rest small."""
    high = max(top - 1, 1)
    steps = torch.cat([torch.linspace(1.0, 0.95, high), torch.full((1,), 0.5), torch.linspace(-0.8, -1.2, max(outputs - high - 1, 0))])
    return steps[:outputs][torch.randperm(outputs, generator=g)]


def weights(cfg, seed=0):
    """bf16 tensors under their checkpoint names.  Scores spread over several units, so that few keys carry a position's
    output; sinks as large as a good score.  The routers' choices are far from close calls: the class of a token stands in
    channels that no layer writes, and the choice is between scores with wide steps.  One expert's correction lifts it into
    every choice (where one is chosen: bars it from all)."""
    g = torch.Generator().manual_seed(seed)
    top_of = {f"l{i}.mlp.": la["mlp"]["router"]["top"] for i, la in enumerate(cfg["layers"]) if la["mlp"] and la["mlp"]["kind"] == "moe"}
    out = {}
    for name, shape in shapes(cfg).items():
        x = torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if last.startswith("norm"):
            x = 1 + 0.2 * x
            if "norm2" in name:
                x[:CLASS] = 1
        elif last == "b":
            x = 0.3 * x
            if "norm2" in name:
                x[:CLASS] = 0
        elif last == "sink":
            x = 3 + x
        elif last == "conv":
            x = x * 0.6
            x[:, -1] += 0.5
        elif name != "embed" and last != "correction":
            x = x * shape[-1] ** -0.5
        if name == "embed":
            x[:, :CLASS] = 6.5 * torch.nn.functional.one_hot(torch.arange(shape[0]) % CLASS, CLASS)
        elif last in ("o", "down"):
            x[:CLASS] = 0
            x *= 0.7
        elif last == "router":
            x = 0.004 * x
            for c in range(CLASS):
                x[:, c] = router_steps(shape[0], top_of[name[:-len("router")]], g)
        elif last == "correction":
            x = 0.002 * x
            x[int(torch.randint(shape[0], (1,), generator=g))] = 0.7 if top_of[name[:-len("correction")]] > 1 else -0.9
        out[name] = x.to(torch.bfloat16)
    return out
