"""Plain restatement of the Gitopel design, one function per mechanism, for tests only.

Everything is written for reading: token-by-token recurrences, explicit key sets, no caches, no pages, no
batching.  ``dtype`` of the inputs is the dtype of the arithmetic (float32 or float64 tensors on the CPU).

Notation: ``h [T, W]`` the input of a sublayer, one row per position; weights are ``[out, in]``.
"""
from __future__ import annotations

import math

import torch


def grouped_rms_norm(x: torch.Tensor, w: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """Each of ``groups`` equal consecutive parts of the last dimension over its own root mean square, times ``w``."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    parts = parts / torch.sqrt((parts * parts).mean(dim=-1, keepdim=True) + eps)
    return parts.reshape(x.shape) * w


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1 + torch.exp(-z))


def rotate_interleaved(x: torch.Tensor, positions, dims: int, base: float) -> torch.Tensor:
    """``x [T, heads, D]``: dimensions (2i, 2i + 1), i < dims / 2, as the pair (u, v) turned by p * base^(-2i/dims)."""
    out = x.clone()
    for t, p in enumerate(positions):
        for i in range(dims // 2):
            a = float(p) * base ** (-2.0 * i / dims)
            c, s = math.cos(a), math.sin(a)
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            out[t, :, 2 * i] = u * c - v * s
            out[t, :, 2 * i + 1] = v * c + u * s
    return out


def rotate_interleaved_fast(x: torch.Tensor, positions, dims: int, base: float) -> torch.Tensor:
    """The same with one table for all rows (angles in double precision)."""
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    a = torch.as_tensor(positions, dtype=torch.float64)[:, None] * f
    c, s = a.cos().to(x.dtype)[:, None], a.sin().to(x.dtype)[:, None]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def visible_tokens(i: int, size: int) -> range:
    return range(max(0, i - size + 1), i + 1)


def visible_blocks(i: int, size: int, pool: int) -> list[int]:
    """Blocks of ``pool`` tokens whose last token left the window of position ``i``."""
    return [b for b in range(i // pool + 1) if b * pool + pool - 1 <= i - size]


def pooled_blocks(rows: torch.Tensor, pool: int) -> torch.Tensor:
    """Means of consecutive full blocks of ``pool`` rows."""
    n = rows.shape[0] // pool
    return torch.stack([rows[b * pool:(b + 1) * pool].mean(dim=0) for b in range(n)]) if n else rows[:0]


def sigmoid_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, bias: torch.Tensor, scale: float,
                      size: int, pool: int) -> torch.Tensor:
    """``q [T, H, D]``, ``k/v [T, G, D]`` -> ``[T, H, Dv]``: unnormalised sigmoid weights over the window's tokens and
    the pooled blocks behind it."""
    T, H, _ = q.shape
    G = k.shape[1]
    pk, pv = pooled_blocks(k, pool), pooled_blocks(v, pool)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for i in range(T):
        toks = visible_tokens(i, size)
        blocks = visible_blocks(i, size, pool)
        keys = torch.cat([k[toks.start:toks.stop], pk[blocks]])
        vals = torch.cat([v[toks.start:toks.stop], pv[blocks]])
        for h in range(H):
            g = h // (H // G)
            score = keys[:, g] @ q[i, h] * scale
            w = 1 / (1 + torch.exp(-(score + bias[h])))
            out[i, h] = w @ vals[:, g]
    return out


def attention_mixer(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    """``w``: the mixer's tensors by their short names; ``m``: its sizes and constants."""
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    T = h.shape[0]
    q = (h @ w["q"].T + w["q.b"]).view(T, H, D)
    k = (h @ w["k"].T + w["k.b"]).view(T, G, D)
    v = k
    pos = range(T)
    rot = lambda x: rotate_interleaved_fast(x, list(pos), m["rot"]["dims"], m["rot"]["base"])
    q, k = unit_rms(rot(q), eps), unit_rms(rot(k), eps)
    o = sigmoid_attention(q, k, v, w["pb"], m["scale"], m["mask"]["size"], m["mask"]["pool"])
    gate = 1 / (1 + torch.exp(-(h @ w["g"].T)))
    o = o * gate[:, :, None]
    return o.reshape(T, -1) @ w["o"].T + w["o.b"]


def gla_recurrence(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, log_alpha: torch.Tensor,
                   state: torch.Tensor | None = None):
    """``q/k/log_alpha [T, H, D]``, ``v [T, H, Dv]``, state ``[H, D, Dv]`` -> (o ``[T, H, Dv]``, last state)."""
    T, H, D = q.shape
    s = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(T):
        s = torch.exp(log_alpha[t])[:, :, None] * s + k[t][:, :, None] * v[t][:, None, :]
        out.append((s * q[t][:, :, None]).sum(dim=1))
    return torch.stack(out), s


def gla_mixer(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ w["q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w["k"].T).view(T, H, D)
    v = (h @ w["v"].T).view(T, H, Dv)
    z = ((h @ w["a1"].T) @ w["a2"].T + w["a2.b"]).view(T, H, D)
    log_alpha = -torch.nn.functional.softplus(-z) / m["tau"]          # log of sigmoid(z)^(1/tau)
    o, _ = gla_recurrence(q, k, v, log_alpha)
    o = (unit_rms(o, eps) * w["norm"]).reshape(T, H * Dv)
    return (o * silu(h @ w["g"].T)) @ w["o"].T


def dense_mlp(h: torch.Tensor, w: dict) -> torch.Tensor:
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


MIXERS = {"attention": attention_mixer, "gla": gla_mixer}


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, keep_layers: bool = False):
    """Logits ``[T, vocab]`` of one sequence; with ``keep_layers`` also the residual stream after every layer."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = t["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    layers = []

    def sub(prefix):
        return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}

    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = grouped_rms_norm(x, t[p + "norm1"], groups, eps)
        y = MIXERS[layer["type"]](h, sub(p + "mix."), layer["mixer"], eps)
        x = x + grouped_rms_norm(y, t[p + "norm1b"], groups, eps)
        if layer.get("mlp"):
            h = grouped_rms_norm(x, t[p + "norm2"], groups, eps)
            x = x + grouped_rms_norm(dense_mlp(h, sub(p + "mlp.")), t[p + "norm2b"], groups, eps)
        layers.append(x)
    logits = grouped_rms_norm(x, t["final.norm"], groups, eps) @ t["head"].T
    return (logits, layers) if keep_layers else logits
