"""Plain restatement of the Gigopel design, one function per mechanism, for tests only.

Explicit key sets, full keys and values for every head (nothing is absorbed), experts applied token by token, no
caches, no pages, no batching.  ``dtype`` of the inputs is the dtype of the arithmetic (CPU tensors).

Notation: ``h [T, W]`` the input of a layer's sublayers, one row per position; weights are ``[out, in]``.
"""
from __future__ import annotations

import torch

from .gitopel import rotate_interleaved_fast


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Root mean square of the last dimension, with ``eps`` under the root."""
    return torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def zero_centred_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / rms(x, eps) * (1 + w)


def plain_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / rms(x, eps) * w


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0)


def xielu(z: torch.Tensor, p: torch.Tensor, q: torch.Tensor) -> torch.Tensor:
    """``a z^2 + z/2`` above zero, ``b (e^z - 1 - z) + z/2`` below, ``a = softplus(p)``, ``b = 1/2 + softplus(q)``."""
    above = softplus(p) * z * z + z / 2
    low = z.clamp(max=0)
    below = (0.5 + softplus(q)) * (torch.expm1(low) - low) + z / 2
    return torch.where(z > 0, above, below)


def window_keys(i: int, size: int) -> range:
    return range(max(0, i - size + 1), i + 1)


def softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, size: int) -> torch.Tensor:
    """``q``/``k [T, H, D]``, ``v [T, H, Dv]``: softmax over the ``size`` keys up to a position."""
    T = q.shape[0]
    out = torch.zeros(T, v.shape[1], v.shape[2], dtype=q.dtype)
    for i in range(T):
        at = window_keys(i, size)
        s = torch.einsum("hd,khd->hk", q[i], k[at.start:at.stop]) * scale
        e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
        out[i] = torch.einsum("hk,khd->hd", e / e.sum(dim=-1, keepdim=True), v[at.start:at.stop])
    return out


def latent_keys_values(c: torch.Tensor, turned: torch.Tensor, uk: torch.Tensor, uv: torch.Tensor, heads: int):
    """Per-head keys ``[own part | shared rotated part]`` and values from the latent ``c [T, R]``."""
    T = c.shape[0]
    own = (c @ uk.T).view(T, heads, -1)
    k = torch.cat([own, turned[:, None].expand(T, heads, turned.shape[-1])], dim=-1)
    return k, (c @ uv.T).view(T, heads, -1)


def latent_attention_mixer(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    """``w``: the mixer's tensors by their short names; ``m``: its sizes and constants."""
    H, D, R, rank = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    T = h.shape[0]
    turn = lambda x: rotate_interleaved_fast(x, list(range(T)), m["rot"]["dims"], m["rot"]["base"])
    q = (h @ w["q"].T).view(T, H, D + R)
    q = torch.cat([q[..., :D], turn(q[..., D:])], dim=-1)
    low = h @ w["dkv"].T
    c = plain_norm(low[:, :rank], w["dkv.norm"], eps)
    turned = turn(low[:, None, rank:])[:, 0]
    k, v = latent_keys_values(c, turned, w["uk"], w["uv"], H)
    o = softmax_attention(q, k, v, m["scale"], m["mask"]["size"])
    return o.reshape(T, -1) @ w["o"].T


def dense_mlp(h: torch.Tensor, w: dict) -> torch.Tensor:
    return xielu(h @ w["up"].T, w["act"][0], w["act"][1]) @ w["down"].T


def route(h: torch.Tensor, router: torch.Tensor, top: int):
    """Chosen experts (largest first) and their sigmoid scores, per row."""
    s = 1 / (1 + torch.exp(-(h @ router.T)))
    best = s.topk(top, dim=-1)
    return best.indices, best.values


def clipped_expert(x: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float) -> torch.Tensor:
    g = (x @ gate.T).clamp(max=limit)
    u = (x @ up.T).clamp(min=-limit, max=limit)
    return (g / (1 + torch.exp(-1.702 * g)) * (u + 1)) @ down.T


def moe_mlp(h: torch.Tensor, w: dict, m: dict) -> torch.Tensor:
    chosen, scores = route(h, w["router"], m["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        for t, k in (chosen == e).nonzero().tolist():
            x = scores[t, k] * h[t:t + 1]
            out[t] += clipped_expert(x, w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], m["expert"]["limit"])[0]
    return out


def feed_forward(h: torch.Tensor, w: dict, m: dict) -> torch.Tensor:
    return dense_mlp(h, w) if m["kind"] == "dense" else moe_mlp(h, w, m)


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, keep_layers: bool = False):
    """Logits ``[T, vocab]`` of one sequence; with ``keep_layers`` also the residual stream after every layer."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = t["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    layers = []

    def sub(prefix):
        return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}

    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = zero_centred_norm(x, t[p + "norm1"], eps)
        y = latent_attention_mixer(h, sub(p + "mix."), layer["mixer"], eps)
        if layer.get("mlp"):
            y = y + feed_forward(h, sub(p + "mlp."), layer["mlp"])
        x = x + mult * y
        layers.append(x)
    logits = zero_centred_norm(x, t["final.norm"], eps) @ t["embed"].T
    return (logits, layers) if keep_layers else logits
