"""Plain restatement of the Zuzunex design, one function per mechanism, for tests only.

Explicit key sets, positions and convolutions token by token, experts applied token by token; no caches, no pages, no
batching.  ``dtype`` of the inputs is the dtype of the arithmetic (CPU tensors).

Notation: ``h [T, W]`` the input of a sublayer, one row per position; weights are ``[out, in]``.
"""
from __future__ import annotations

import math

import torch


def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    centred = x - x.mean(dim=-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(dim=-1, keepdim=True) + eps) * w + b


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1 + torch.exp(-z))


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1 / (1 + torch.exp(-z))


def causal_conv(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """``u [T, C]``, ``w [C, taps]``: the last tap meets the token itself, the one before it the token before, ..."""
    T, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        for back in range(min(taps, t + 1)):
            out[t] += w[:, taps - 1 - back] * u[t - back]
    return out


def query_temperature(position: int, coef: float, every: float) -> float:
    return 1 + coef * math.log(math.floor((position + 1) / every) + 1)


def rotation_frequencies(rot: dict) -> tuple[list, float]:
    """Frequency per pair and the factor of cos and sin.  With ``scaling`` (YaRN): pairs that turn more than ``fast`` times
    within ``original`` positions keep their frequency, those that turn less than ``slow`` times have it divided by ``factor``,
    in between a linear ramp over the pair index."""
    dims, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0
    turning = lambda t: dims * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))
    lo = max(math.floor(turning(sc["fast"])), 0)
    hi = min(math.ceil(turning(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1


def rotate_halves(x: torch.Tensor, positions, rot: dict) -> torch.Tensor:
    """``x [T, H, D]``: dimension ``i`` turns with dimension ``i + dims / 2``; dimensions from ``dims`` on pass."""
    f, mult = rotation_frequencies(rot)
    half = rot["dims"] // 2
    angle = torch.tensor([[p * fi for fi in f] for p in positions], dtype=torch.float64).view(len(positions), 1, half)
    co, si = (angle.cos() * mult).to(x.dtype), (angle.sin() * mult).to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * co - v * si, v * co + u * si, x[..., 2 * half:]], dim=-1)


def soft_cap(s: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(s / cap)


def sink_attention(q, k, v, scale: float, sink, cap=None) -> torch.Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, Dv]``: causal softmax whose denominator has ``exp(sink)`` more."""
    T, H = q.shape[:2]
    share = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = q[:, h] @ k[:, h // share].T * scale
        if cap is not None:
            s = soft_cap(s, cap)
        s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf)
        top = s.max(dim=-1, keepdim=True).values
        if sink is not None:
            top = top.clamp(min=sink[h].item())
        e = torch.exp(s - top)
        den = e.sum(dim=-1, keepdim=True)
        if sink is not None:
            den = den + torch.exp(sink[h] - top)
        out[:, h] = e / den @ v[:, h // share]
    return out


def mixer(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    """``w``: the mixer's tensors by their short names; ``m``: its sizes and constants."""
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def project(name):
        u = h @ w[name].T
        if name + ".b" in w:
            u = u + w[name + ".b"]
        return causal_conv(u, w[name + ".conv"]) if name + ".conv" in w else u

    q, k, v = project("q").view(T, H, D), project("k").view(T, G, D), project("v").view(T, G, Dv)
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    if "q.norm" in w:
        q, k = q * w["q.norm"], k * w["k.norm"]
    if m.get("q_temp"):
        q = q * torch.tensor([query_temperature(p, m["q_temp"]["coef"], m["q_temp"]["every"]) for p in range(T)], dtype=q.dtype).view(T, 1, 1)
    if m.get("rot"):
        q, k = rotate_halves(q, range(T), m["rot"]), rotate_halves(k, range(T), m["rot"])
    o = sink_attention(q, k, v, m["scale"], w.get("sink"), m.get("softcap")).reshape(T, H * Dv)
    return (o * sigmoid(h @ w["g"].T)) @ w["o"].T


def gated_mlp(h: torch.Tensor, gate, up, down) -> torch.Tensor:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(h: torch.Tensor, router: torch.Tensor, correction: torch.Tensor, top: int):
    """Chosen experts and their weights: chosen by softmax score plus correction, weighted by the scores alone, sum 1."""
    z = h @ router.T
    e = torch.exp(z - z.max(dim=-1, keepdim=True).values)
    s = e / e.sum(dim=-1, keepdim=True)
    chosen = (s + correction).topk(top, dim=-1).indices
    weights = s.gather(-1, chosen)
    return chosen, weights / (weights.sum(dim=-1, keepdim=True) + 1e-20)


def moe_mlp(h: torch.Tensor, w: dict, m: dict) -> torch.Tensor:
    r = m["router"]
    chosen, weights = route(h, w["router"], w["correction"], r["top"])
    out = gated_mlp(h, w["shared.gate"], w["shared.up"], w["shared.down"]) if m.get("shared") else torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, f in zip(chosen[t].tolist(), weights[t]):
            x = h[t:t + 1]
            y = x if e >= r["experts"] else gated_mlp(x, w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
            out[t] += f * y[0]
    return out


def feed_forward(h: torch.Tensor, w: dict, m: dict) -> torch.Tensor:
    return gated_mlp(h, w["gate"], w["up"], w["down"]) if m["kind"] == "dense" else moe_mlp(h, w, m)


def layer_order(cfg: dict) -> list:
    """Indices of the layers in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    inside = list(range(loop["start"], loop["stop"]))
    return list(range(loop["start"])) + inside * loop["times"] + list(range(loop["stop"], n))


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, keep_layers: bool = False):
    """Logits ``[T, vocab]`` of one sequence; with ``keep_layers`` also the residual stream after every layer run."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    norm = lambda x, name: layer_norm(x, t[name], t[name + ".b"], eps)
    x = t["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    kept = []

    def sub(prefix):
        return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}

    for i in layer_order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        x = x + mixer(norm(x, p + "norm1"), sub(p + "mix."), layer["mixer"], eps)
        if layer.get("mlp"):
            x = x + feed_forward(norm(x, p + "norm2"), sub(p + "mlp."), layer["mlp"])
        kept.append(x)
    logits = norm(x, "final.norm") @ t["head"].T * cfg["logit_scale"]
    return (logits, kept) if keep_layers else logits
