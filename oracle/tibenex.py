"""Plain restatement of the Tibenex design, one function per mechanism, for tests only.

Explicit key sets, recurrences and convolutions token by token; no caches, no pages, no chunks, no batching.  ``dtype`` of the
inputs is the dtype of the arithmetic (CPU tensors).

Notation: ``x [T, W]`` the stream, ``h [T, W]`` the input of a sublayer, one row per position; weights are ``[out, in]``.
"""
from __future__ import annotations

import math

import torch


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def grouped_rms_norm(x: torch.Tensor, w: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """Equal parts of a row, each by its own root mean square."""
    parts = x.view(x.shape[0], groups, -1)
    return (parts / torch.sqrt((parts * parts).mean(dim=-1, keepdim=True) + eps)).reshape(x.shape) * w


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1 / (1 + torch.exp(-z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return z.clamp(min=0) + torch.log1p(torch.exp(-z.abs()))


def token_shift(x: torch.Tensor, mix: torch.Tensor) -> torch.Tensor:
    """Every row moved towards the row before it (zeros before the first), by ``mix`` per channel."""
    before = torch.cat([torch.zeros_like(x[:1]), x[:-1]])
    return x + (before - x) * mix


def post_norm(x: torch.Tensor, y: torch.Tensor, alpha: float, layer_scale, w, eps: float) -> torch.Tensor:
    return rms_norm(alpha * x + y * layer_scale, w, eps)


def causal_conv(u: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """``u [T, C]``, ``w [C, taps]``: the last tap meets the token itself, the one before it the token before, ..."""
    T, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        for back in range(min(taps, t + 1)):
            out[t] += w[:, taps - 1 - back] * u[t - back]
    return out + b


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


def angles(x: torch.Tensor, positions, rot: dict):
    f, mult = rotation_frequencies(rot)
    a = torch.tensor([[p * fi for fi in f] for p in positions], dtype=torch.float64).view(len(positions), 1, len(f))
    return (a.cos() * mult).to(x.dtype), (a.sin() * mult).to(x.dtype)


def rotate_halves(x: torch.Tensor, positions, rot: dict) -> torch.Tensor:
    """``x [T, H, D]``: dimension ``i`` turns with dimension ``i + dims / 2``; dimensions from ``dims`` on pass."""
    half = rot["dims"] // 2
    co, si = angles(x, positions, rot)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * co - v * si, v * co + u * si, x[..., 2 * half:]], dim=-1)


def rotate_neighbours(x: torch.Tensor, positions, rot: dict) -> torch.Tensor:
    """``x [T, H, D]``: dimension ``2 i`` turns with dimension ``2 i + 1``; dimensions from ``dims`` on pass."""
    dims = rot["dims"]
    co, si = angles(x, positions, rot)
    out = x.clone()
    out[..., 0:dims:2] = x[..., 0:dims:2] * co - x[..., 1:dims:2] * si
    out[..., 1:dims:2] = x[..., 1:dims:2] * co + x[..., 0:dims:2] * si
    return out


def causal_weights(s: torch.Tensor) -> torch.Tensor:
    """Softmax over the keys up to a query's own place; ``s [..., T, T]``."""
    T = s.shape[-1]
    s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf)
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def talking_attention(q, k, v, scale: float, temp, talk) -> torch.Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, Dv]``: every head's weights are a mix of all heads' softmax weights."""
    H, share = q.shape[1], q.shape[1] // k.shape[1]
    w = torch.stack([causal_weights(q[:, h] @ k[:, h // share].T * scale * temp[h]) for h in range(H)])
    mixed = [sum(talk[h, g] * w[g] for g in range(H)) for h in range(H)]
    return torch.stack([mixed[h] @ v[:, h // share] for h in range(H)], dim=1)


def attention_mixer(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    """``w``: the mixer's tensors by their short names; ``m``: its sizes and constants."""
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ w["q"].T, w["q.norm"], eps).view(T, H, D)
    k = rms_norm(h @ w["k"].T, w["k.norm"], eps).view(T, G, D)
    v = (h @ w["v"].T).view(T, G, Dv)
    q, k = rotate_neighbours(q, range(T), m["rot"]), rotate_neighbours(k, range(T), m["rot"])
    return talking_attention(q, k, v, m["scale"], w["temp"], w["talk"]).reshape(T, H * Dv) @ w["o"].T


def latent_mixer(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    T, H, D, R, Dv, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).view(T, H, D + R)
    down = h @ w["dkv"].T
    c, kr = rms_norm(down[:, :rank], w["dkv.norm"], eps), down[:, rank:].view(T, 1, R)
    q_rot, kr = rotate_halves(q[..., D:], range(T), m["rot"]), rotate_halves(kr, range(T), m["rot"])
    k, v = (c @ w["uk"].T).view(T, H, D), (c @ w["uv"].T).view(T, H, Dv)
    gate = sigmoid(h @ w["g"].T)
    out = []
    for i in range(H):
        s = (q[:, i, :D] @ k[:, i].T + q_rot[:, i] @ kr[:, 0].T) * m["scale"]
        out.append(causal_weights(s) @ v[:, i] * gate[:, i:i + 1])
    return torch.cat(out, dim=1) @ w["o"].T


def state_space_scan(x, B, C, dt, A_log, D) -> torch.Tensor:
    """``x [T, H, P]``, ``B, C [T, G, N]``, ``dt [T, H]``: one state ``[N, P]`` per head, token by token."""
    T, H, P = x.shape
    share = H // B.shape[1]
    y = torch.zeros_like(x)
    for h in range(H):
        S = torch.zeros(B.shape[2], P, dtype=x.dtype)
        for t in range(T):
            S = torch.exp(-torch.exp(A_log[h]) * dt[t, h]) * S + dt[t, h] * B[t, h // share][:, None] * x[t, h][None, :]
            y[t, h] = S.T @ C[t, h // share] + D[h] * x[t, h]
    return y


def mamba2_mixer(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    T, H, P, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = (h @ w["in"].T).split([inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = xbc.split([inner, G * N, G * N], dim=-1)
    dt = softplus(dt + w["dt_bias"])
    y = state_space_scan(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), dt, w["A_log"], w["D"]).reshape(T, inner)
    return grouped_rms_norm(y * silu(z), w["norm"], m["norm_groups"], eps) @ w["o"].T


MIXERS = {"attention": attention_mixer, "latent_attention": latent_mixer, "mamba2": mamba2_mixer}


def gated_mlp(h: torch.Tensor, gate, up, down) -> torch.Tensor:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, keep_layers: bool = False):
    """Logits ``[T, vocab]`` of one sequence; with ``keep_layers`` also the stream after every layer."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = t["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] * cfg["embedding"]["scale"]
    kept = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        w = {k[len(p) + 4:]: v for k, v in t.items() if k.startswith(p + "mix.")}
        y = MIXERS[layer["type"]](token_shift(x, t[p + "shift"]), w, layer["mixer"], eps)
        x = post_norm(x, y, alpha, t[p + "ls1"], t[p + "norm1"], eps)
        if layer.get("mlp"):
            y = gated_mlp(x, t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"])
            x = post_norm(x, y, alpha, t[p + "ls2"], t[p + "norm2"], eps)
        kept.append(x)
    logits = rms_norm(x, t["final.norm"], eps) @ t["head"].T
    return (logits, kept) if keep_layers else logits
