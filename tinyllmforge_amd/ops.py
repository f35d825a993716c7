"""Tensor-level wrappers over the C ABI: one function per hot-path op.

Each wrapper validates what only Python can see (device, dtype), allocates the
output through torch (the caller owns every buffer, as in the reference) and
enqueues the kernel on torch's current stream, so calls are capturable by
``torch.cuda.graph``.  A tensor that is not on the GPU is an error.
"""
from __future__ import annotations

import torch

from . import _lib
from ._lib import DT_BF16, DT_F32, KV_BF16, KV_FP8_E4M3, check

BF16 = torch.bfloat16


def _stream():
    return torch.cuda.current_stream().cuda_stream


def _need(t: torch.Tensor, dtype, name: str):
    if not t.is_cuda:
        raise _lib.TlfError(f"{name} must be a GPU tensor (the HIP path has no CPU fallback)")
    if dtype is not None and t.dtype != dtype:
        raise _lib.TlfError(f"{name} must be {dtype}, got {t.dtype}")


_workspaces: dict = {}
_retired: list = []   # outgrown buffers stay alive: a captured graph may still point at them


def _workspace(nbytes: int, device, tag: str) -> torch.Tensor:
    """Grow-only scratch buffer per (device, tag).  Never freed, so pointers recorded in a
    captured graph stay valid.  No kernel needs it cleared."""
    key = (device, tag)
    ws = _workspaces.get(key)
    if ws is None or ws.numel() < nbytes:
        if ws is not None:
            _retired.append(ws)
        ws = torch.empty(max(nbytes, 256), dtype=torch.uint8, device=device)
        _workspaces[key] = ws
    return ws


def kv_dtype_code(cache: torch.Tensor) -> int:
    if cache.dtype == BF16:
        return KV_BF16
    if cache.dtype == torch.float8_e4m3fn:
        return KV_FP8_E4M3
    raise _lib.TlfError(f"unsupported KV-cache dtype {cache.dtype}")


# ------------------------------------------------------------------ a1
def store_kvcache(key, value, k_cache, v_cache, slot_mapping, k_scale=None, v_scale=None):
    """``key``/``value`` ``[N, Hkv, Dh]`` (row stride free), caches ``[nblk, bs, Hkv, Dh]``."""
    lib = _lib.load()
    _need(key, BF16, "key"); _need(value, BF16, "value")
    _need(slot_mapping, torch.int32, "slot_mapping")
    n, h, d = key.shape
    assert key.stride(-1) == 1 and value.stride(-1) == 1
    assert key.stride(1) == d and value.stride(1) == d
    assert k_cache.is_contiguous() and v_cache.is_contiguous()
    assert slot_mapping.numel() == n
    num_slots = k_cache.numel() // (h * d)
    if k_cache.dtype == BF16:
        check(lib.tlf_store_kvcache(key.data_ptr(), key.stride(0) * 2, value.data_ptr(), value.stride(0) * 2,
                                    k_cache.data_ptr(), v_cache.data_ptr(), slot_mapping.data_ptr(),
                                    n, h * d * 2, num_slots, _stream()), "tlf_store_kvcache")
    else:
        _need(k_scale, torch.float32, "k_scale"); _need(v_scale, torch.float32, "v_scale")
        check(lib.tlf_store_kvcache_fp8(key.data_ptr(), key.stride(0) * 2, value.data_ptr(), value.stride(0) * 2,
                                        k_cache.data_ptr(), v_cache.data_ptr(), slot_mapping.data_ptr(),
                                        n, h, d, k_scale.data_ptr(), v_scale.data_ptr(), num_slots, _stream()),
              "tlf_store_kvcache_fp8")


# ------------------------------------------------------------------ a5 / a6
def rms_norm(x, weight, eps):
    """``x [..., cols]`` bf16; leading dims may be a strided view ``[outer, inner, cols]``."""
    lib = _lib.load()
    _need(x, BF16, "x"); _need(weight, BF16, "weight")
    cols = x.shape[-1]
    assert x.stride(-1) == 1
    if x.dim() == 3 and not x.is_contiguous():
        outer, inner = x.shape[0], x.shape[1]
        assert x.stride(1) == cols
        ostride = x.stride(0)
    else:
        x = x if x.is_contiguous() else x.contiguous()
        outer, inner, ostride = x.numel() // cols, 1, cols
    y = torch.empty(x.shape, dtype=BF16, device=x.device)
    check(lib.tlf_rmsnorm(x.data_ptr(), ostride, weight.data_ptr(), y.data_ptr(), outer, inner, cols,
                          float(eps), _stream()), "tlf_rmsnorm")
    return y


def add_rms_norm(x, residual, weight, eps):
    lib = _lib.load()
    _need(x, BF16, "x"); _need(residual, BF16, "residual"); _need(weight, BF16, "weight")
    assert x.is_contiguous() and residual.is_contiguous() and x.shape == residual.shape
    cols = x.shape[-1]
    rows = x.numel() // cols
    y = torch.empty_like(x)
    r = torch.empty_like(x)
    check(lib.tlf_add_rmsnorm(x.data_ptr(), residual.data_ptr(), weight.data_ptr(), y.data_ptr(),
                              r.data_ptr(), rows, cols, float(eps), _stream()), "tlf_add_rmsnorm")
    return y, r


# ------------------------------------------------------------------ a7
def rope(positions, q, k, cos_sin, head_dim):
    lib = _lib.load()
    _need(positions, torch.int64, "positions"); _need(q, BF16, "q"); _need(k, BF16, "k")
    _need(cos_sin, torch.float32, "cos_sin_cache")
    n = positions.numel()
    assert q.stride(-1) == 1 and k.stride(-1) == 1 and q.dim() == 2 and k.dim() == 2
    hq, hkv = q.shape[1] // head_dim, k.shape[1] // head_dim
    qo = torch.empty(q.shape, dtype=BF16, device=q.device)
    ko = torch.empty(k.shape, dtype=BF16, device=k.device)
    check(lib.tlf_rope(positions.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0),
                       cos_sin.data_ptr(), qo.data_ptr(), ko.data_ptr(), n, hq, hkv, head_dim,
                       cos_sin.shape[0], _stream()), "tlf_rope")
    return qo, ko


def qknorm_rope_store(qkv, q_weight, k_weight, eps, positions, cos_sin, num_q_heads, num_kv_heads, head_dim,
                      k_cache=None, v_cache=None, slot_mapping=None, k_scale=None, v_scale=None,
                      want_kv=False):
    """Fused q/k-norm + RoPE + KV store.  Returns ``(q, k, v)``; ``k``/``v`` are None unless ``want_kv``."""
    lib = _lib.load()
    _need(qkv, BF16, "qkv"); _need(positions, torch.int64, "positions")
    n = qkv.shape[0]
    assert qkv.stride(-1) == 1
    q = torch.empty(n, num_q_heads * head_dim, dtype=BF16, device=qkv.device)
    k = v = None
    if want_kv:
        k = torch.empty(n, num_kv_heads * head_dim, dtype=BF16, device=qkv.device)
        v = torch.empty(n, num_kv_heads * head_dim, dtype=BF16, device=qkv.device)
    has_cache = k_cache is not None and k_cache.numel() > 0 and slot_mapping is not None
    kvd = kv_dtype_code(k_cache) if has_cache else KV_BF16
    num_slots = (k_cache.numel() // (num_kv_heads * head_dim)) if has_cache else 0
    check(lib.tlf_qknorm_rope_store(
        qkv.data_ptr(), qkv.stride(0), q_weight.data_ptr(), k_weight.data_ptr(), float(eps),
        positions.data_ptr(), cos_sin.data_ptr(), cos_sin.shape[0], q.data_ptr(),
        k.data_ptr() if k is not None else None, v.data_ptr() if v is not None else None,
        k_cache.data_ptr() if has_cache else None, v_cache.data_ptr() if has_cache else None,
        slot_mapping.data_ptr() if has_cache else None, num_slots, kvd,
        k_scale.data_ptr() if k_scale is not None else None,
        v_scale.data_ptr() if v_scale is not None else None,
        n, num_q_heads, num_kv_heads, head_dim, _stream()), "tlf_qknorm_rope_store")
    return q, k, v


# ------------------------------------------------------------------ a8
def silu_and_mul(x):
    lib = _lib.load()
    if x.dtype == torch.float32:
        _need(x, torch.float32, "x")
        assert x.is_contiguous() and x.shape[-1] % 2 == 0
        inter = x.shape[-1] // 2
        y = torch.empty(*x.shape[:-1], inter, dtype=x.dtype, device=x.device)
        check(lib.tlf_f32_silu_and_mul(x.data_ptr(), y.data_ptr(), x.numel() // (2 * inter), inter, _stream()),
              "tlf_f32_silu_and_mul")
        return y
    _need(x, BF16, "x")
    assert x.is_contiguous() and x.shape[-1] % 2 == 0
    inter = x.shape[-1] // 2
    rows = x.numel() // (2 * inter)
    y = torch.empty(*x.shape[:-1], inter, dtype=BF16, device=x.device)
    check(lib.tlf_silu_and_mul(x.data_ptr(), y.data_ptr(), rows, inter, _stream()), "tlf_silu_and_mul")
    return y


# ------------------------------------------------------------------ a9
def argmax(logits):
    lib = _lib.load()
    if logits.dtype == torch.float32:
        _need(logits, torch.float32, "logits")
        assert logits.dim() == 2 and logits.stride(1) == 1
        out = torch.empty(logits.shape[0], dtype=torch.int64, device=logits.device)
        check(lib.tlf_f32_argmax(logits.data_ptr(), logits.stride(0), out.data_ptr(), *logits.shape, _stream()), "tlf_f32_argmax")
        return out
    _need(logits, BF16, "logits")
    assert logits.dim() == 2 and logits.stride(1) == 1
    rows, vocab = logits.shape
    out = torch.empty(rows, dtype=torch.int64, device=logits.device)
    nbytes = lib.tlf_argmax_workspace_bytes(rows, vocab)
    ws = _workspace(nbytes, logits.device, "argmax")
    check(lib.tlf_argmax(logits.data_ptr(), logits.stride(0), out.data_ptr(), rows, vocab,
                         ws.data_ptr(), ws.numel(), _stream()), "tlf_argmax")
    return out


def sample(logits, temperatures, seed: int, offset: int):
    """Sampler with temperatures: greedy where ``temperatures == 0``, else one draw from
    ``softmax(logits / T)`` by the exponential-race formula of the reference, noise from Philox4x32-10
    at (``seed``, ``offset``).  int64 ``[rows]``."""
    lib = _lib.load()
    if logits.dtype == torch.float32 and logits.is_cuda:
        # the draw's noise is far coarser than the rounding; rows stay 16-byte aligned
        rows = torch.empty(logits.shape[0], (logits.shape[1] + 7) // 8 * 8, dtype=BF16, device=logits.device)
        logits = rows[:, :logits.shape[1]].copy_(logits)
    _need(logits, BF16, "logits"); _need(temperatures, torch.float32, "temperatures")
    assert logits.dim() == 2 and logits.stride(1) == 1 and temperatures.is_contiguous()
    rows, vocab = logits.shape
    assert temperatures.numel() == rows
    out = torch.empty(rows, dtype=torch.int64, device=logits.device)
    ws = _workspace(lib.tlf_argmax_workspace_bytes(rows, vocab), logits.device, "argmax")
    check(lib.tlf_sample(logits.data_ptr(), logits.stride(0), temperatures.data_ptr(), out.data_ptr(), rows,
                         vocab, seed & (2 ** 64 - 1), offset & (2 ** 64 - 1), ws.data_ptr(), ws.numel(),
                         _stream()), "tlf_sample")
    return out


# ------------------------------------------------------------------ K9
def embedding(ids, weight):
    lib = _lib.load()
    _need(ids, torch.int64, "ids"); _need(weight, BF16, "weight")
    assert weight.is_contiguous() and ids.is_contiguous()
    n = ids.numel()
    y = torch.empty(*ids.shape, weight.shape[1], dtype=BF16, device=weight.device)
    check(lib.tlf_embedding(ids.data_ptr(), weight.data_ptr(), y.data_ptr(), n, weight.shape[0],
                            weight.shape[1], _stream()), "tlf_embedding")
    return y


# ------------------------------------------------------------------ a10
class PackedW8:
    """An int8 weight ``[n, k]`` in the tile order the W8A16 kernels read (``tlf_w8a16_pack_weight``):
    same bytes as the row-major tensor, rows padded to a multiple of 32."""
    __slots__ = ("data", "n", "k")

    def __init__(self, data: torch.Tensor, n: int, k: int):
        self.data, self.n, self.k = data, n, k

    @property
    def shape(self):
        return (self.n, self.k)

    @property
    def device(self):
        return self.data.device

    def data_ptr(self):
        return self.data.data_ptr()


def pack_w8(wq: torch.Tensor) -> PackedW8:
    """Row-major int8 ``[N, K]`` -> ``PackedW8`` (one pass on the GPU)."""
    lib = _lib.load()
    _need(wq, torch.int8, "wq")
    assert wq.dim() == 2
    wq = wq.contiguous()
    N, K = wq.shape
    nbytes = lib.tlf_w8a16_packed_bytes(N, K)
    if nbytes == 0:
        raise _lib.TlfError(f"cannot pack an int8 weight of shape {tuple(wq.shape)} (K % 64 != 0)")
    out = torch.empty(nbytes, dtype=torch.int8, device=wq.device)
    check(lib.tlf_w8a16_pack_weight(wq.data_ptr(), out.data_ptr(), N, K, _stream()), "tlf_w8a16_pack_weight")
    return PackedW8(out, N, K)


def _packed(wq) -> PackedW8:
    """Weights may be given row-major (packed on the fly: convenient for one-off calls) or packed."""
    return wq if isinstance(wq, PackedW8) else pack_w8(wq)


def w8a16_linear(x, wq, scale):
    lib = _lib.load()
    w = _packed(wq)
    _need(x, BF16, "x"); _need(scale, torch.float32, "scale")
    assert x.stride(-1) == 1
    x2 = x.reshape(-1, x.shape[-1])
    M, K = x2.shape
    N = w.n
    assert w.k == K and scale.numel() == N
    y = torch.empty(M, N, dtype=BF16, device=x.device)
    nbytes = lib.tlf_w8a16_gemm_workspace_bytes(M, N, K)
    ws = _workspace(nbytes, x.device, "gemm")
    check(lib.tlf_w8a16_gemm(x2.data_ptr(), x2.stride(0), w.data_ptr(), scale.data_ptr(), y.data_ptr(),
                             M, N, K, ws.data_ptr(), ws.numel(), _stream()), "tlf_w8a16_gemm")
    return y.view(*x.shape[:-1], N)


def gate_up_interleave_index(n: int, device=None):
    """Row order of the fused gate_up weight: rows ``16 j .. 16 j + 7`` = gate channels ``8 j ..``, rows
    ``16 j + 8 .. 16 j + 15`` = the matching up channels; ``n`` = 2 x intermediate size.  ``w[idx]``
    interleaves a ``[gate; up]`` stacked weight (or scale)."""
    assert n % 16 == 0
    half = n // 2
    j = torch.arange(n, device=device)
    group, r = j // 16, j % 16
    return torch.where(r < 8, group * 8 + r, half + group * 8 + (r - 8))


def w8a16_linear_silu_mul(x, wq_interleaved, scale_interleaved):
    """``silu(gate) * up`` of the int8 gate_up projection in one kernel; weight rows interleaved as
    ``gate_up_interleave_index`` says.  Returns ``[..., N / 2]``."""
    lib = _lib.load()
    w = _packed(wq_interleaved)
    _need(x, BF16, "x"); _need(scale_interleaved, torch.float32, "scale")
    assert x.stride(-1) == 1
    x2 = x.reshape(-1, x.shape[-1])
    M, K = x2.shape
    N = w.n
    assert w.k == K
    y = torch.empty(M, N // 2, dtype=BF16, device=x.device)
    check(lib.tlf_w8a16_gemm_silu_mul(x2.data_ptr(), x2.stride(0), w.data_ptr(),
                                      scale_interleaved.data_ptr(), y.data_ptr(), M, N, K, _stream()),
          "tlf_w8a16_gemm_silu_mul")
    return y.view(*x.shape[:-1], N // 2)


def bf16_linear_silu_mul(x, w_interleaved):
    """``silu(gate) * up`` of the bf16 gate_up projection in one kernel; weight rows interleaved as
    ``gate_up_interleave_index`` says.  Returns ``[..., N / 2]``; the bits of ``silu_and_mul(bf16_linear(x, w))``."""
    lib = _lib.load()
    _need(x, BF16, "x"); _need(w_interleaved, BF16, "w")
    assert x.stride(-1) == 1 and w_interleaved.is_contiguous()
    x2 = x.reshape(-1, x.shape[-1])
    M, K = x2.shape
    N = w_interleaved.shape[0]
    assert w_interleaved.shape[1] == K and N % 16 == 0
    y = torch.empty(M, N // 2, dtype=BF16, device=x.device)
    check(lib.tlf_bf16_gemm_silu_mul(x2.data_ptr(), x2.stride(0), w_interleaved.data_ptr(), y.data_ptr(), M, N, K,
                                     _stream()), "tlf_bf16_gemm_silu_mul")
    return y.view(*x.shape[:-1], N // 2)


def linear(x, w):
    """``x . w^T`` in the weight's dtype (bf16 or 32-bit)."""
    return f32_linear(x, w) if w.dtype == torch.float32 else bf16_linear(x, w)


def f32_linear(x, w):
    lib = _lib.load()
    _need(x, torch.float32, "x"); _need(w, torch.float32, "w")
    assert x.stride(-1) == 1 and w.is_contiguous()
    x2 = x.reshape(-1, x.shape[-1])
    M, K = x2.shape
    N = w.shape[0]
    assert w.shape[1] == K
    y = torch.empty(M, N, dtype=torch.float32, device=x.device)
    check(lib.tlf_f32_gemm(x2.data_ptr(), x2.stride(0), w.data_ptr(), y.data_ptr(), M, N, K, _stream()), "tlf_f32_gemm")
    return y.view(*x.shape[:-1], N)


def bf16_linear(x, w):
    lib = _lib.load()
    _need(x, BF16, "x"); _need(w, BF16, "w")
    assert x.stride(-1) == 1 and w.is_contiguous()
    x2 = x.reshape(-1, x.shape[-1])
    M, K = x2.shape
    N = w.shape[0]
    y = torch.empty(M, N, dtype=BF16, device=x.device)
    nbytes = lib.tlf_w8a16_gemm_workspace_bytes(M, N, K)
    ws = _workspace(nbytes, x.device, "gemm")
    check(lib.tlf_bf16_gemm(x2.data_ptr(), x2.stride(0), w.data_ptr(), y.data_ptr(), M, N, K,
                            ws.data_ptr(), ws.numel(), _stream()), "tlf_bf16_gemm")
    return y.view(*x.shape[:-1], N)


def bf16_linear_argmax(x, w):
    """``argmax(bf16_linear(x, w), -1)`` (first index among ties) without the logits: int64 ``[M]``."""
    lib = _lib.load()
    _need(x, BF16, "x"); _need(w, BF16, "w")
    assert x.stride(-1) == 1 and w.is_contiguous() and x.dim() == 2
    M, K = x.shape
    N = w.shape[0]
    out = torch.empty(M, dtype=torch.int64, device=x.device)
    ws = _workspace(lib.tlf_gemm_argmax_workspace_bytes(M, N, K), x.device, "gemm")
    check(lib.tlf_bf16_gemm_argmax(x.data_ptr(), x.stride(0), w.data_ptr(), out.data_ptr(), M, N, K,
                                   ws.data_ptr(), ws.numel(), _stream()), "tlf_bf16_gemm_argmax")
    return out


def linear_add_rms_norm(x, w, scale, residual, norm_weight, eps):
    """``add_rms_norm(linear(x), residual)`` behind one call: ``w`` int8 with ``scale`` (weight-only int8)
    or bf16 with ``scale=None``.  Returns ``(normed, new_residual)``, the bits of the two separate calls."""
    lib = _lib.load()
    w8 = scale is not None
    if w8:
        w = _packed(w)
    else:
        _need(w, BF16, "w")
        assert w.is_contiguous()
    _need(x, BF16, "x"); _need(residual, BF16, "residual"); _need(norm_weight, BF16, "norm_weight")
    assert x.stride(-1) == 1 and residual.is_contiguous()
    x2 = x.reshape(-1, x.shape[-1])
    M, K = x2.shape
    N = w.shape[0]
    assert residual.numel() == M * N
    y = torch.empty(M, N, dtype=BF16, device=x.device)
    r = torch.empty(M, N, dtype=BF16, device=x.device)
    ws = _workspace(lib.tlf_gemm_add_rmsnorm_workspace_bytes(M, N, K), x.device, "gemm")
    if w8:
        _need(scale, torch.float32, "scale")
        check(lib.tlf_w8a16_gemm_add_rmsnorm(
            x2.data_ptr(), x2.stride(0), w.data_ptr(), scale.data_ptr(), residual.data_ptr(),
            norm_weight.data_ptr(), y.data_ptr(), r.data_ptr(), M, N, K, float(eps), ws.data_ptr(),
            ws.numel(), _stream()), "tlf_w8a16_gemm_add_rmsnorm")
    else:
        check(lib.tlf_bf16_gemm_add_rmsnorm(
            x2.data_ptr(), x2.stride(0), w.data_ptr(), residual.data_ptr(), norm_weight.data_ptr(),
            y.data_ptr(), r.data_ptr(), M, N, K, float(eps), ws.data_ptr(), ws.numel(), _stream()),
            "tlf_bf16_gemm_add_rmsnorm")
    shape = (*x.shape[:-1], N)
    return y.view(shape), r.view(shape)


def linear_qknorm_rope_store(x, w, scale, q_weight, k_weight, eps, positions, cos_sin, num_q_heads, num_kv_heads,
                             head_dim, k_cache=None, v_cache=None, slot_mapping=None, k_scale=None, v_scale=None,
                             want_kv=False):
    """``qknorm_rope_store(linear(x), ...)`` behind one call: ``w`` int8 with ``scale`` (weight-only int8) or
    bf16 with ``scale=None``.  Returns ``(q, k, v)`` with the bits of the two separate calls."""
    lib = _lib.load()
    w8 = scale is not None
    if w8:
        w = _packed(w)
        _need(scale, torch.float32, "scale")
    else:
        _need(w, BF16, "w")
        assert w.is_contiguous()
    _need(x, BF16, "x"); _need(positions, torch.int64, "positions")
    assert x.stride(-1) == 1
    x2 = x.reshape(-1, x.shape[-1])
    n, K = x2.shape
    N = (num_q_heads + 2 * num_kv_heads) * head_dim
    assert w.shape[0] == N
    q = torch.empty(n, num_q_heads * head_dim, dtype=BF16, device=x.device)
    k = v = None
    if want_kv:
        k = torch.empty(n, num_kv_heads * head_dim, dtype=BF16, device=x.device)
        v = torch.empty(n, num_kv_heads * head_dim, dtype=BF16, device=x.device)
    has_cache = k_cache is not None and k_cache.numel() > 0 and slot_mapping is not None
    kvd = kv_dtype_code(k_cache) if has_cache else KV_BF16
    num_slots = (k_cache.numel() // (num_kv_heads * head_dim)) if has_cache else 0
    ws = _workspace(lib.tlf_gemm_qknorm_rope_store_workspace_bytes(n, N, K), x.device, "gemm")
    tail = (q_weight.data_ptr(), k_weight.data_ptr(), float(eps), positions.data_ptr(), cos_sin.data_ptr(),
            cos_sin.shape[0], q.data_ptr(), k.data_ptr() if k is not None else None,
            v.data_ptr() if v is not None else None, k_cache.data_ptr() if has_cache else None,
            v_cache.data_ptr() if has_cache else None, slot_mapping.data_ptr() if has_cache else None, num_slots,
            kvd, k_scale.data_ptr() if k_scale is not None else None,
            v_scale.data_ptr() if v_scale is not None else None, n, num_q_heads, num_kv_heads, head_dim, K,
            ws.data_ptr(), ws.numel(), _stream())
    if w8:
        check(lib.tlf_w8a16_gemm_qknorm_rope_store(x2.data_ptr(), x2.stride(0), w.data_ptr(), scale.data_ptr(),
                                                   *tail), "tlf_w8a16_gemm_qknorm_rope_store")
    else:
        check(lib.tlf_bf16_gemm_qknorm_rope_store(x2.data_ptr(), x2.stride(0), w.data_ptr(), *tail),
              "tlf_bf16_gemm_qknorm_rope_store")
    return q, k, v


# ------------------------------------------------------------------ a3
def paged_decode_plan(context_lens, block_tables, block_size, out=None):
    """The work split of ``paged_decode_attention`` for one decode step, made once for all layers (they share the
    lengths and the block tables).  Returns an int32 tensor to pass as ``plan=``; ``out`` re-uses one (a captured
    graph keeps its pointer)."""
    lib = _lib.load()
    _need(context_lens, torch.int32, "context_lens"); _need(block_tables, torch.int32, "block_tables")
    assert block_tables.stride(1) == 1 and context_lens.is_contiguous()
    nbytes = lib.tlf_paged_decode_plan_bytes()
    plan = out if out is not None else torch.empty(nbytes // 4, dtype=torch.int32, device=context_lens.device)
    assert plan.dtype == torch.int32 and plan.numel() * 4 >= nbytes and plan.is_contiguous()
    check(lib.tlf_paged_decode_plan(context_lens.data_ptr(), block_tables.data_ptr(), block_tables.stride(0),
                                    context_lens.numel(), int(block_size), block_tables.shape[1], plan.data_ptr(),
                                    plan.numel() * 4, _stream()), "tlf_paged_decode_plan")
    return plan


def paged_decode_attention(q, k_cache, v_cache, context_lens, block_tables, scale,
                           k_scale=None, v_scale=None, plan=None):
    """``q [B, Hq, Dh]`` -> ``[B, Hq*Dh]``; caches ``[nblk, bs, Hkv, Dh]``.  ``plan``: the output of
    ``paged_decode_plan`` for these lengths and tables (same bits, a shorter start)."""
    lib = _lib.load()
    _need(q, BF16, "q"); _need(context_lens, torch.int32, "context_lens")
    _need(block_tables, torch.int32, "block_tables")
    B, Hq, Dh = q.shape
    assert q.stride(2) == 1 and q.stride(1) == Dh
    nblk, bs, Hkv, _ = k_cache.shape
    assert k_cache.is_contiguous() and v_cache.is_contiguous() and block_tables.stride(1) == 1
    maxb = block_tables.shape[1]
    out = torch.empty(B, Hq * Dh, dtype=BF16, device=q.device)
    # sized for the largest batch so that one buffer serves every call (graph capture keeps its pointer)
    nbytes = lib.tlf_paged_decode_attn_workspace_bytes(max(B, 1024), Hq, Dh, maxb, bs)
    ws = _workspace(nbytes, q.device, "decode")
    args = (q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(), kv_dtype_code(k_cache),
            k_scale.data_ptr() if k_scale is not None else None,
            v_scale.data_ptr() if v_scale is not None else None,
            block_tables.data_ptr(), block_tables.stride(0), context_lens.data_ptr(), out.data_ptr(),
            B, Hq, Hkv, Dh, bs, maxb, nblk, float(scale), ws.data_ptr(), ws.numel())
    if plan is None:
        check(lib.tlf_paged_decode_attn(*args, _stream()), "tlf_paged_decode_attn")
    else:
        assert plan.dtype == torch.int32 and plan.device == q.device
        check(lib.tlf_paged_decode_attn_planned(*args, plan.data_ptr(), _stream()), "tlf_paged_decode_attn_planned")
    return out


# ------------------------------------------------------------------ a4
def varlen_prefill_attention(q, k, v, cu_seqlens_q, cu_seqlens_k, max_seqlen_q, scale,
                             block_tables=None, k_scale=None, v_scale=None):
    """``q [Sq, Hq, Dh]``; ``k``/``v`` packed ``[Sk, Hkv, Dh]`` or the paged caches with ``block_tables``."""
    lib = _lib.load()
    _need(q, BF16, "q"); _need(cu_seqlens_q, torch.int32, "cu_seqlens_q")
    _need(cu_seqlens_k, torch.int32, "cu_seqlens_k")
    Sq, Hq, Dh = q.shape
    assert q.stride(2) == 1 and q.stride(1) == Dh
    out = torch.empty(Sq, Hq * Dh, dtype=BF16, device=q.device)
    nseq = cu_seqlens_q.numel() - 1
    if block_tables is None:
        _need(k, BF16, "k"); _need(v, BF16, "v")
        Hkv = k.shape[1]
        assert k.stride(2) == 1 and k.stride(1) == Dh and v.stride(2) == 1 and v.stride(1) == Dh
        ks, vs, bs, nblk, kvd = k.stride(0), v.stride(0), 0, 0, KV_BF16
        btp, bts = None, 0
    else:
        _need(block_tables, torch.int32, "block_tables")
        nblk, bs, Hkv, _ = k.shape
        assert k.is_contiguous() and v.is_contiguous()
        ks = vs = Hkv * Dh
        kvd = kv_dtype_code(k)
        btp, bts = block_tables.data_ptr(), block_tables.stride(0)
    check(lib.tlf_varlen_prefill_attn(
        q.data_ptr(), q.stride(0), k.data_ptr(), ks, v.data_ptr(), vs, kvd,
        k_scale.data_ptr() if k_scale is not None else None,
        v_scale.data_ptr() if v_scale is not None else None,
        cu_seqlens_q.data_ptr(), cu_seqlens_k.data_ptr(), btp, bts, out.data_ptr(), nseq,
        int(max_seqlen_q), Hq, Hkv, Dh, bs, nblk, float(scale), _stream()), "tlf_varlen_prefill_attn")
    return out


# ------------------------------------------------------------------ hybrid decoders
def _dt(t: torch.Tensor) -> int:
    if t.dtype == BF16:
        return DT_BF16
    if t.dtype == torch.float32:
        return DT_F32
    raise _lib.TlfError(f"unsupported dtype {t.dtype}")


def _opt(t):
    return t.data_ptr() if t is not None else None


class Deferred:
    """A bf16 projection ``[M, N]`` that may still be partial sums in the GEMM workspace (``splits > 1``): the very next
    kernels that read it add them up.  ``rows()`` is the plain tensor."""
    __slots__ = ("y", "partials", "splits", "scale", "shape", "dtype", "device")

    def __init__(self, y, partials, splits, scale):
        self.y, self.partials, self.splits, self.scale = y, partials, splits, scale
        self.shape, self.dtype, self.device = y.shape, y.dtype, y.device

    def rows(self):
        assert self.splits == 1
        return self.y


def linear_deferred(x, w, scale=None) -> Deferred:
    """``linear`` (``w`` bf16) or ``w8a16_linear`` (``w`` packed int8, ``scale``) without the kernel that adds partial sums."""
    import ctypes
    lib = _lib.load()
    if scale is not None:
        w = _packed(w)
        _need(scale, torch.float32, "scale")
    else:
        _need(w, BF16, "w")
        assert w.is_contiguous()
    _need(x, BF16, "x")
    assert x.dim() == 2 and x.stride(1) == 1
    (M, K), N = x.shape, w.shape[0]
    assert w.shape[1] == K
    y = torch.empty(M, N, dtype=BF16, device=x.device)
    ws = _workspace(lib.tlf_w8a16_gemm_workspace_bytes(M, N, K), x.device, "gemm")
    splits = ctypes.c_int32(1)
    check(lib.tlf_gemm_deferred(x.data_ptr(), x.stride(0), w.data_ptr(), _opt(scale), y.data_ptr(), M, N, K, ws.data_ptr(),
                                ws.numel(), ctypes.addressof(splits), _stream()), "tlf_gemm_deferred")
    return Deferred(y, ws, splits.value, scale)


def _source(y):
    """(row tensor, row stride, partials, splits, scale) of a tensor or a ``Deferred``."""
    if isinstance(y, Deferred):
        return y.y.data_ptr(), y.y.stride(0), y.partials.data_ptr(), y.splits, _opt(y.scale)
    assert y.stride(1) == 1
    return y.data_ptr(), y.stride(0), None, 1, None


def group_rms_norm_add(y, y_bias, w_post, x, w_next, groups, eps):
    """In place ``x += norm(y + y_bias) * w_post`` (``x`` fp32 ``[N, W]``), then ``norm(x) * w_next`` in y's dtype."""
    lib = _lib.load()
    assert y.dtype == w_post.dtype
    _need(x, torch.float32, "x"); _need(w_next, y.dtype, "w_next")
    rows, width = x.shape
    assert y.shape[0] == rows and y.shape[1] >= width and x.is_contiguous()
    assert w_post.numel() == width and w_next.numel() == width and (y_bias is None or y_bias.numel() == width)
    h = torch.empty(rows, width, dtype=y.dtype, device=x.device)
    check(lib.tlf_group_rmsnorm_add(*_source(y), _opt(y_bias), w_post.data_ptr(), x.data_ptr(),
                                    w_next.data_ptr(), h.data_ptr(), rows, width, groups, float(eps), _dt(y), _stream()),
          "tlf_group_rmsnorm_add")
    return h


def embed_group_rms_norm(ids, table, w_next, groups, eps, w_offset=0.0):
    """``x = table[ids]`` in fp32 and ``norm(x) * (w_next + w_offset)`` in the table's dtype."""
    lib = _lib.load()
    _need(ids, torch.int64, "ids"); _need(table, w_next.dtype, "table")
    assert ids.is_contiguous() and table.is_contiguous()
    rows, (vocab, width) = ids.numel(), table.shape
    x = torch.empty(rows, width, dtype=torch.float32, device=table.device)
    h = torch.empty(rows, width, dtype=table.dtype, device=table.device)
    check(lib.tlf_embed_group_rmsnorm(ids.data_ptr(), table.data_ptr(), vocab, x.data_ptr(), w_next.data_ptr(),
                                      float(w_offset), h.data_ptr(), rows, width, groups, float(eps), _dt(table), _stream()),
          "tlf_embed_group_rmsnorm")
    return x, h


def attn_prep(proj, q_bias, k_bias, positions, cos_sin, rot_dims, slot_mapping, k_cache, v_cache, num_q_heads, head_dim, eps):
    """Biases, V store, interleaved RoPE, unit RMS, K store.  Returns ``(q [N, Hq, Dp], gate fp32 [N, Hq])``."""
    lib = _lib.load()
    assert proj.dtype == k_cache.dtype
    _need(positions, torch.int64, "positions"); _need(slot_mapping, torch.int32, "slot_mapping")
    n = proj.shape[0]
    pages, bs, hkv, dp = k_cache.shape
    assert positions.numel() == n and slot_mapping.numel() == n
    assert k_cache.is_contiguous() and v_cache.is_contiguous() and (rot_dims == 0 or cos_sin.shape[1] == rot_dims)
    q = torch.empty(n, num_q_heads, dp, dtype=proj.dtype, device=proj.device)
    gate = torch.empty(n, num_q_heads, dtype=torch.float32, device=proj.device)
    check(lib.tlf_attn_prep(*_source(proj), _opt(q_bias), _opt(k_bias), positions.data_ptr(),
                            _opt(cos_sin), cos_sin.shape[0] if cos_sin is not None else 0, rot_dims,
                            slot_mapping.data_ptr(), pages * bs, q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(),
                            gate.data_ptr(), n, num_q_heads, hkv, head_dim, dp, float(eps), _dt(proj), _stream()),
          "tlf_attn_prep")
    return q, gate


class PooledKV:
    """The paged caches of one windowed layer with pooled blocks, and the layer's constants."""
    __slots__ = ("k", "v", "pk", "pv", "head_dim", "pool", "window")

    def __init__(self, pages, block_size, kv_heads, head_dim, pool, window, dtype, device):
        dp = (head_dim + 31) // 32 * 32
        rows = -(-block_size // pool)
        self.k, self.v = torch.zeros(2, pages, block_size, kv_heads, dp, dtype=dtype, device=device)
        self.pk, self.pv = torch.zeros(2, pages, rows, kv_heads, dp, dtype=dtype, device=device)
        self.head_dim, self.pool, self.window = head_dim, pool, window

    @staticmethod
    def page_bytes(block_size, kv_heads, head_dim, pool, itemsize):
        return 2 * (block_size + -(-block_size // pool)) * kv_heads * ((head_dim + 31) // 32 * 32) * itemsize


def pool_blocks(kv: PooledKV, block_tables, cu_seqlens_q, seq_starts, first_seq, num_seqs, max_tokens):
    lib = _lib.load()
    pages, bs, hkv, _ = kv.k.shape
    assert block_tables.shape[0] >= first_seq + num_seqs and block_tables.stride(1) == 1
    check(lib.tlf_pool_blocks(kv.k.data_ptr(), kv.v.data_ptr(), kv.pk.data_ptr(), kv.pv.data_ptr(), block_tables.data_ptr(),
                              block_tables.stride(0), cu_seqlens_q.data_ptr(), seq_starts.data_ptr(), first_seq, num_seqs,
                              max_tokens, hkv, kv.head_dim, bs, kv.pool, kv.window, pages, _dt(kv.k), _stream()),
          "tlf_pool_blocks")


def pooled_attention_rows(q, score_bias, gate, kv: PooledKV, block_tables, positions, slot_mapping, scale, max_len,
                          out, row_seq=None, pool_new=False):
    """Rows of ``out`` ``[N, Hq * D]`` from ``q [N, Hq, Dp]``; see ``tlf_pooled_attn_rows``."""
    lib = _lib.load()
    _need(q, kv.k.dtype, "q"); _need(score_bias, q.dtype, "score_bias"); _need(gate, torch.float32, "gate")
    _need(block_tables, torch.int32, "block_tables"); _need(positions, torch.int64, "positions")
    n, hq, dp = q.shape
    pages, bs, hkv, _ = kv.k.shape
    assert q.is_contiguous() and gate.is_contiguous() and gate.numel() == n * hq and out.stride(1) == 1
    assert out.shape[0] == n and positions.numel() == n and slot_mapping.numel() == n and dp == kv.k.shape[3]
    assert row_seq is not None or block_tables.shape[0] >= n
    nbytes = lib.tlf_pooled_attn_rows_workspace_bytes(n, hq, hkv, kv.head_dim, kv.pool, kv.window, max_len)
    ws = _workspace(nbytes, q.device, "pooled_rows")
    check(lib.tlf_pooled_attn_rows(
        q.data_ptr(), score_bias.data_ptr(), gate.data_ptr(), kv.k.data_ptr(), kv.v.data_ptr(), kv.pk.data_ptr(),
        kv.pv.data_ptr(), block_tables.data_ptr(), block_tables.stride(0), positions.data_ptr(), slot_mapping.data_ptr(),
        _opt(row_seq), out.data_ptr(), out.stride(0), n, hq, hkv, kv.head_dim, bs, kv.pool, kv.window, max_len, pages,
        float(scale), int(pool_new), _dt(q), ws.data_ptr(), ws.numel(), _stream()), "tlf_pooled_attn_rows")
    return out


def pooled_attention_prefill(q, score_bias, gate, kv: PooledKV, block_tables, cu_seqlens_q, seq_starts, first_seq,
                             num_seqs, max_tokens, scale, out):
    """Portions of sequences ``first_seq ..`` on the matrix cores (bf16); rows indexed as in the step."""
    lib = _lib.load()
    _need(q, BF16, "q"); _need(score_bias, BF16, "score_bias"); _need(gate, torch.float32, "gate")
    n, hq, dp = q.shape
    pages, bs, hkv, _ = kv.k.shape
    assert q.is_contiguous() and gate.is_contiguous() and out.stride(1) == 1 and out.shape[0] == n
    check(lib.tlf_pooled_attn_prefill(
        q.data_ptr(), score_bias.data_ptr(), gate.data_ptr(), kv.k.data_ptr(), kv.v.data_ptr(), kv.pk.data_ptr(),
        kv.pv.data_ptr(), block_tables.data_ptr(), block_tables.stride(0), cu_seqlens_q.data_ptr(), seq_starts.data_ptr(),
        first_seq, num_seqs, max_tokens, out.data_ptr(), out.stride(0), hq, hkv, kv.head_dim, bs, kv.pool, kv.window,
        pages, float(scale), _stream()), "tlf_pooled_attn_prefill")
    return out


def gla_decode(proj, a2, a2_bias, norm_weight, state, state_slots, positions, tau, eps, out):
    """One token per row of ``proj``; ``state`` fp32 ``[slots, H, dk, dv]`` updated in place."""
    lib = _lib.load()
    assert proj.dtype == a2.dtype
    _need(state, torch.float32, "state"); _need(state_slots, torch.int32, "state_slots")
    slots, heads, dk, dv = state.shape
    rows = proj.shape[0]
    assert out.stride(1) == 1 and out.shape[0] == rows and state.is_contiguous()
    assert a2.is_contiguous() and a2.shape[0] == heads * dk and state_slots.numel() >= rows and positions.numel() == rows
    check(lib.tlf_gla_decode(*_source(proj), a2.data_ptr(), a2_bias.data_ptr(), norm_weight.data_ptr(),
                             state.data_ptr(), state_slots.data_ptr(), slots, positions.data_ptr(), out.data_ptr(),
                             out.stride(0), rows, heads, dk, dv, a2.shape[1], float(tau), dk ** -0.5, float(eps),
                             _dt(proj), _stream()), "tlf_gla_decode")
    return out


def gla_portions(proj, a2, a2_bias, norm_weight, state, state_slots, seq_starts, chunk_rows, chunk_lens, cu_chunks,
                 first_seq, num_seqs, tau, eps, out):
    """Portions of sequences ``first_seq ..``; ``proj`` / ``out`` begin at the first portion's row."""
    lib = _lib.load()
    _need(proj, a2.dtype, "proj"); _need(state, torch.float32, "state"); _need(state_slots, torch.int32, "state_slots")
    slots, heads, dk, dv = state.shape
    rows, chunks = proj.shape[0], chunk_rows.numel()
    assert proj.stride(1) == 1 and out.stride(1) == 1 and out.shape[0] == rows and state.is_contiguous()
    assert a2.is_contiguous() and a2.shape[0] == heads * dk and cu_chunks.numel() == num_seqs + 1
    assert state_slots.numel() >= first_seq + num_seqs and chunk_lens.numel() == chunks
    ws = _workspace(lib.tlf_gla_portions_workspace_bytes(rows, chunks, num_seqs, heads, dk, dv), proj.device, "gla")
    check(lib.tlf_gla_portions(
        proj.data_ptr(), proj.stride(0), a2.data_ptr(), a2_bias.data_ptr(), norm_weight.data_ptr(), state.data_ptr(),
        state_slots.data_ptr(), slots, seq_starts.data_ptr(), chunk_rows.data_ptr(), chunk_lens.data_ptr(),
        cu_chunks.data_ptr(), chunks, first_seq, num_seqs, out.data_ptr(), out.stride(0), rows, heads, dk, dv,
        a2.shape[1], float(tau), dk ** -0.5, float(eps), _dt(proj), ws.data_ptr(), ws.numel(), _stream()),
        "tlf_gla_portions")
    return out


def residual_rms_norm(y, x, mult, w_next, w_offset, eps, extra=None, extra_rows=None):
    """In place ``x += mult * (y + sum of the rows extra[extra_rows])`` (``x`` fp32 ``[N, W]``, ``extra_rows`` int32
    ``[N, top]``), then ``x / rms(x) * (w_next + w_offset)`` in y's dtype."""
    lib = _lib.load()
    _need(x, torch.float32, "x"); _need(w_next, y.dtype, "w_next")
    rows, width = x.shape
    assert y.shape[0] == rows and y.shape[1] >= width and x.is_contiguous() and w_next.numel() == width
    top, stride = 0, 0
    if extra is not None:
        _need(extra, y.dtype, "extra"); _need(extra_rows, torch.int32, "extra_rows")
        assert extra.stride(1) == 1 and extra_rows.is_contiguous() and extra_rows.shape[0] == rows
        top, stride = extra_rows.shape[1], extra.stride(0)
    h = torch.empty(rows, width, dtype=y.dtype, device=x.device)
    check(lib.tlf_residual_rmsnorm(*_source(y), _opt(extra), stride, _opt(extra_rows), top, float(mult), x.data_ptr(),
                                   w_next.data_ptr(), float(w_offset), h.data_ptr(), rows, width, float(eps), _dt(y),
                                   _stream()), "tlf_residual_rmsnorm")
    return h


def embed_layer_norm(ids, table, w_next, b_next, eps, out_scale=1.0):
    """``x = table[ids]`` in fp32 and ``layer_norm(x) * out_scale`` in the table's dtype."""
    lib = _lib.load()
    _need(ids, torch.int64, "ids"); _need(table, w_next.dtype, "table"); _need(b_next, w_next.dtype, "b_next")
    assert ids.is_contiguous() and table.is_contiguous()
    rows, (vocab, width) = ids.numel(), table.shape
    assert w_next.numel() == width and b_next.numel() == width
    x = torch.empty(rows, width, dtype=torch.float32, device=table.device)
    h = torch.empty(rows, width, dtype=table.dtype, device=table.device)
    check(lib.tlf_embed_layernorm(ids.data_ptr(), table.data_ptr(), vocab, x.data_ptr(), w_next.data_ptr(), b_next.data_ptr(),
                                  float(out_scale), h.data_ptr(), rows, width, float(eps), _dt(table), _stream()),
          "tlf_embed_layernorm")
    return x, h


def residual_layer_norm(y, x, w_next, b_next, eps, out_scale=1.0, extra=None, extra_rows=None, extra_weights=None, own=None):
    """In place ``x += y + sum of extra_weights * extra[extra_rows]`` (``x`` fp32 ``[N, W]``, ``y`` may be None, ``extra_rows``
    int32 ``[N, top]``, a negative one stands for the row of ``own``), then ``layer_norm(x) * out_scale`` in w_next's dtype."""
    lib = _lib.load()
    _need(x, torch.float32, "x"); _need(w_next, None, "w_next"); _need(b_next, w_next.dtype, "b_next")
    rows, width = x.shape
    assert x.is_contiguous() and w_next.numel() == width and b_next.numel() == width
    assert y is None or (y.shape[0] == rows and y.shape[1] >= width and y.dtype == w_next.dtype)
    top, stride, own_stride = 0, 0, 0
    if extra is not None:
        _need(extra, w_next.dtype, "extra"); _need(extra_rows, torch.int32, "extra_rows"); _need(own, w_next.dtype, "own")
        assert extra.stride(1) == 1 and extra_rows.is_contiguous() and extra_rows.shape[0] == rows
        assert own.shape[0] == rows and own.shape[1] >= width and own.stride(1) == 1
        if extra_weights is not None:
            _need(extra_weights, torch.float32, "extra_weights")
            assert extra_weights.is_contiguous() and extra_weights.shape == extra_rows.shape
        top, stride, own_stride = extra_rows.shape[1], extra.stride(0), own.stride(0)
    h = torch.empty(rows, width, dtype=w_next.dtype, device=x.device)
    check(lib.tlf_residual_layernorm(*(_source(y) if y is not None else (None, 0, None, 1, None)), _opt(extra), stride,
                                     _opt(extra_rows), _opt(extra_weights), top, _opt(own), own_stride, x.data_ptr(),
                                     w_next.data_ptr(), b_next.data_ptr(), float(out_scale), h.data_ptr(), rows, width,
                                     float(eps), _dt(w_next), _stream()), "tlf_residual_layernorm")
    return h


class LatentShape:
    """Sizes of a latent-attention layer and of the padded rows its kernels read (``include/tlf_hip.h``)."""
    __slots__ = ("heads", "dim", "rot", "rank", "vdim", "da", "ta", "ra", "va", "dq", "lp", "rp")

    def __init__(self, heads, dim, rot, rank, vdim):
        up = lambda v, m: -(-v // m) * m
        self.heads, self.dim, self.rot, self.rank, self.vdim = heads, dim, rot, rank, vdim
        self.da, self.ta, self.ra, self.va = up(dim, 8), up(rot, 8), up(rank, 8), up(vdim, 8)
        self.dq, self.lp, self.rp = up(self.da + self.ta, 32), up(self.ra + self.ta, 64), up(self.ra, 32)

    @property
    def sizes(self):
        return self.heads, self.dim, self.rot, self.rank, self.vdim


def latent_prep(proj, latent_col, norm_weight, positions, cos_sin, slot_mapping, cache, shape: LatentShape, eps):
    """Rotated queries ``[N, H, Dq]``; the normed latent and the rotated key part go to ``cache [pages, bs, Lp]``."""
    q = _latent_queries(proj, shape)
    _latent_prep(proj, positions, cos_sin, shape, eps, False, q=q, cache=cache, latent_col=latent_col, norm=norm_weight, slot_mapping=slot_mapping)
    return q


def latent_prep_queries(proj, positions, cos_sin, shape: LatentShape, halves: bool):
    """Rotated queries ``[N, H, Dq]`` from rows of their own."""
    q = _latent_queries(proj, shape)
    _latent_prep(proj, positions, cos_sin, shape, 1.0, halves, q=q)
    return q


def latent_prep_down(proj, latent_col, norm_weight, positions, cos_sin, slot_mapping, cache, shape: LatentShape, eps, halves: bool,
                     cq_col=0, cq_norm=None, gate_col=None):
    """The latent and the rotated key into the cache; ``(normed query latent or None, gates fp32 [N, H] or None)``: the columns
    from ``cq_col`` on (padded with zeros to a multiple of 64) and sigmoids of those from ``gate_col`` on."""
    n, dev = proj.shape[0], cache.device
    cq = torch.empty(n, -(-cq_norm.numel() // 64) * 64, dtype=cache.dtype, device=dev) if cq_norm is not None else None
    gate = torch.empty(n, shape.heads, dtype=torch.float32, device=dev) if gate_col is not None else None
    _latent_prep(proj, positions, cos_sin, shape, eps, halves, cache=cache, latent_col=latent_col, norm=norm_weight,
                 slot_mapping=slot_mapping, cq_col=cq_col, cq_norm=cq_norm, cq=cq, gate_col=gate_col or 0, gate=gate)
    return cq, gate


def _latent_queries(proj, shape):
    return torch.empty(proj.shape[0], shape.heads, shape.dq, dtype=proj.dtype, device=proj.device)


def _latent_prep(proj, positions, cos_sin, shape, eps, halves, q=None, cache=None, latent_col=0, norm=None, slot_mapping=None,
                 cq_col=0, cq_norm=None, cq=None, gate_col=0, gate=None):
    lib = _lib.load()
    n = proj.shape[0]
    _need(positions, torch.int64, "positions")
    assert positions.numel() == n and (cos_sin is None or cos_sin.shape[1] == shape.rot)
    if cache is not None:
        _need(slot_mapping, torch.int32, "slot_mapping")
        assert proj.dtype == cache.dtype == norm.dtype and cache.is_contiguous() and cache.shape[2] == shape.lp
        assert slot_mapping.numel() == n and norm.numel() == shape.rank
    assert cq_norm is None or cq_norm.dtype == proj.dtype
    check(lib.tlf_latent_prep(*_source(proj), latent_col, _opt(norm), positions.data_ptr(), _opt(cos_sin),
                              cos_sin.shape[0] if cos_sin is not None else 0, int(halves), _opt(slot_mapping),
                              cache.shape[0] * cache.shape[1] if cache is not None else 0, _opt(q), _opt(cache), cq_col,
                              cq_norm.numel() if cq_norm is not None else 0, _opt(cq_norm), _opt(cq), cq.shape[1] if cq is not None else 0,
                              gate_col, _opt(gate), n, *shape.sizes, float(eps), _dt(proj), _stream()), "tlf_latent_prep")


def head_gemm(x, w, n_main=0, k_main=0):
    """``y[row, head] = w[head] @ x[row, head]``: ``x [N, H, K]``, ``w [H, Nout, K]`` -> ``[N, H, Nout]``."""
    lib = _lib.load()
    _need(x, w.dtype, "x")
    rows, heads, K = x.shape
    assert x.is_contiguous() and w.is_contiguous() and w.shape[0] == heads and w.shape[2] == K
    y = torch.empty(rows, heads, w.shape[1], dtype=x.dtype, device=x.device)
    check(lib.tlf_head_gemm(x.data_ptr(), w.data_ptr(), y.data_ptr(), rows, heads, w.shape[1], K, n_main, k_main, _dt(x),
                            _stream()), "tlf_head_gemm")
    return y


def latent_attn_supported(shape: LatentShape) -> bool:
    return bool(_lib.load().tlf_latent_attn_supported(*shape.sizes))


def latent_prefill_supported(shape: LatentShape) -> bool:
    return bool(_lib.load().tlf_latent_prefill_supported(*shape.sizes))


def latent_rows(q, cache, block_tables, positions, slot_mapping, row_seq, window, scale, shape: LatentShape):
    """Absorbed attention of any rows; ``q [N, H, Lp]``.  Returns ``(part, ml)`` for ``latent_values``."""
    lib = _lib.load()
    _need(q, cache.dtype, "q"); _need(block_tables, torch.int32, "block_tables"); _need(positions, torch.int64, "positions")
    rows = q.shape[0]
    assert q.is_contiguous() and q.shape[1:] == (shape.heads, shape.lp) and block_tables.stride(1) == 1
    assert positions.numel() == rows and slot_mapping.numel() == rows and (row_seq is not None or block_tables.shape[0] >= rows)
    part = torch.empty(rows, shape.heads, shape.rp, dtype=torch.float32, device=q.device)
    ml = torch.empty(rows, shape.heads, 2, dtype=torch.float32, device=q.device)
    step = 32768                                     # rows per launch (grid limit)
    for lo in range(0, rows, step):
        n = min(step, rows - lo)
        assert row_seq is not None or lo == 0
        check(lib.tlf_latent_rows(q[lo:].data_ptr(), cache.data_ptr(), block_tables.data_ptr(), block_tables.stride(0),
                                  positions[lo:].data_ptr(), slot_mapping[lo:].data_ptr(),
                                  row_seq[lo:].data_ptr() if row_seq is not None else None, part[lo:].data_ptr(),
                                  ml[lo:].data_ptr(), n, *shape.sizes, cache.shape[1], window, cache.shape[0],
                                  float(scale), _dt(q), _stream()), "tlf_latent_rows")
    return part, ml


class LatentBatch:
    """Sequences that attend in the latent space in one call: ``num_seqs`` single rows (``positions``, ``slot_mapping``), or
    portions of at most ``max_tokens`` rows (``cu_seqlens_q``, ``seq_starts``, ``row_seq`` of their rows, the step's row of
    the first one)."""
    __slots__ = ("positions", "slot_mapping", "cu_seqlens_q", "seq_starts", "row_seq", "first_seq", "first_row", "num_seqs",
                 "max_tokens")

    def __init__(self, num_seqs, max_tokens=1, positions=None, slot_mapping=None, cu_seqlens_q=None, seq_starts=None,
                 row_seq=None, first_seq=0, first_row=0):
        self.num_seqs, self.max_tokens, self.positions, self.slot_mapping = num_seqs, max_tokens, positions, slot_mapping
        self.cu_seqlens_q, self.seq_starts, self.row_seq = cu_seqlens_q, seq_starts, row_seq
        self.first_seq, self.first_row = first_seq, first_row

    @property
    def where(self):
        return (_opt(self.positions), _opt(self.slot_mapping), _opt(self.cu_seqlens_q), _opt(self.seq_starts), self.first_seq,
                self.first_row, self.num_seqs, self.max_tokens)

    def layout(self, heads, row_size):
        """int32 values of a plan, pieces, units of a piece."""
        import ctypes
        out = (ctypes.c_int32 * 3)()
        check(_lib.load().tlf_latent_attn_layout(self.num_seqs, self.max_tokens, heads, row_size, ctypes.addressof(out)),
              "tlf_latent_attn_layout")
        return tuple(out)


def latent_plan(batch: LatentBatch, heads, row_size, window):
    """How a batch's keys are cut into pieces for the workgroups: once per step and window, for all layers of these sizes."""
    device = (batch.positions if batch.cu_seqlens_q is None else batch.cu_seqlens_q).device
    plan = torch.empty(batch.layout(heads, row_size)[0], dtype=torch.int32, device=device)
    check(_lib.load().tlf_latent_attn_plan(*batch.where, heads, row_size, window, plan.data_ptr(), _stream()), "tlf_latent_attn_plan")
    return plan


def latent_attention(q, cache, block_tables, window, scale, shape: LatentShape, batch: LatentBatch, plan):
    """Absorbed attention on the matrix cores; ``q`` holds the batch's rows.  Returns ``(part, ml)`` for ``latent_values``."""
    lib = _lib.load()
    _need(q, BF16, "q"); _need(block_tables, torch.int32, "block_tables"); _need(plan, torch.int32, "plan")
    assert q.is_contiguous() and q.shape[1:] == (shape.heads, shape.lp) and block_tables.stride(1) == 1
    assert block_tables.shape[0] >= batch.first_seq + batch.num_seqs and cache.is_contiguous() and cache.dtype == BF16
    if batch.cu_seqlens_q is None:
        assert q.shape[0] == batch.num_seqs <= min(batch.positions.numel(), batch.slot_mapping.numel())
    need, pieces, units = batch.layout(shape.heads, shape.lp)
    assert plan.numel() >= need
    part = torch.empty(pieces, units, shape.rp, dtype=torch.float32, device=q.device)
    ml = torch.empty(pieces, units, 2, dtype=torch.float32, device=q.device)
    check(lib.tlf_latent_attn(q.data_ptr(), cache.data_ptr(), block_tables.data_ptr(), block_tables.stride(0), *batch.where,
                              plan.data_ptr(), part.data_ptr(), ml.data_ptr(), *shape.sizes, cache.shape[1], window,
                              cache.shape[0], float(scale), _stream()), "tlf_latent_attn")
    return part, ml


def _check_gate(gate, rows, shape):
    if gate is not None:
        _need(gate, torch.float32, "gate")
        assert gate.is_contiguous() and gate.shape == (rows, shape.heads)


def latent_values(part, ml, uv, out, shape: LatentShape, batch: LatentBatch | None = None, plan=None, gate=None):
    """``out [N, >= H * vdim]`` from the pieces' mixed latents; ``uv [H, vdim rounded up to 16, Rp]``, ``gate`` fp32 ``[N, H]``."""
    lib = _lib.load()
    rows = out.shape[0]
    assert out.stride(1) == 1 and out.dtype == uv.dtype and part.is_contiguous() and uv.is_contiguous()
    assert plan is not None or part.shape[0] == rows
    _check_gate(gate, rows, shape)
    where = (None, None, 0, 0, 0, 0)
    if plan is not None:
        where = (_opt(batch.cu_seqlens_q), _opt(batch.row_seq), batch.first_seq, batch.first_row, batch.num_seqs, batch.max_tokens)
        assert batch.row_seq is None or batch.row_seq.numel() >= rows
    check(lib.tlf_latent_values(part.data_ptr(), ml.data_ptr(), _opt(plan), *where, uv.data_ptr(), _opt(gate), out.data_ptr(),
                                out.stride(0), rows, *shape.sizes, _dt(uv), _stream()), "tlf_latent_values")


def latent_gather(cache, block_tables, cu_seqlens_q, seq_starts, kv_offsets, kv_rows, first_seq, num_seqs, max_rows, window):
    """Cache rows of the keys that the portions see, dense: ``[kv_rows, Lp]``."""
    lib = _lib.load()
    _need(kv_offsets, torch.int32, "kv_offsets")
    assert cache.dtype == BF16 and kv_offsets.is_contiguous() and kv_offsets.numel() == num_seqs + 1
    out = torch.empty(kv_rows, cache.shape[2], dtype=cache.dtype, device=cache.device)
    check(lib.tlf_latent_gather(cache.data_ptr(), block_tables.data_ptr(), block_tables.stride(0), cu_seqlens_q.data_ptr(),
                                seq_starts.data_ptr(), kv_offsets.data_ptr(), first_seq, num_seqs, max_rows, out.data_ptr(),
                                cache.shape[2], cache.shape[1], window, cache.shape[0], _stream()), "tlf_latent_gather")
    return out


def latent_prefill(q, expanded, latents, cu_seqlens_q, seq_starts, kv_offsets, first_seq, num_seqs, max_tokens, window, scale,
                   shape: LatentShape, out, gate=None):
    """Portions from expanded keys and values; ``q``, ``out`` and ``gate`` are indexed by the step's rows."""
    lib = _lib.load()
    _check_gate(gate, q.shape[0], shape)
    _need(q, BF16, "q"); _need(expanded, BF16, "expanded"); _need(latents, BF16, "latents")
    assert q.is_contiguous() and q.shape[1:] == (shape.heads, shape.dq) and out.stride(1) == 1
    assert expanded.stride(1) == 1 and latents.is_contiguous() and latents.shape[1] == shape.lp
    check(lib.tlf_latent_prefill(q.data_ptr(), expanded.data_ptr(), expanded.stride(0), latents.data_ptr(),
                                 cu_seqlens_q.data_ptr(), seq_starts.data_ptr(), kv_offsets.data_ptr(), first_seq, num_seqs,
                                 max_tokens, _opt(gate), out.data_ptr(), out.stride(0), *shape.sizes, window, float(scale),
                                 _stream()), "tlf_latent_prefill")
    return out


# ------------------------------------------------------------------ grouped-query attention with a sink
class SinkKV:
    """The paged, head-major caches of one layer: ``k [pages, G, block, Dp]``, ``v [pages, G, block, Vp]``."""
    __slots__ = ("k", "v", "dim", "vdim")

    def __init__(self, pages, block_size, kv_heads, dim, vdim, dtype, device):
        self.k = torch.zeros(pages, kv_heads, block_size, self.padded(dim), dtype=dtype, device=device)
        self.v = torch.zeros(pages, kv_heads, block_size, self.padded(vdim), dtype=dtype, device=device)
        self.dim, self.vdim = dim, vdim

    @staticmethod
    def padded(dim):
        return -(-dim // 32) * 32

    @staticmethod
    def page_bytes(block_size, kv_heads, dim, vdim, itemsize):
        return block_size * kv_heads * (SinkKV.padded(dim) + SinkKV.padded(vdim)) * itemsize


def sink_prep(proj, kv: SinkKV, heads, positions, slot_mapping, eps, scale=1.0, cap=None, bias=None, conv=None, ring=None, state_slots=None,
              row_seq=None, cu_seqlens_q=None, q_norm=None, k_norm=None, cos_sin=None, rot_dims=0, q_mult=None):
    """Projection rows ``[q | k | v | gate]`` -> ``(q [N, H, Dp], gate rows [N, >= H * vdim])``; keys and values go to the
    caches, the score's constants into q.  See ``tlf_sink_prep``; ``proj`` may be ``Deferred`` when every row is a sequence of its own."""
    lib = _lib.load()
    dt = kv.k.dtype
    assert proj.dtype == dt
    _need(positions, torch.int64, "positions"); _need(slot_mapping, torch.int32, "slot_mapping")
    n = proj.shape[0]
    pages, G, bs, dp = kv.k.shape
    channels = (heads + G) * kv.dim + G * kv.vdim
    assert positions.numel() == n and slot_mapping.numel() == n and proj.shape[1] >= channels + heads * kv.vdim
    for t, count in ((bias, channels), (q_norm, kv.dim), (k_norm, kv.dim)):
        assert t is None or (t.dtype == dt and t.numel() == count and t.is_contiguous())
    taps = 0
    if conv is not None:
        taps = conv.shape[0]
        assert conv.dtype == ring.dtype == dt and conv.is_contiguous() and ring.is_contiguous()
        assert conv.shape == (taps, channels) and ring.shape[1:] == (taps, channels)
        _need(state_slots, torch.int32, "state_slots")
        assert row_seq is not None or state_slots.numel() >= n
    if row_seq is not None:
        _need(row_seq, torch.int32, "row_seq"); _need(cu_seqlens_q, torch.int32, "cu_seqlens_q")
        assert row_seq.numel() == n
    tables = [t for t in (cos_sin, q_mult) if t is not None]
    for t in tables:
        _need(t, torch.float32, "table")
        assert t.is_contiguous() and t.shape[0] == tables[0].shape[0]
    assert rot_dims == 0 or cos_sin.shape[1] == rot_dims
    q = torch.empty(n, heads, dp, dtype=dt, device=kv.k.device)
    gate = out = None
    if isinstance(proj, Deferred):
        gate = out = torch.empty(n, heads * kv.vdim, dtype=dt, device=kv.k.device)
    else:
        gate = proj[:, channels:]
    check(lib.tlf_sink_prep(*_source(proj), _opt(bias), _opt(conv), taps, _opt(ring), _opt(state_slots),
                            ring.shape[0] if ring is not None else 0, _opt(row_seq), _opt(cu_seqlens_q), _opt(q_norm),
                            _opt(k_norm), positions.data_ptr(), _opt(cos_sin), _opt(q_mult),
                            tables[0].shape[0] if tables else 1 << 30, rot_dims, slot_mapping.data_ptr(), q.data_ptr(),
                            kv.k.data_ptr(), kv.v.data_ptr(), _opt(out), n, heads, G, kv.dim, kv.vdim, bs, pages, float(eps),
                            float(scale), float(cap or 0), _dt(kv.k), _stream()), "tlf_sink_prep")
    return q, gate


def conv_tail(proj, ring, state_slots, cu_seqlens_q, seq_starts, first_seq, num_seqs):
    """The last projected rows of the portions of sequences ``first_seq ..`` into ``ring [slots, taps, channels]``."""
    _need(proj, ring.dtype, "proj"); _need(state_slots, torch.int32, "state_slots")
    slots, taps, channels = ring.shape
    assert proj.stride(1) == 1 and proj.shape[1] >= channels and ring.is_contiguous()
    assert state_slots.numel() >= first_seq + num_seqs and cu_seqlens_q.numel() > first_seq + num_seqs
    check(_lib.load().tlf_conv_tail(proj.data_ptr(), proj.stride(0), ring.data_ptr(), state_slots.data_ptr(), slots,
                                    cu_seqlens_q.data_ptr(), seq_starts.data_ptr(), first_seq, num_seqs, taps, channels,
                                    _dt(ring), _stream()), "tlf_conv_tail")


def sink_attention_rows(q, kv: SinkKV, block_tables, positions, slot_mapping, sink, gate, cap, max_len, out, row_seq=None):
    """Row by row: ``q [N, H, Dp]`` as from ``sink_prep`` -> ``out [N, H * vdim]``; ``row_seq`` None: row r is sequence r."""
    lib = _lib.load()
    _need(q, kv.k.dtype, "q"); _need(block_tables, torch.int32, "block_tables"); _need(positions, torch.int64, "positions")
    n, heads, dp = q.shape
    pages, G, bs, _ = kv.k.shape
    assert q.is_contiguous() and dp == kv.k.shape[3] and out.stride(1) == 1 and out.shape[0] == n and out.dtype == q.dtype
    assert gate is None or (gate.dtype == q.dtype and gate.shape[0] == n and gate.stride(1) == 1)
    assert sink is None or (sink.dtype == q.dtype and sink.numel() == heads)
    assert positions.numel() == n and slot_mapping.numel() == n and block_tables.stride(1) == 1
    assert row_seq.numel() == n if row_seq is not None else block_tables.shape[0] >= n
    max_len = min(max_len, block_tables.shape[1] * bs)
    step = 32768                                     # rows per launch (grid limit)
    for lo in range(0, n, step):
        m = min(step, n - lo)
        assert row_seq is not None or lo == 0
        nbytes = lib.tlf_sink_attn_rows_workspace_bytes(m, heads, G, kv.dim, kv.vdim, max_len, _dt(q))
        ws = _workspace(nbytes, q.device, "sink_rows")
        check(lib.tlf_sink_attn_rows(
            q[lo:].data_ptr(), kv.k.data_ptr(), kv.v.data_ptr(), block_tables.data_ptr(), block_tables.stride(0),
            positions[lo:].data_ptr(), slot_mapping[lo:].data_ptr(), row_seq[lo:].data_ptr() if row_seq is not None else None,
            _opt(sink), gate[lo:].data_ptr() if gate is not None else None, gate.stride(0) if gate is not None else 0,
            out[lo:].data_ptr(), out.stride(0), m, heads, G, kv.dim, kv.vdim, bs, max_len, pages, float(cap or 0),
            _dt(q), ws.data_ptr(), ws.numel(), _stream()), "tlf_sink_attn_rows")
    return out


def sink_prefill_supported(dim, vdim) -> bool:
    return bool(_lib.load().tlf_sink_attn_prefill_supported(dim, vdim))


def sink_attention_prefill(q, kv: SinkKV, block_tables, cu_seqlens_q, seq_starts, first_seq, num_seqs, max_tokens, sink, gate,
                           cap, out):
    """Portions of sequences ``first_seq ..`` on the matrix cores (bf16); rows indexed as in the step."""
    _need(q, BF16, "q"); _need(block_tables, torch.int32, "block_tables")
    n, heads, dp = q.shape
    pages, G, bs, _ = kv.k.shape
    assert q.is_contiguous() and dp == kv.k.shape[3] and kv.k.dtype == BF16 and out.stride(1) == 1 and out.shape[0] == n
    assert gate is None or (gate.dtype == BF16 and gate.shape[0] == n and gate.stride(1) == 1)
    assert sink is None or (sink.dtype == BF16 and sink.numel() == heads)
    assert block_tables.stride(1) == 1 and block_tables.shape[0] >= first_seq + num_seqs
    check(_lib.load().tlf_sink_attn_prefill(
        q.data_ptr(), kv.k.data_ptr(), kv.v.data_ptr(), block_tables.data_ptr(), block_tables.stride(0), cu_seqlens_q.data_ptr(),
        seq_starts.data_ptr(), first_seq, num_seqs, max_tokens, _opt(sink), _opt(gate), gate.stride(0) if gate is not None else 0,
        out.data_ptr(), out.stride(0), heads, G, kv.dim, kv.vdim, bs, pages, float(cap or 0), _stream()),
        "tlf_sink_attn_prefill")
    return out


# ------------------------------------------------------------------ post-norm and token shift
class ShiftArguments:
    """Token shift: ``mix [W]``, the rows before (``ring`` fp32 ``[slots, 2, W]``), and where a step's rows belong (``row_seq`` None:
    row r is the one row of sequence r)."""
    __slots__ = ("mix", "ring", "state_slots", "positions", "row_seq", "cu_seqlens_q")

    def __init__(self, mix, ring, state_slots, positions, row_seq=None, cu_seqlens_q=None):
        self.mix, self.ring, self.state_slots, self.positions = mix, ring, state_slots, positions
        self.row_seq, self.cu_seqlens_q = row_seq, cu_seqlens_q

    def pointers(self, rows, width, dtype):
        _need(self.ring, torch.float32, "ring"); _need(self.state_slots, torch.int32, "state_slots")
        _need(self.positions, torch.int64, "positions")
        assert self.mix.numel() == width and self.mix.dtype == dtype and self.ring.is_contiguous() and self.ring.shape[1:] == (2, width)
        assert self.positions.numel() == rows and (self.row_seq is not None or self.state_slots.numel() >= rows)
        assert self.row_seq is None or (self.row_seq.numel() == rows and self.cu_seqlens_q.dtype == torch.int32)
        return (self.mix.data_ptr(), self.ring.data_ptr(), self.ring.shape[0], self.state_slots.data_ptr(), _opt(self.row_seq),
                _opt(self.cu_seqlens_q), self.positions.data_ptr())


def post_rms_norm(y, x, alpha, layer_scale, w, eps, shift: ShiftArguments | None = None, w_next=None):
    """``x' = rms_norm(alpha x + layer_scale * y) * w`` (``x`` fp32 ``[N, W]``; in place unless portions are shifted) and in w's
    dtype its rows, shifted rows or ``rms_norm(x') * w_next``.  Returns ``(x', rows)``."""
    lib = _lib.load()
    _need(x, torch.float32, "x"); _need(w, y.dtype, "w"); _need(layer_scale, y.dtype, "layer_scale")
    rows, width = x.shape
    assert y.shape[0] == rows and y.shape[1] >= width and x.is_contiguous() and w.numel() == layer_scale.numel() == width
    assert w_next is None or (w_next.numel() == width and w_next.dtype == w.dtype)
    out = torch.empty_like(x) if shift is not None and shift.row_seq is not None else x
    plain = shift is None and w_next is None and w.dtype == torch.float32          # the rows are x' itself
    h = out if plain else torch.empty(rows, width, dtype=w.dtype, device=x.device)
    where = shift.pointers(rows, width, w.dtype) if shift is not None else (None, None, 0, None, None, None, None)
    check(lib.tlf_post_rmsnorm(*_source(y), layer_scale.data_ptr(), float(alpha), x.data_ptr(), w.data_ptr(), float(eps), out.data_ptr(),
                               *where, _opt(w_next), None if plain else h.data_ptr(), rows, width, _dt(w), _stream()), "tlf_post_rmsnorm")
    return out, h


def embed_shift(ids, table, embed_scale, shift: ShiftArguments):
    """``x = embed_scale * table[ids]`` in fp32 and its shifted rows in the table's dtype."""
    lib = _lib.load()
    _need(ids, torch.int64, "ids"); _need(table, None, "table")
    assert ids.is_contiguous() and table.is_contiguous()
    rows, (vocab, width) = ids.numel(), table.shape
    x = torch.empty(rows, width, dtype=torch.float32, device=table.device)
    h = torch.empty(rows, width, dtype=table.dtype, device=table.device)
    check(lib.tlf_embed_shift(ids.data_ptr(), table.data_ptr(), vocab, float(embed_scale), x.data_ptr(),
                              *shift.pointers(rows, width, table.dtype), h.data_ptr(), rows, width, _dt(table), _stream()), "tlf_embed_shift")
    return x, h


def rows_rms_norm(x, w, groups, eps, pad=1):
    """Rows of ``x [N, C]`` in ``groups`` equal parts, each divided by its root mean square, times ``w``; zero columns up to a multiple
    of ``pad``."""
    _need(x, w.dtype, "x")
    (rows, cols), dt = x.shape, x.dtype
    assert x.stride(1) == 1 and w.numel() == cols
    out = torch.empty(rows, -(-cols // pad) * pad, dtype=dt, device=x.device)
    check(_lib.load().tlf_rows_rmsnorm(x.data_ptr(), x.stride(0), w.data_ptr(), out.data_ptr(), out.stride(0), rows, cols, groups, float(eps),
                                       _dt(x), _stream()), "tlf_rows_rmsnorm")
    return out


# ------------------------------------------------------------------ attention whose heads mix their weights
def talk_prep(proj, kv: SinkKV, heads, positions, slot_mapping, q_norm, k_norm, temp, cos_sin, rot_dims, eps, scale):
    """Projection rows ``[q | k | v]`` -> ``q [N, H, Dp]`` with the score's constants; keys and values go to the caches."""
    lib = _lib.load()
    dt, n = kv.k.dtype, proj.shape[0]
    _need(positions, torch.int64, "positions"); _need(slot_mapping, torch.int32, "slot_mapping")
    pages, G, bs, dp = kv.k.shape
    assert proj.dtype == q_norm.dtype == k_norm.dtype == dt and (temp is None or (temp.dtype == dt and temp.numel() == heads))
    assert positions.numel() == n and slot_mapping.numel() == n and proj.shape[1] >= (heads + G) * kv.dim + G * kv.vdim
    assert q_norm.numel() == heads * kv.dim and k_norm.numel() == G * kv.dim
    assert rot_dims == 0 or (cos_sin.dtype == torch.float32 and cos_sin.is_contiguous() and cos_sin.shape[1] == rot_dims)
    q = torch.empty(n, heads, dp, dtype=dt, device=kv.k.device)
    check(lib.tlf_talk_prep(*_source(proj), q_norm.data_ptr(), k_norm.data_ptr(), _opt(temp), positions.data_ptr(), _opt(cos_sin),
                            cos_sin.shape[0] if cos_sin is not None else 0, rot_dims, slot_mapping.data_ptr(), q.data_ptr(),
                            kv.k.data_ptr(), kv.v.data_ptr(), n, heads, G, kv.dim, kv.vdim, bs, pages, float(eps), float(scale), _dt(kv.k),
                            _stream()), "tlf_talk_prep")
    return q


def talk_attention_rows(q, kv: SinkKV, block_tables, positions, slot_mapping, talk, max_len, out, row_seq=None):
    """Row by row: ``q [N, H, Dp]`` as from ``talk_prep`` -> ``out [N, H * vdim]``; ``row_seq`` None: row r is sequence r."""
    lib = _lib.load()
    _need(q, kv.k.dtype, "q"); _need(talk, q.dtype, "talk"); _need(block_tables, torch.int32, "block_tables")
    _need(positions, torch.int64, "positions")
    n, heads, dp = q.shape
    pages, G, bs, _ = kv.k.shape
    assert q.is_contiguous() and dp == kv.k.shape[3] and out.stride(1) == 1 and out.shape[0] == n and out.dtype == q.dtype
    assert talk.is_contiguous() and talk.shape == (heads, heads) and block_tables.stride(1) == 1
    assert positions.numel() == n and slot_mapping.numel() == n
    assert row_seq.numel() == n if row_seq is not None else block_tables.shape[0] >= n
    max_len = min(max_len, block_tables.shape[1] * bs)
    step = max(1, min(32768, (1 << 28) // (heads * -(-max_len // 64) * 64)))     # rows per launch: grid limit, a gigabyte of scores
    for lo in range(0, n, step):
        m = min(step, n - lo)
        tables = block_tables if row_seq is not None else block_tables[lo:]
        nbytes = lib.tlf_talk_attn_rows_workspace_bytes(m, heads, G, kv.dim, kv.vdim, max_len, _dt(q))
        ws = _workspace(nbytes, q.device, "talk_rows")
        check(lib.tlf_talk_attn_rows(
            q[lo:].data_ptr(), kv.k.data_ptr(), kv.v.data_ptr(), tables.data_ptr(), tables.stride(0), positions[lo:].data_ptr(),
            slot_mapping[lo:].data_ptr(), row_seq[lo:].data_ptr() if row_seq is not None else None, talk.data_ptr(), out[lo:].data_ptr(),
            out.stride(0), m, heads, G, kv.dim, kv.vdim, bs, max_len, pages, _dt(q), ws.data_ptr(), ws.numel(), _stream()),
            "tlf_talk_attn_rows")
    return out


def talk_prefill_supported(heads, kv_heads, dim, vdim) -> bool:
    return bool(_lib.load().tlf_talk_attn_prefill_supported(heads, kv_heads, dim, vdim))


def talk_attention_prefill(q, kv: SinkKV, block_tables, cu_seqlens_q, seq_starts, first_seq, num_seqs, max_tokens, talk, out):
    """Portions of sequences ``first_seq ..`` on the matrix cores (bf16); rows indexed as in the step."""
    _need(q, BF16, "q"); _need(talk, BF16, "talk"); _need(block_tables, torch.int32, "block_tables")
    n, heads, dp = q.shape
    pages, G, bs, _ = kv.k.shape
    assert q.is_contiguous() and dp == kv.k.shape[3] and kv.k.dtype == BF16 and out.stride(1) == 1 and out.shape[0] == n
    assert talk.is_contiguous() and talk.shape == (heads, heads)
    assert block_tables.stride(1) == 1 and block_tables.shape[0] >= first_seq + num_seqs
    stats = torch.empty(n, heads, dtype=torch.float32, device=q.device)
    check(_lib.load().tlf_talk_attn_prefill(
        q.data_ptr(), kv.k.data_ptr(), kv.v.data_ptr(), block_tables.data_ptr(), block_tables.stride(0), cu_seqlens_q.data_ptr(),
        seq_starts.data_ptr(), first_seq, num_seqs, max_tokens, talk.data_ptr(), stats.data_ptr(), out.data_ptr(), out.stride(0), heads, G, kv.dim, kv.vdim,
        bs, pages, _stream()), "tlf_talk_attn_prefill")
    return out


# ------------------------------------------------------------------ state-space layer
class SsdWeights:
    """``conv [taps, channels]``, ``conv_bias [channels]``, ``dt_bias``, ``A_log``, ``D [heads]``, all of one dtype."""
    __slots__ = ("conv", "conv_bias", "dt_bias", "A_log", "D")

    def __init__(self, conv, conv_bias, dt_bias, A_log, D):
        self.conv, self.conv_bias, self.dt_bias, self.A_log, self.D = conv, conv_bias, dt_bias, A_log, D

    def pointers(self, proj, ring, state, state_slots, groups):
        """Checked; the arguments from ``conv`` to ``num_slots`` and the sizes."""
        slots, heads, N, P = state.shape
        taps, channels = self.conv.shape
        _need(state, torch.float32, "state"); _need(state_slots, torch.int32, "state_slots")
        for t in (self.conv, self.conv_bias, self.dt_bias, self.A_log, self.D, ring):
            assert t.dtype == proj.dtype and t.is_contiguous()
        assert channels == heads * P + 2 * groups * N == self.conv_bias.numel() and self.dt_bias.numel() == self.A_log.numel() == self.D.numel() == heads
        assert state.is_contiguous() and ring.shape == (slots, taps, channels) and proj.shape[1] >= heads * P + channels + heads
        return ((self.conv.data_ptr(), self.conv_bias.data_ptr(), taps, self.dt_bias.data_ptr(), self.A_log.data_ptr(), self.D.data_ptr(),
                 ring.data_ptr(), state.data_ptr(), state_slots.data_ptr(), slots), (heads, P, N, groups))


def ssd_decode(proj, weights: SsdWeights, ring, state, state_slots, positions, groups, out):
    """One token per row of ``proj [N, z | x | B | C | dt]``; ``ring`` and ``state`` updated in place; ``out`` gated, not normed."""
    lib = _lib.load()
    rows = proj.shape[0]
    args, sizes = weights.pointers(proj, ring, state, state_slots, groups)
    assert out.stride(1) == 1 and out.shape[0] == rows and state_slots.numel() >= rows and positions.numel() == rows
    check(lib.tlf_ssd_decode(*_source(proj), *args, positions.data_ptr(), out.data_ptr(), out.stride(0), rows, *sizes, _dt(proj), _stream()),
          "tlf_ssd_decode")
    return out


def ssd_portions(proj, weights: SsdWeights, ring, state, state_slots, positions, row_seq, cu_seqlens_q, seq_starts, first_seq, num_seqs,
                 first_row, max_tokens, groups, out):
    """Portions of sequences ``first_seq ..``, whose rows begin at ``first_row`` of the step's; the ring is only read."""
    lib = _lib.load()
    rows = proj.shape[0] - first_row
    args, sizes = weights.pointers(proj, ring, state, state_slots, groups)
    _need(row_seq, torch.int32, "row_seq"); _need(cu_seqlens_q, torch.int32, "cu_seqlens_q")
    assert proj.stride(1) == 1 and out.stride(1) == 1 and out.shape[0] == proj.shape[0] == positions.numel() == row_seq.numel()
    assert state_slots.numel() >= first_seq + num_seqs and cu_seqlens_q.numel() > first_seq + num_seqs
    ws = _workspace(lib.tlf_ssd_portions_workspace_bytes(rows, num_seqs, max_tokens, *sizes, _dt(proj)), proj.device, "ssd")
    check(lib.tlf_ssd_portions(proj.data_ptr(), proj.stride(0), *args, positions.data_ptr(), row_seq.data_ptr(), cu_seqlens_q.data_ptr(),
                               seq_starts.data_ptr(), first_seq, num_seqs, first_row, max_tokens, out.data_ptr(), out.stride(0), rows, *sizes,
                               _dt(proj), ws.data_ptr(), ws.numel(), _stream()), "tlf_ssd_portions")
    return out


# ------------------------------------------------------------------ mixture of experts
def moe_logits(h, router):
    """Router logits of every row as fp32 partial sums ``[splits, N, experts rounded up to 16]``."""
    import ctypes
    if router.dtype == torch.float32:
        return f32_linear(h, router)[None]
    lib = _lib.load()
    _need(h, BF16, "h"); _need(router, BF16, "router")
    (M, K), N = h.shape, router.shape[0]
    assert h.stride(1) == 1 and router.is_contiguous() and router.shape[1] == K
    splits = ctypes.c_int32(1)
    nbytes = lib.tlf_gemm_f32_sums_bytes(M, N, K)
    sums = torch.empty(nbytes // 4, dtype=torch.float32, device=h.device)
    check(lib.tlf_gemm_f32_sums(h.data_ptr(), h.stride(0), router.data_ptr(), sums.data_ptr(), nbytes, M, N, K,
                                ctypes.addressof(splits), _stream()), "tlf_gemm_f32_sums")
    return sums.view(splits.value, M, N)


class ExpertRows:
    """The chosen experts ``ids`` / ``scores [N, top]`` and the rows (token, k) in expert order: ``row_of [N, top]``, ``src`` /
    ``weight`` per row, tiles of ``tile_rows`` rows."""
    __slots__ = ("ids", "scores", "row_of", "src", "weight", "tiles", "num_tiles", "tile_rows")


def moe_group(logits, experts, top, tile_rows, correction=None, identity=0) -> ExpertRows:
    """``logits``: partial sums as from ``moe_logits``.  Without ``correction`` sigmoid scores of the largest logits; with it
    the largest of softmax + correction, weighted by their normalised softmax values.  The last ``identity`` of the router's
    outputs have no rows (``row_of`` -1)."""
    lib = _lib.load()
    _need(logits, torch.float32, "logits")
    assert logits.is_contiguous() and logits.shape[2] == -(-(experts + identity) // 16) * 16
    assert correction is None or (correction.is_cuda and correction.numel() == experts + identity)
    splits, n = logits.shape[:2]
    r, dev = ExpertRows(), logits.device
    i32 = lambda *s: torch.empty(*s, dtype=torch.int32, device=dev)
    f32 = lambda *s: torch.empty(*s, dtype=torch.float32, device=dev)
    r.ids, r.scores, r.row_of, r.src, r.weight = i32(n, top), f32(n, top), i32(n, top), i32(n * top), f32(n * top)
    r.tiles, r.num_tiles, r.tile_rows = i32(n * top // tile_rows + min(experts, n * top), 4), i32(1), tile_rows
    ws = _workspace(lib.tlf_moe_group_workspace_bytes(n, top, experts), dev, "moe")
    check(lib.tlf_moe_group(logits.data_ptr(), splits, r.ids.data_ptr(), r.scores.data_ptr(), r.row_of.data_ptr(),
                            r.src.data_ptr(), r.weight.data_ptr(), r.tiles.data_ptr(), r.num_tiles.data_ptr(),
                            r.tiles.shape[0], n, top, experts, identity, _opt(correction),
                            _dt(correction) if correction is not None else DT_BF16, tile_rows, ws.data_ptr(), ws.numel(),
                            _stream()),
          "tlf_moe_group")
    return r


def moe_gemm(x, w, rows: ExpertRows, gather: bool, clipped_glu: bool = False, limit: float = 0.0, swiglu: bool = False):
    """One product per expert, ``w [E, Nout, K]``.  ``gather``: x rows are tokens (otherwise rows in expert order);
    ``clipped_glu``: interleaved gate / up channels, activated, the row's weight on both products; ``swiglu``: interleaved
    channels, ``silu(gate) * up``."""
    lib = _lib.load()
    _need(x, w.dtype, "x")
    assert x.stride(1) == 1 and w.is_contiguous() and w.shape[2] == x.shape[1]
    n, N = rows.src.numel(), w.shape[1]
    assert gather or x.shape[0] == n
    assert not (clipped_glu and swiglu)
    y = torch.empty(n, N // 2 if clipped_glu or swiglu else N, dtype=x.dtype, device=x.device)
    check(lib.tlf_moe_gemm(x.data_ptr(), x.stride(0), x.shape[0], w.data_ptr(), y.data_ptr(), rows.tiles.data_ptr(),
                           rows.num_tiles.data_ptr(), rows.tiles.shape[0], rows.tile_rows,
                           rows.src.data_ptr() if gather else None, rows.weight.data_ptr() if clipped_glu else None, n, N,
                           w.shape[2], 1 if clipped_glu else 2 if swiglu else 0, float(limit), _dt(x), _stream()), "tlf_moe_gemm")
    return y


def xielu(x, col, cols, pq, out):
    """``out[:, :cols] = xielu(x[:, col:col + cols])``, zeros in the rest of ``out``'s columns."""
    lib = _lib.load()
    _need(pq, out.dtype, "pq")
    assert pq.numel() == 2 and out.stride(1) == 1 and x.shape[0] == out.shape[0]
    check(lib.tlf_xielu(*_source(x), col, pq.data_ptr(), out.data_ptr(), out.stride(0), out.shape[0], cols, out.shape[1],
                        _dt(out), _stream()), "tlf_xielu")
    return out


def linear_xielu(x, w, act_col, pq, out):
    """``bf16_linear(x, w)`` with xIELU on the columns from ``act_col`` on, which go to ``out`` instead; returns the rest (its
    columns from ``act_col`` on are not written)."""
    lib = _lib.load()
    _need(x, BF16, "x"); _need(w, BF16, "w"); _need(pq, BF16, "pq"); _need(out, BF16, "out")
    assert x.dim() == 2 and x.stride(1) == 1 and w.is_contiguous() and out.stride(1) == 1 and out.shape[0] == x.shape[0]
    (M, K), N = x.shape, w.shape[0]
    assert w.shape[1] == K and pq.numel() == 2
    y = torch.empty(M, N, dtype=BF16, device=x.device)
    check(lib.tlf_bf16_gemm_xielu(x.data_ptr(), x.stride(0), w.data_ptr(), y.data_ptr(), M, N, K, act_col, pq.data_ptr(),
                                  out.data_ptr(), out.stride(0), out.shape[1], _stream()), "tlf_bf16_gemm_xielu")
    return y
