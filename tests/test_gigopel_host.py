"""Gigopel on the CPU: the plain implementation against closed forms, planted mistakes, configuration and checkpoint
routing, the host side of short and long portions, and argument checks of the entry points."""
import copy
import json
import math

import pytest
import torch

from oracle import gigopel as O
from tests import gigopel_cases as C
from tinyllmforge_amd.config import Config, GigopelConfig, model_config
from tinyllmforge_amd.engine import inputs as I
from tinyllmforge_amd.engine.scheduler import Scheduler
from tinyllmforge_amd.engine.sequence import Sequence
from tinyllmforge_amd.sampling_params import SamplingParams

F64 = torch.float64


# ---------------------------------------------------------------------------------------------- plain implementation
def test_norms_closed_form():
    x, w = torch.tensor([[3.0, 4.0]], dtype=F64), torch.tensor([1.0, -0.5], dtype=F64)
    r = math.sqrt(12.5 + 0.5)
    assert torch.allclose(O.zero_centred_norm(x, w, 0.5), torch.tensor([[6 / r, 2 / r]], dtype=F64))
    assert torch.allclose(O.plain_norm(x, w, 0.5), torch.tensor([[3 / r, -2 / r]], dtype=F64))


def test_xielu_closed_form():
    p, q = torch.tensor(0.3, dtype=F64), torch.tensor(-1.2, dtype=F64)
    a, b = math.log(1 + math.exp(0.3)), 0.5 + math.log(1 + math.exp(-1.2))
    z = torch.tensor([2.0, 0.0, -1.5, 1e-4, -1e-4, -50.0], dtype=F64)
    want = [a * 4 + 1, 0.0, b * (math.exp(-1.5) - 1 + 1.5) - 0.75, a * 1e-8 + 5e-5, b * (math.expm1(-1e-4) + 1e-4) - 5e-5, b * 49 - 25]
    assert torch.allclose(O.xielu(z, p, q), torch.tensor(want, dtype=F64), atol=1e-15)


def test_softmax_attention_sees_its_window():
    T = 7
    q = torch.zeros(T, 1, 2, dtype=F64)
    v = torch.arange(T, dtype=F64).view(T, 1, 1)
    o = O.softmax_attention(q, torch.zeros(T, 1, 2, dtype=F64), v, 1.0, size=3)[:, 0, 0]
    assert o.tolist() == pytest.approx([0, 0.5, 1, 2, 3, 4, 5])           # means of the last three positions
    k = torch.zeros(T, 1, 2, dtype=F64)
    k[2], q[:] = 10.0, 10.0
    o = O.softmax_attention(q, k, v, 1.0, size=3)[:, 0, 0]
    assert o[2:5].tolist() == pytest.approx([2, 2, 2]) and o[5].item() == pytest.approx(4)


def test_absorbing_the_keys_changes_nothing():
    """Scores from q_own . (Uk c) equal (Uk^T q_own) . c, values mixed after Uv equal Uv of the mixed latents."""
    g = torch.Generator().manual_seed(0)
    T, H, D, R, rank, V = 9, 2, 5, 4, 6, 3
    c, turned = torch.randn(T, rank, generator=g, dtype=F64), torch.randn(T, R, generator=g, dtype=F64)
    uk, uv = torch.randn(H * D, rank, generator=g, dtype=F64), torch.randn(H * V, rank, generator=g, dtype=F64)
    q = torch.randn(T, H, D + R, generator=g, dtype=F64)
    k, v = O.latent_keys_values(c, turned, uk, uv, H)
    full = O.softmax_attention(q, k, v, 0.3, 4)
    q2 = torch.cat([torch.einsum("thd,hdr->thr", q[..., :D], uk.view(H, D, rank)), q[..., D:]], dim=-1)
    row = torch.cat([c, turned], dim=-1)[:, None].expand(T, H, rank + R)
    mixed = O.softmax_attention(q2, row, c[:, None].expand(T, H, rank), 0.3, 4)
    assert torch.allclose(torch.einsum("thr,hvr->thv", mixed, uv.view(H, V, rank)), full)


def test_experts_closed_form():
    x = torch.tensor([[2.0]], dtype=F64)
    one = torch.ones(1, 1, dtype=F64)
    y = O.clipped_expert(x, one, -one, 3 * one, limit=1.5)                 # gate 2 -> 1.5, up -2 -> -1.5
    assert y.item() == pytest.approx(3 * 1.5 / (1 + math.exp(-1.702 * 1.5)) * (-0.5))
    low = O.clipped_expert(-x, one, one, one, limit=1.5)                   # the gate is not cut from below
    assert low.item() == pytest.approx(-2 / (1 + math.exp(1.702 * 2)) * (1 - 1.5))
    h = torch.tensor([[1.0, 0.0]], dtype=F64)
    ids, s = O.route(h, torch.tensor([[0.1, 9], [2.0, 9], [-1.0, 9], [1.0, 9]], dtype=F64), 2)
    assert ids.tolist() == [[1, 3]] and s[0].tolist() == pytest.approx([1 / (1 + math.exp(-2)), 1 / (1 + math.exp(-1))])


def plant(monkeypatch, cfg, w, fault):
    """``(configuration, weights)`` with a mistake, or the mistake put into the plain implementation."""
    cfg, w = copy.deepcopy(cfg), dict(w)
    mixers = [la["mixer"] for la in cfg["layers"]]
    if fault.startswith("window"):
        for m in mixers:
            m["mask"]["size"] += 1 if "+" in fault else -1
    elif fault == "rotation base":
        for m in mixers:
            m["rot"]["base"] *= 2
    elif fault == "pairs half apart":
        def halves(x, positions, dims, base):
            order = torch.arange(dims).view(2, -1).T.reshape(-1)          # (i, i + dims / 2) next to each other
            y = rotate(torch.cat([x[..., order], x[..., dims:]], dim=-1), positions, dims, base)
            return torch.cat([y[..., torch.argsort(order)], y[..., dims:]], dim=-1)
        rotate = O.rotate_interleaved_fast
        monkeypatch.setattr(O, "rotate_interleaved_fast", halves)
    elif fault == "latent not normed":
        monkeypatch.setattr(O, "plain_norm", lambda x, w, eps: x * w)
    elif fault == "norm weight not around zero":
        monkeypatch.setattr(O, "zero_centred_norm", lambda x, w, eps: x / O.rms(x, eps) * (0.5 + w))
    elif fault == "no multiplier":
        cfg["residual_mult"] = 1.0
    elif fault == "activation's numbers swapped":
        for n in w:
            if n.endswith("mlp.act"):
                w[n] = w[n].flip(0)
    elif fault == "scores renormalised":
        route = O.route
        monkeypatch.setattr(O, "route", lambda h, r, top: (lambda i, s: (i, s / s.sum(-1, keepdim=True)))(*route(h, r, top)))
    elif fault == "scores on the output":
        def late(h, w, m):
            ids, s = O.route(h, w["router"], m["router"]["top"])
            return torch.stack([sum(s[t, k] * O.clipped_expert(h[t:t + 1], *(w[f"e{e}.{p}"] for p in ("gate", "up", "down")),
                                                               m["expert"]["limit"])[0] for k, e in enumerate(ids[t].tolist()))
                                for t in range(h.shape[0])])
        monkeypatch.setattr(O, "moe_mlp", late)
    else:
        for la in cfg["layers"]:
            if la["mlp"] and la["mlp"]["kind"] == "moe":
                if fault == "limit":
                    la["mlp"]["expert"]["limit"] *= 1.3
                elif fault == "one expert fewer":
                    la["mlp"]["router"]["top"] -= 1
    return cfg, w


@pytest.mark.parametrize("fault", ["window + 1", "window - 1", "rotation base", "pairs half apart", "latent not normed",
                                   "norm weight not around zero", "no multiplier", "activation's numbers swapped",
                                   "scores renormalised", "scores on the output", "limit", "one expert fewer"])
def test_the_tests_weights_show_a_fault(fault, monkeypatch):
    """A mistake planted in the plain implementation is far above the GPU tests' tolerances."""
    cfg = C.CONFIGS["odd"]
    w, toks = C.weights(cfg), C.tokens(cfg, 90)
    want = O.forward(cfg, w, toks)
    err = C.logit_error(O.forward(*plant(monkeypatch, cfg, w, fault), toks), want)
    assert err.max() > 0.02          # 32-bit runs are held to 5e-5


@pytest.mark.parametrize("name", C.CONFIGS)
def test_routing_is_no_close_call(name):
    """The tests' routers leave room for rounding between the last expert chosen and the first one left out."""
    cfg = C.CONFIGS[name]
    w, toks = C.weights(cfg), C.tokens(cfg, 40)
    seen, route = [], O.route

    def watch(h, r, top):
        z = (h @ r.T).sort(dim=-1, descending=True).values
        if top < r.shape[0]:
            seen.append((z[:, top - 1] - z[:, top]).min().item())
        return route(h, r, top)
    O.route = watch
    try:
        O.forward(cfg, w, toks)
    finally:
        O.route = route
    assert not seen or min(seen) > 0.02


# ---------------------------------------------------------------------------------------------- configuration, loading
def test_registry_and_config(tmp_path):
    from tinyllmforge_amd.models.gigopel import GigopelForCausalLM
    from tinyllmforge_amd.models.registry import model_class
    cfg = C.CONFIGS["odd"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    hf = model_config(str(tmp_path))
    assert isinstance(hf, GigopelConfig) and model_class(hf) is GigopelForCausalLM
    assert hf.windows == (5, 37, 150) and hf.residual_mult == 0.7 and hf.hidden_size == 90 and hf.vocab_size == 203
    assert hf.portioned and not hf.recurrent and hf.float32 and not hf.position_quirk
    c = Config(str(tmp_path), max_model_len=300, kvcache_block_size=64, max_num_batched_tokens=64, dtype="float32")
    assert c.hf_config.torch_dtype == torch.float32 and c.hf_config.max_position_embeddings == 300
    bad = copy.deepcopy(cfg)
    bad["layers"][0]["type"] = "other"
    with pytest.raises(AssertionError, match="other"):
        model_config(bad)


def build(cfg, dtype=torch.bfloat16):
    from tinyllmforge_amd.models.gigopel import GigopelForCausalLM
    hf = model_config(copy.deepcopy(cfg))
    hf.max_position_embeddings, hf.torch_dtype = 32, dtype
    torch.set_default_dtype(dtype)
    try:
        return GigopelForCausalLM(hf)
    finally:
        torch.set_default_dtype(torch.float32)


def test_loading_fills_every_parameter(tmp_path):
    from safetensors.torch import save_file
    from tinyllmforge_amd.utils.loader import load_model, load_state_dict
    cfg = C.CONFIGS["odd"]
    w = C.weights(cfg)
    model = build(cfg)
    assert model.expected_tensors() == set(w)
    save_file(w, str(tmp_path / "model.safetensors"))
    load_model(model, str(tmp_path))
    la = model.layers[0]
    assert torch.equal(la.inp.weight[:78, :90], w["l0.mix.q"]) and torch.equal(la.inp.weight[78:111, :90], w["l0.mix.dkv"])
    assert torch.equal(la.inp.weight[111:161, :90], w["l0.mlp.up"]) and not la.inp.weight[161:].any()
    assert torch.equal(la.out.weight[:90, :39], w["l0.mix.o"]) and torch.equal(la.out.weight[:90, 64:114], w["l0.mlp.down"])
    assert not la.out.weight[:, 39:64].any() and la.out.weight.shape == (96, 128)
    assert torch.equal(la.attn.uk, w["l0.mix.uk"]) and torch.equal(la.act.pq, w["l0.mlp.act"])
    ex = model.layers[1].experts
    gu = ex.gate_up[3].view(8, 2, 8, 128)                                  # 20 channels in 64, 8 gate rows then the 8 up rows
    assert torch.equal(gu[:, 0].reshape(64, 128)[:20, :90], w["l1.mlp.e3.gate"])
    assert torch.equal(gu[:, 1].reshape(64, 128)[:20, :90], w["l1.mlp.e3.up"]) and not gu[3:].any()
    assert torch.equal(ex.down[4, :90, :20], w["l1.mlp.e4.down"]) and torch.equal(ex.router[:5, :90], w["l1.mlp.router"])
    other = build(cfg)
    load_state_dict(other, w)
    assert all(torch.equal(a, b) for a, b in zip(model.layers.parameters(), other.layers.parameters()))
    with pytest.raises(ValueError, match="l1.mlp.e2.up"):
        load_state_dict(build(cfg), {k: v for k, v in w.items() if k != "l1.mlp.e2.up"})
    for name in ("l9.norm1", "l0.mlp.router", "head", "l2.mlp.up"):
        with pytest.raises(KeyError):
            model.route_tensor(name)


def test_random_initialisation_keeps_pads_and_norms():
    from tinyllmforge_amd.utils.loader import random_init_
    model = random_init_(build(C.CONFIGS["odd"]), seed=3)
    ex = model.layers[1].experts
    ex.zero_pads_()
    gu = ex.gate_up.view(5, 8, 2, 8, 128)
    assert not gu[:, 3:].any() and not gu[:, 2, :, 4:].any() and not gu[..., 90:].any() and gu[:, 2, :, :4, :90].any()
    assert not ex.down[:, 90:].any() and not ex.down[..., 20:].any() and not ex.router[5:].any()
    assert not model.norm.weight.any() and (model.layers[0].attn.norm.weight == 1).all()


# ---------------------------------------------------------------------------------------------- portions on the host
def seq_of(n, computed, scheduled, table):
    s = Sequence(list(range(100, 100 + n)))
    s.num_computed, s.num_scheduled, s.block_table = computed, scheduled, table
    return s


def test_short_and_long_portions():
    seqs = [seq_of(70, 69, 1, [4, 9]), seq_of(100, 60, 7, [7, 3]), seq_of(30, 0, 9, [5]), seq_of(200, 20, 40, [1, 2, 6, 8]), seq_of(64, 0, 64, [10])]
    d = I.portion_inputs(seqs, 64, long_portion=10, windows=(5, 30, 500))
    assert (d["num_single"], d["num_short"], d["num_short_rows"], d["max_short"], d["max_portion"]) == (1, 2, 17, 9, 64)
    # keys from max(0, start - size + 1) to the portion's end
    assert d["kv_offsets"].tolist() == [[0, 44, 108], [0, 60, 124], [0, 60, 124]]
    assert d["kv_rows"] == (108, 124, 124) and d["max_kv_rows"] == (64, 64, 64)
    none = I.portion_inputs(seqs[:3], 64, long_portion=10, windows=(5,))
    assert none["kv_rows"] == (0,) and none["max_kv_rows"] == (0,) and none["num_short"] == 2
    plain = I.portion_inputs(seqs, 64)
    assert plain["num_short"] == 0 and plain["num_short_rows"] == 1 and plain["kv_offsets"].shape == (0, 5)
    with pytest.raises(AssertionError):
        I.portion_inputs(list(reversed(seqs)), 64, long_portion=10)
    assert [I.portion_kind(n, 10) for n in (1, 2, 9, 10, 11)] == [0, 1, 1, 2, 2] and I.portion_kind(2, None) == 2


def test_scheduler_needs_no_state_slots():
    cfg = Config(C.CONFIGS["ones"], max_model_len=512, kvcache_block_size=64, max_num_batched_tokens=48, max_num_seqs=4,
                 num_kvcache_blocks=6)
    Sequence.block_size = 64
    s = Scheduler(cfg)
    assert s.state_slots is None and s.portioned
    a, b = Sequence([1] * 5, SamplingParams(0.0, 3, True)), Sequence([2] * 70, SamplingParams(0.0, 2, True))
    s.add(a)
    s.add(b)
    sizes = []
    while not s.is_finished():
        batch, _ = s.schedule()
        sizes.append([q.num_scheduled for q in batch])
        ends = [q.num_computed + q.num_scheduled == len(q) for q in batch]
        s.postprocess(batch, [7 if e else None for e in ends])
    assert sizes == [[5, 43], [1, 27], [1, 1]] and len(s.block_manager.free_block_ids) == 6


# ---------------------------------------------------------------------------------------------- argument checks
def test_entry_points_reject_bad_arguments_on_the_host():
    import ctypes
    from tinyllmforge_amd import _lib, ops
    lib, a = _lib.load(), 4096
    shape = (3, 20, 6, 27, 13)             # heads, dim, rotated dim, latent, value dim
    s = ops.LatentShape(*shape)
    assert (s.da, s.ta, s.ra, s.va, s.dq, s.lp, s.rp) == (24, 8, 32, 16, 32, 64, 32)
    prep = lambda sizes=shape, ld=120, col=78, q=a, n=2, sp=1, p=None, c=a: lib.tlf_latent_prep(
        a, ld, p, sp, None, col, a, a, a, 10, 0, a, 64, q, c, 0, 0, None, None, 0, 0, None, n, *sizes, 1e-6, 0, None)
    assert prep(q=None, c=None) == -1 and prep(ld=100) == -2 and prep(col=70) == -2 and prep(n=0) == 0 and prep(sp=3) == -1
    assert prep(sizes=(3, 20, 5, 27, 13)) == -2 and prep(sizes=(3, 20, 6, 2000, 13)) == -2 and prep(sizes=(0, 20, 6, 27, 13)) == -2
    assert lib.tlf_head_gemm(a, a, a, 2, 3, 20, 32, 0, 0, 0, None) == -2 and lib.tlf_head_gemm(a, a, None, 2, 3, 32, 32, 0, 0, 0, None) == -1
    rows = lambda bs=64, win=5, ml=a, dt=0: lib.tlf_latent_rows(a, a, a, 4, a, a, None, a, ml, 2, *shape, bs, win, 10, 0.1, dt, None)
    assert rows(bs=100) == -2 and rows(win=0) == -2 and rows(ml=None) == -1 and rows(dt=5) == -5
    tile = lambda sizes=shape, plan=a, cu=None, starts=None, most=1, win=5: lib.tlf_latent_attn(
        a, a, a, 4, a, a, cu, starts, 0, 0, 2, most, plan, a, a, *sizes, 64, win, 10, 0.1, None)
    assert tile(plan=None) == -1 and tile(most=2) == -2 and tile(cu=a) == -1 and tile(win=0) == -2
    assert tile(sizes=(3, 20, 6, 600, 13)) == -5                             # cache rows too long for two tiles in LDS
    out = (ctypes.c_int32 * 3)()
    layout = lambda seqs, most, heads, lp: (lib.tlf_latent_attn_layout(seqs, most, heads, lp, ctypes.addressof(out)), list(out))
    assert layout(5, 1, 3, 576) == (0, [4 + 4 * 261 + 2 * 5, 261, 16])
    assert layout(2, 10, 40, 576)[1][1:] == [256 + 2 * 10 * 2, 32]           # two passes over 40 heads, a row a job
    assert layout(2, 10, 3, 100)[0] == -2
    assert lib.tlf_latent_attn_plan(a, None, None, None, 0, 0, 2, 1, 3, 64, 5, a, None) == -1
    values = lambda ld=39, plan=None, uv=a, cu=None: lib.tlf_latent_values(a, a, plan, cu, None, 0, 0, 2, 1, uv, None, a, ld, 2, *shape, 0, None)
    assert values(ld=38) == -2 and values(uv=None) == -1 and values(plan=a, cu=a) == -1
    pre = lambda sizes=shape, lde=120, win=5: lib.tlf_latent_prefill(a, a, lde, a, a, a, a, 0, 1, 8, None, None, 39, *sizes, win, 0.1, None)
    assert pre() == -1 and pre(lde=112) == -2 and pre(sizes=(3, 300, 6, 27, 13)) == -5 and pre(win=0) == -2
    assert lib.tlf_latent_gather(a, a, 4, a, a, a, 0, 1, 8, a, 100, 64, 5, 10, None) == -2
    assert lib.tlf_latent_attn_supported(2, 20, 6, 27, 13) == 1 and lib.tlf_latent_attn_supported(2, 20, 64, 600, 13) == 0
    assert lib.tlf_latent_prefill_supported(2, 20, 6, 27, 129) == 0
    group = lambda top=2, E=5, tiles=9, splits=1, n=4: lib.tlf_moe_group(a, splits, a, a, a, a, a, a, a, tiles, n, top, E, 0, None, 0, 32, None, 0, None)
    assert group(top=6) == -2 and group(E=600) == -2 and group(tiles=4) == -2 and group(n=0) == 0 and group(n=4000, tiles=9999) == -4
    gemm = lambda rows=32, N=32, K=64, dt=0, xs=64, count=4: lib.tlf_moe_gemm(a, xs, count, a, a, a, a, 9, rows, a, None, 8, N, K, 0, 0.0, dt, None)
    assert gemm(rows=48) == -2 and gemm(N=20) == -2 and gemm(xs=32) == -2 and gemm(dt=1, rows=32) == -2 and gemm(count=1 << 30) == -6
    assert gemm(K=80, xs=80) == -2
    assert lib.tlf_gemm_f32_sums(a, 64, a, a, 16, 4, 16, 64, ctypes.addressof(out), None) == -4
    res = lambda top=0, extra=None, es=0, ys=64: lib.tlf_residual_rmsnorm(a, ys, None, 1, None, extra, es, None, top, 0.5, a, a, 1.0, a, 2, 64, 1e-6, 0, None)
    assert res(top=2) == -1 and res(ys=32) == -2 and res(top=2, extra=a, es=64) == -1
    fused = lambda col=40, cols=64, ld=64, pq=a: lib.tlf_bf16_gemm_xielu(a, 64, a, a, 600, 112, 64, col, pq, a, ld, cols, None)
    assert fused(col=44) == -2 and fused(cols=60) == -2 and fused(ld=56) == -2 and fused(pq=None) == -1
    assert lib.tlf_xielu(a, 10, None, 1, None, 4, a, a, 8, 2, 8, 8, 0, None) == -2
    assert lib.tlf_xielu(a, 16, None, 1, None, 4, None, a, 8, 2, 8, 8, 0, None) == -1
