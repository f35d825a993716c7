"""Zuzunex on the CPU: the plain implementation against closed forms, planted mistakes, configuration and checkpoint routing,
tables, the host side of loops and state slots, and argument checks of the entry points."""
import copy
import json
import math

import pytest
import torch

from oracle import zuzunex as O
from tests import zuzunex_cases as C
from tinyllmforge_amd.config import Config, ZuzunexConfig, model_config
from tinyllmforge_amd.engine.scheduler import Scheduler
from tinyllmforge_amd.engine.sequence import Sequence
from tinyllmforge_amd.sampling_params import SamplingParams

F64 = torch.float64
t64 = lambda *v: torch.tensor(v, dtype=F64)


# ---------------------------------------------------------------------------------------------- plain implementation
def test_norms_closed_form():
    x = t64([1.0, 3.0, 8.0])
    r = math.sqrt((9 + 1 + 16) / 3 + 0.25)
    assert torch.allclose(O.layer_norm(x, t64(1.0, 2.0, 0.5), t64(0.0, 1.0, -1.0), 0.25), t64([-3 / r, -2 / r + 1, 2 / r - 1]))
    assert torch.allclose(O.unit_rms(t64([3.0, 4.0]), 0.5), t64([3.0, 4.0]) / math.sqrt(13))


def test_convolution_looks_back():
    u = t64([1.0], [10.0], [100.0], [1000.0])
    w = t64([0.5, 2.0, 3.0])                                    # two back, one back, the token itself
    assert O.causal_conv(u, w)[:, 0].tolist() == [3, 32, 320.5, 3205]


def test_query_temperature_steps():
    at = lambda p: O.query_temperature(p, 0.5, 4)
    assert [at(p) for p in (0, 2, 3, 6, 7)] == pytest.approx([1, 1] + [1 + 0.5 * math.log(2)] * 2 + [1 + 0.5 * math.log(3)])


def test_rotation_closed_form():
    rot = dict(dims=4, base=100.0)
    x = torch.arange(1.0, 7.0, dtype=F64).view(1, 1, 6)
    y = O.rotate_halves(x, [3], rot)[0, 0].tolist()             # pairs (0, 2) and (1, 3), angles 3 and 0.3
    assert y == pytest.approx([math.cos(3) - 3 * math.sin(3), 2 * math.cos(.3) - 4 * math.sin(.3), 3 * math.cos(3) + math.sin(3),
                               4 * math.cos(.3) + 2 * math.sin(.3), 5, 6])


def test_scaled_frequencies():
    rot = dict(dims=16, base=1000.0, scaling=dict(factor=4.0, original=100, fast=10.0, slow=1.0))
    pair = lambda t: 16 * math.log(100 / (2 * math.pi * t)) / (2 * math.log(1000))
    lo, hi = math.floor(pair(10)), math.ceil(pair(1))
    assert (lo, hi) == (0, 4)
    f, mult = O.rotation_frequencies(rot)
    plain = [1000 ** (-i / 8) for i in range(8)]
    ramp = [0, .25, .5, .75, 1, 1, 1, 1]
    assert f == pytest.approx([p * (1 - r) + p / 4 * r for p, r in zip(plain, ramp)]) and mult == pytest.approx(0.1 * math.log(4) + 1)
    # bounds that coincide: a step; bounds outside the pairs are cut
    step = O.rotation_frequencies(dict(dims=8, base=1e6, scaling=dict(factor=2.0, original=10, fast=500.0, slow=300.0)))[0]
    assert step == pytest.approx([1e6 ** (-i / 4) / (1 if i == 0 else 2) for i in range(4)])


def test_attention_closed_form():
    T = 3
    q, v = torch.zeros(T, 2, 2, dtype=F64), t64(1.0, 4.0, 10.0).view(T, 1, 1)
    o = O.sink_attention(q, torch.zeros(T, 1, 2, dtype=F64), v, 1.0, t64(0.0, math.log(3.0)))
    assert o[:, 0, 0].tolist() == pytest.approx([1 / 2, 5 / 3, 15 / 4])       # the sink counts like one more key of value 0 ...
    assert o[:, 1, 0].tolist() == pytest.approx([1 / 4, 5 / 5, 15 / 6])       # ... or like three
    k = torch.zeros(T, 1, 2, dtype=F64)
    k[0, 0, 0], q[2, 0, 0] = 8.0, 3.0
    o = O.sink_attention(q, k, v, 0.5, None, cap=5.0)
    e = math.exp(5 * math.tanh(12 / 5))
    assert o[2, 0, 0].item() == pytest.approx((e + 14) / (e + 2)) and o[2, 1, 0].item() == pytest.approx(5)


def test_routing_closed_form():
    h = t64([1.0])
    router = torch.log(t64([1.0], [2.0], [4.0], [1.0]))
    ids, w = O.route(h, router.view(4, 1), t64(0.0, 0.0, 0.0, 0.2), 2)        # scores 1/8, 2/8, 4/8, 1/8 (+ 0.2)
    assert ids.tolist() == [[2, 3]] and w[0].tolist() == pytest.approx([0.8, 0.2])
    tensors = {"router": router.view(4, 1), "correction": t64(0.0, 0.0, 0.0, 0.2)}
    for e in ("e0", "e1", "e2"):
        tensors |= {f"{e}.gate": t64([2.0]), f"{e}.up": t64([3.0]), f"{e}.down": t64([0.5])}
    tensors |= {"shared.gate": t64([1.0]), "shared.up": t64([1.0]), "shared.down": t64([-1.0])}
    y = O.moe_mlp(h.view(1, 1), tensors, C.moe(3, 1, 2, 1, 1))
    silu = lambda z: z / (1 + math.exp(-z))
    assert y.item() == pytest.approx(0.8 * silu(2) * 1.5 + 0.2 * 1 - silu(1))


def test_order_of_a_loop():
    assert O.layer_order(C.CONFIGS["odd"]) == [0, 1, 2, 1, 2, 1, 2, 3] == model_config(C.CONFIGS["odd"]).layer_runs()
    for name in C.CONFIGS:
        assert model_config(C.CONFIGS[name]).layer_runs() == O.layer_order(C.CONFIGS[name])
    assert O.layer_order(dict(layers=[0] * 3, loop=None)) == [0, 1, 2]
    assert model_config(dict(C.CONFIGS["odd"], loop=None)).layer_runs() == [0, 1, 2, 3]


def plant(monkeypatch, cfg, w, fault):
    """``(configuration, weights)`` with a mistake, or the mistake put into the plain implementation."""
    cfg, w = copy.deepcopy(cfg), dict(w)
    mixers = [la["mixer"] for la in cfg["layers"]]
    change = lambda end, f: w.update({n: f(x) for n, x in w.items() if n.endswith(end)})
    if fault == "no sink":
        change("sink", lambda x: x - 50)
    elif fault == "sink scaled":
        change("sink", lambda x: x * 0.5)
    elif fault == "no cap":
        for m in mixers:
            m.pop("softcap", None)
    elif fault == "scale inside the cap's result":
        monkeypatch.setattr(O, "soft_cap", lambda s, cap: s)
    elif fault == "temperature one position late":
        real = O.query_temperature
        monkeypatch.setattr(O, "query_temperature", lambda p, c, e: real(p - 1, c, e))
    elif fault == "no gate":
        monkeypatch.setattr(O, "sigmoid", lambda z: 0 * z + 0.5)
    elif fault == "taps reversed":
        change("conv", lambda x: x.flip(-1))
    elif fault == "convolution forgets at 64":
        real = O.causal_conv
        monkeypatch.setattr(O, "causal_conv", lambda u, k: torch.cat([real(u[:64], k), real(u[64:], k)]))
    elif fault == "bias after the convolution's zeros":
        real = O.causal_conv
        monkeypatch.setattr(O, "causal_conv", lambda u, k: real(torch.cat([u[:1], u]), k)[1:])
    elif fault == "no bias":
        change(".b", lambda x: x if x.shape[0] == cfg["width"] else 0 * x)
    elif fault == "one plus the weight":
        change("q.norm", lambda x: 1 + x)
    elif fault == "no mean":
        monkeypatch.setattr(O, "layer_norm", lambda x, g, b, eps: O.unit_rms(x, eps) * g + b)
    elif fault == "no scaling of the rotation":
        for m in mixers:
            m.get("rot", {}).pop("scaling", None)
    elif fault == "no factor on cos and sin":
        real = O.rotation_frequencies
        monkeypatch.setattr(O, "rotation_frequencies", lambda rot: (real(rot)[0], 1.0))
    elif fault == "neighbours rotated":
        real = O.rotate_halves
        def neighbours(x, positions, rot):
            d = rot["dims"]
            order = torch.arange(d).view(-1, 2).T.reshape(-1)
            y = real(torch.cat([x[..., order], x[..., d:]], dim=-1), positions, rot)
            return torch.cat([y[..., torch.argsort(order)], y[..., d:]], dim=-1)
        monkeypatch.setattr(O, "rotate_halves", neighbours)
    elif fault == "loop once less":
        cfg["loop"]["times"] -= 1
    elif fault == "logits not scaled":
        cfg["logit_scale"] = 1.0
    elif fault == "correction in the weights":
        def late(h, router, correction, top):
            ids, _ = route(h, router, correction, top)
            s = torch.softmax(h @ router.T, -1) + correction
            s = s.gather(-1, ids)
            return ids, s / s.sum(-1, keepdim=True)
        route = O.route
        monkeypatch.setattr(O, "route", late)
    elif fault == "no correction":
        change("correction", lambda x: 0 * x)
    elif fault == "scores not normalised":
        def raw(h, router, correction, top):
            ids, _ = route(h, router, correction, top)
            return ids, torch.softmax(h @ router.T, -1).gather(-1, ids)
        route = O.route
        monkeypatch.setattr(O, "route", raw)
    elif fault == "identity gives nothing":
        def silent(h, x, m):
            ids, f = O.route(h, x["router"], x["correction"], m["router"]["top"])
            return moe(h, x, m) - (f * (ids >= m["router"]["experts"])).sum(-1, keepdim=True) * h
        moe = O.moe_mlp
        monkeypatch.setattr(O, "moe_mlp", silent)
    elif fault == "no shared expert":
        change("shared.down", lambda x: 0 * x)
    else:
        raise KeyError(fault)
    return cfg, w


FAULTS = ["no sink", "sink scaled", "no cap", "scale inside the cap's result", "temperature one position late", "no gate", "taps reversed",
          "convolution forgets at 64", "bias after the convolution's zeros", "no bias", "one plus the weight", "no mean",
          "no scaling of the rotation", "no factor on cos and sin", "neighbours rotated", "loop once less", "logits not scaled",
          "correction in the weights", "no correction", "scores not normalised", "identity gives nothing", "no shared expert"]


@pytest.mark.parametrize("fault", FAULTS)
def test_the_tests_weights_show_a_fault(fault, monkeypatch):
    """A mistake planted in the plain implementation is far above the GPU tests' tolerances."""
    cfg = C.CONFIGS["odd"]
    w, toks = C.weights(cfg), C.tokens(cfg, 80)
    want = O.forward(cfg, w, toks)
    err = C.logit_error(O.forward(*plant(monkeypatch, cfg, w, fault), toks), want)
    assert err.max() > 0.02          # 32-bit runs are held to 5e-5


@pytest.mark.parametrize("name", C.CONFIGS)
def test_routing_is_no_close_call(name, monkeypatch):
    """The tests' routers leave room for rounding between the last expert chosen and the first one left out."""
    cfg = C.CONFIGS[name]
    w, toks = C.weights(cfg), C.tokens(cfg, 60)
    seen, chosen, route = [], set(), O.route

    def watch(h, r, c, top):
        s = (torch.softmax(h @ r.T, -1) + c).sort(dim=-1, descending=True)
        if top < r.shape[0]:
            seen.append((1 - s.values[:, top] / s.values[:, top - 1]).min().item())       # rounding errors are relative
            chosen.update((r.shape[0], e) for e in s.indices[:, :top].flatten().tolist())
        return route(h, r, c, top)
    monkeypatch.setattr(O, "route", watch)
    O.forward(cfg, w, toks)
    assert not seen or min(seen) > 0.06
    assert not seen or len(chosen) > 2


# ---------------------------------------------------------------------------------------------- configuration, loading
def test_registry_and_config(tmp_path):
    from tinyllmforge_amd.models.registry import model_class
    from tinyllmforge_amd.models.zuzunex import ZuzunexForCausalLM
    cfg = C.CONFIGS["odd"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    hf = model_config(str(tmp_path))
    assert isinstance(hf, ZuzunexConfig) and model_class(hf) is ZuzunexForCausalLM
    assert hf.logit_scale == 0.3 and hf.hidden_size == 90 and hf.vocab_size == 203 and hf.loop["times"] == 3
    assert hf.portioned and hf.recurrent and hf.float32 and not hf.position_quirk
    assert not model_config(C.config(64, 64, [C.attention(1, 1, 8, 8)])).recurrent         # no convolution, no state
    c = Config(str(tmp_path), max_model_len=300, kvcache_block_size=64, max_num_batched_tokens=64, dtype="float32")
    assert c.hf_config.torch_dtype == torch.float32 and c.hf_config.max_position_embeddings == 300
    for where, value in ((("layers", 0, "type"), "other"), (("loop", "stop"), 5), (("layers", 1, "mlp", "router", "top"), 7),
                         (("layers", 0, "mixer", "rot", "dims"), 22)):
        bad = copy.deepcopy(cfg)
        at = bad
        for k in where[:-1]:
            at = at[k]
        at[where[-1]] = value
        with pytest.raises(AssertionError):
            model_config(bad)


def build(cfg, dtype=torch.bfloat16, positions=32):
    from tinyllmforge_amd.models.zuzunex import ZuzunexForCausalLM
    hf = model_config(copy.deepcopy(cfg))
    hf.max_position_embeddings, hf.torch_dtype = positions, dtype
    torch.set_default_dtype(dtype)
    try:
        return ZuzunexForCausalLM(hf)
    finally:
        torch.set_default_dtype(torch.float32)


def test_loading_fills_every_parameter(tmp_path):
    from safetensors.torch import save_file
    from tinyllmforge_amd.utils.loader import load_model, load_state_dict
    cfg = C.CONFIGS["odd"]
    w = C.weights(cfg)
    model = build(cfg)
    assert model.expected_tensors() == set(w) == set(C.shapes(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    load_model(model, str(tmp_path))
    mix, at = model.layers[0].mix, 0                            # 3 heads of 20, one key of 20 and value of 13, gate 39
    for part, rows in (("q", 60), ("k", 20), ("v", 13), ("g", 39)):
        assert torch.equal(mix.qkvg.weight[at:at + rows, :90], w["l0.mix." + part])
        if part != "g":
            assert torch.equal(mix.attn.bias[at:at + rows], w[f"l0.mix.{part}.b"])
            assert torch.equal(mix.attn.conv[:, at:at + rows], w[f"l0.mix.{part}.conv"].T)
        at += rows
    assert torch.equal(mix.attn.q_norm.weight, w["l0.mix.q.norm"]) and torch.equal(mix.attn.sink, w["l0.mix.sink"])
    la = model.layers[1]
    assert la.mix.attn.bias is None and la.mix.attn.conv is None and la.mix.attn.q_norm is None and la.mix.attn.cap == 6.0
    assert torch.equal(la.norm2.bias, w["l1.norm2.b"]) and torch.equal(model.norm.bias, w["final.norm.b"])
    ex = la.mlp.experts
    assert torch.equal(ex.router[:6, :90], w["l1.mlp.router"]) and torch.equal(ex.correction, w["l1.mlp.correction"])
    gu = ex.gate_up[3].view(8, 2, 8, 128)                       # 20 channels in 64, 8 gate rows then the 8 up rows
    assert torch.equal(gu[:, 0].reshape(64, 128)[:20, :90], w["l1.mlp.e3.gate"])
    assert torch.equal(la.mlp.shared.down.weight[:90, :30], w["l1.mlp.shared.down"])
    assert model.norm.out_scale == 0.3 and model.layers[3].mlp is None
    other = build(cfg)
    load_state_dict(other, w)
    assert all(torch.equal(a, b) for a, b in zip(model.layers.parameters(), other.layers.parameters()))
    with pytest.raises(ValueError, match="l1.mlp.e2.up"):
        load_state_dict(build(cfg), {k: v for k, v in w.items() if k != "l1.mlp.e2.up"})
    for name in ("l9.norm1", "l0.mlp.router", "l1.mix.q.b", "l3.norm2", "l1.mlp.e5.up"):
        with pytest.raises(KeyError):
            model.route_tensor(name)


def test_random_initialisation_keeps_norms():
    from tinyllmforge_amd.utils.loader import random_init_
    model = random_init_(build(C.CONFIGS["odd"]), seed=3)
    assert (model.layers[0].norm1.weight == 1).all() and not model.layers[0].norm1.bias.any() and not model.norm.bias.any()
    assert (model.layers[0].mix.attn.q_norm.weight == 1).all() and model.layers[0].mix.attn.conv.any()


def test_tables_agree_with_the_plain_implementation():
    from tinyllmforge_amd.layers.rotary_embedding import rotation_table
    from tinyllmforge_amd.layers.sink_attention import query_temperatures
    temps = query_temperatures(0.4, 7, 500)
    assert torch.equal(temps, torch.tensor([O.query_temperature(p, 0.4, 7) for p in range(500)], dtype=F64).float())
    for rot in (C.CONFIGS["odd"]["layers"][0]["mixer"]["rot"], C.CONFIGS["even"]["layers"][2]["mixer"]["rot"],
                dict(dims=8, base=1e6, scaling=dict(factor=2.0, original=10, fast=500.0, slow=300.0))):
        t = rotation_table(rot["dims"], 9000, rot["base"], **(rot["scaling"] or {}))
        f, mult = O.rotation_frequencies(rot)
        for p in (0, 1, 77, 8999):
            want = [math.cos(p * x) * mult for x in f] + [math.sin(p * x) * mult for x in f]
            assert t[p].tolist() == pytest.approx(want, abs=1e-6)
    model = build(C.CONFIGS["even"], positions=64)
    a, b = (model.layers[i].mix.attn.cos_sin for i in (1, 2))
    assert a.shape == (64, 64) and b.shape == (64, 32) and model.layers[0].mix.attn.cos_sin is None


def test_every_run_of_a_looped_layer_has_its_own_cache_and_state():
    model = build(C.CONFIGS["odd"])
    a, b = model.layers[2].mix.attn, model.layers[3].mix.attn
    assert a.runs == 3 and b.runs == 1 and len(list(model.runs())) == 8
    item = 2
    assert b.page_bytes(64) == 64 * 1 * (32 + 64) * item and a.page_bytes(64) == 3 * 64 * 5 * (32 + 32) * item
    assert b.slot_bytes() == 0 and a.slot_bytes() == 3 * 5 * (5 * 17 * 2 + 5 * 8) * item
    a.bind_pages(2, 64, "cpu")
    a.bind_slots(3, "cpu")
    assert len({kv.k.data_ptr() for kv in a.kv}) == 3 and len({r.data_ptr() for r in a.rings}) == 3
    assert a.kv[0].k.shape == (2, 5, 64, 32) and a.rings[0].shape == (3, 5, 210)
    a.bind_pages(0, 64, "cpu")
    a.bind_slots(0, "cpu")
    assert a.kv == [None] * 3 and a.rings == [None] * 3
    norms = [n for n, _ in model.runs()]
    assert norms[1] is norms[3] is model.layers[1].norm1 and norms[7] is model.layers[3].norm1
    assert [getattr(c, "keywords", {}).get("run") for _, c in model.runs()] == [None, 0, 0, 1, 1, 2, 2, None]


def test_scheduler_hands_out_state_slots():
    cfg = Config(C.CONFIGS["ones"], max_model_len=512, kvcache_block_size=64, max_num_batched_tokens=48, max_num_seqs=4,
                 num_kvcache_blocks=6, num_state_slots=2)
    Sequence.block_size = 64
    s = Scheduler(cfg)
    for n in (5, 9, 7):
        s.add(Sequence([1] * n, SamplingParams(0.0, 3, True)))
    slots = set()
    while not s.is_finished():
        batch, _ = s.schedule()
        assert len(batch) <= 2 and len({q.state_slot for q in batch}) == len(batch)
        slots |= {q.state_slot for q in batch}
        ends = [q.num_computed + q.num_scheduled == len(q) for q in batch]
        s.postprocess(batch, [7 if e else None for e in ends])
    assert slots == {0, 1} and len(s.state_slots.free) == 2 and len(s.block_manager.free_block_ids) == 6


# ---------------------------------------------------------------------------------------------- argument checks
def test_entry_points_reject_bad_arguments_on_the_host():
    from tinyllmforge_amd import _lib
    lib, a = _lib.load(), 4096
    shape = (3, 1, 20, 13)                 # heads, kv heads, dim, value dim: 60 + 20 + 13 + 39 columns
    prep = lambda sizes=shape, ld=136, q=a, n=2, sp=1, p=None, conv=None, taps=0, ring=None, rot=12, bs=64, gate=None, seq=None, dt=0: lib.tlf_sink_prep(
        a, ld, p, sp, None, a, conv, taps, ring, a, 4, seq, None, a, a, a, a, None, 10, rot, a, q, a, a, gate, n, *sizes, bs, 5, 1e-6, 0.1, 0.0, dt, None)
    assert prep(q=None) == -1 and prep(ld=130) == -2 and prep(n=0) == 0 and prep(rot=22) == -2 and prep(rot=3) == -2
    assert prep(bs=100) == -2 and prep(sizes=(3, 2, 20, 13)) == -2 and prep(sizes=(3, 1, 600, 13), ld=9999) == -2
    assert prep(conv=a, taps=3) == -1 and prep(conv=a, taps=99, ring=a) == -2 and prep(conv=a, taps=3, ring=a, seq=a) == -1
    assert prep(sp=3) == -1 and prep(sp=3, p=a) == -5 and prep(sp=3, p=a, gate=a) == -5 and prep(dt=7) == -5      # sizes not multiples of 8
    tail = lambda taps=3, ld=136, ring=a, n=1: lib.tlf_conv_tail(a, ld, ring, a, 4, a, a, 0, n, taps, 93, 0, None)
    assert tail(ld=80) == -2 and tail(ring=None) == -1 and tail(n=0) == 0 and tail(taps=1) == 0 and tail(taps=0) == -2
    rows = lambda sizes=shape, cap=0.0, ldo=39, ldg=39, bt=4, most=200, out=a, ws=None, dt=0, n=2: lib.tlf_sink_attn_rows(
        a, a, a, a, bt, a, a, None, a, a, ldg, out, ldo, n, *sizes, 64, most, 10, cap, dt, ws, 0, None)
    assert rows(cap=-1.0) == -2 and rows(ldo=38) == -2 and rows(ldg=30) == -2 and rows(bt=3) == -2 and rows(out=None) == -1
    assert rows() == -4 and rows(dt=3) == -5 and rows(n=0) == 0 and rows(n=70000) == -2
    size = lambda *v: lib.tlf_sink_attn_rows_workspace_bytes(*v)
    assert size(2, *shape, 128, 0) == 0 and size(2, *shape, 200, 0) == 2 * 2 * 3 * (32 + 2) * 4 and size(0, *shape, 200, 0) == 0
    pre = lambda sizes=shape, ldo=39, out=a, n=1: lib.tlf_sink_attn_prefill(a, a, a, a, 4, a, a, 0, n, 8, a, a, 39, out, ldo, *sizes, 64, 10, 0.0, None)
    assert pre(ldo=38) == -2 and pre(out=None) == -1 and pre(n=0) == 0 and pre(sizes=(3, 1, 270, 13)) == -5
    assert lib.tlf_sink_attn_prefill_supported(256, 256) == 1 and lib.tlf_sink_attn_prefill_supported(64, 257) == 0
    group = lambda top=2, E=5, ident=1, dt=0: lib.tlf_moe_group(a, 1, a, a, a, a, a, a, a, 99, 4, top, E, ident, a, dt, 32, None, 0, None)
    assert group(top=7) == -2 and group(E=510, ident=3) == -2 and group(ident=-1) == -2 and group(dt=9) == -5
    assert lib.tlf_moe_gemm(a, 64, 4, a, a, a, a, 9, 32, a, None, 8, 32, 64, 3, 0.0, 0, None) == -5
    res = lambda y=a, ys=64, top=0, extra=None, own=None, b=a: lib.tlf_residual_layernorm(
        y, ys, None, 1, None, extra, 64, a, None, top, own, 64, a, a, b, 1.0, a, 2, 64, 1e-6, 0, None)
    assert res(b=None) == -1 and res(ys=32) == -2 and res(top=2, extra=a) == -1 and res(top=-1) == -2
    assert lib.tlf_embed_layernorm(a, a, 0, a, a, a, 1.0, a, 2, 64, 1e-6, 0, None) == -2
    assert lib.tlf_embed_layernorm(a, a, 9, a, a, None, 1.0, a, 2, 64, 1e-6, 0, None) == -1
