"""Gitopel on the CPU: the plain implementation against closed forms, configuration and checkpoint routing, the host
side of portions (inputs, scheduler, state slots) and argument checks of the entry points."""
import copy
import json
import math

import numpy as np
import pytest
import torch

from oracle import gitopel as O
from tests import gitopel_cases as C
from tinyllmforge_amd.config import Config, GitopelConfig, ModelConfig, model_config
from tinyllmforge_amd.engine import inputs as I
from tinyllmforge_amd.engine.scheduler import Scheduler
from tinyllmforge_amd.engine.sequence import Sequence
from tinyllmforge_amd.sampling_params import SamplingParams


# ---------------------------------------------------------------------------------------------- plain implementation
def test_grouped_norm_closed_form():
    x = torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=torch.float64)
    w = torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=torch.float64)
    y = O.grouped_rms_norm(x, w, 2, 0.5)
    r0, r1 = math.sqrt(12.5 + 0.5), math.sqrt(2.0 + 0.5)
    assert torch.allclose(y, torch.tensor([[3 / r0, 8 / r0, 0, 8 / r1]], dtype=torch.float64))
    one = O.grouped_rms_norm(x, w, 1, 0.0)
    assert torch.allclose(one, x * w / math.sqrt(29 / 4))


def test_rotation_pairs_neighbours_and_leaves_the_rest():
    x = torch.randn(3, 2, 10, dtype=torch.float64)
    y = O.rotate_interleaved(x, [0, 1, 7], 6, 100.0)
    assert torch.equal(y[0], x[0]) and torch.equal(y[:, :, 6:], x[:, :, 6:])
    for i in range(3):
        z = torch.complex(x[..., 2 * i], x[..., 2 * i + 1])
        turn = torch.tensor([p * 100.0 ** (-2 * i / 6) for p in (0, 1, 7)], dtype=torch.float64)
        want = z * torch.polar(torch.ones_like(turn), turn)[:, None]
        assert torch.allclose(torch.complex(y[..., 2 * i], y[..., 2 * i + 1]), want)
    assert torch.allclose(O.rotate_interleaved_fast(x, [0, 1, 7], 6, 100.0), y)


@pytest.mark.parametrize("size,pool", [(1, 1), (5, 3), (8, 4), (3, 7), (20, 2)])
def test_visible_sets(size, pool):
    for i in range(50):
        toks, blocks = O.visible_tokens(i, size), O.visible_blocks(i, size, pool)
        assert list(toks) == [j for j in range(i + 1) if i - j < size]
        seen = {p for b in blocks for p in range(b * pool, (b + 1) * pool)}
        assert not seen & set(toks)
        # whole blocks only: what is between is less than a block
        between = [j for j in range(toks.start) if j not in seen]
        assert len(between) < pool and blocks == list(range(len(blocks)))


def test_attention_weights_are_sigmoids_of_single_keys():
    q, k = torch.zeros(6, 1, 2, dtype=torch.float64), torch.zeros(6, 1, 2, dtype=torch.float64)
    v = torch.arange(6, dtype=torch.float64).view(6, 1, 1).expand(6, 1, 2)
    o = O.sigmoid_attention(q, k, v, torch.tensor([0.7], dtype=torch.float64), 1.0, size=2, pool=2)
    s = 1 / (1 + math.exp(-0.7))
    # position 4 sees tokens 3, 4 and block 0 (0, 1); position 5: 4, 5 and blocks 0, 1
    assert o[4, 0, 0].item() == pytest.approx(s * (3 + 4 + 0.5))
    assert o[5, 0, 0].item() == pytest.approx(s * (4 + 5 + 0.5 + 2.5))
    assert o[3, 0, 0].item() == pytest.approx(s * (2 + 3 + 0.5)) and o[2, 0, 0].item() == pytest.approx(s * (1 + 2))


def test_gla_recurrence_is_a_decayed_sum():
    T, H, D, Dv = 9, 2, 3, 4
    g = torch.Generator().manual_seed(3)
    q, k = (torch.randn(T, H, D, generator=g, dtype=torch.float64) for _ in range(2))
    v = torch.randn(T, H, Dv, generator=g, dtype=torch.float64)
    la = -torch.rand(T, H, D, generator=g, dtype=torch.float64)
    o, last = O.gla_recurrence(q, k, v, la)
    for t in range(T):
        want = sum(((q[t] * k[s] * torch.exp(la[s + 1:t + 1].sum(0))).sum(-1, keepdim=True) * v[s]) for s in range(t + 1))
        assert torch.allclose(o[t], want)
    a, mid = O.gla_recurrence(q[:4], k[:4], v[:4], la[:4])
    b, end = O.gla_recurrence(q[4:], k[4:], v[4:], la[4:], mid)
    assert torch.allclose(torch.cat([a, b]), o) and torch.allclose(end, last)


def mutated(cfg, key, value, kind="attention"):
    out = copy.deepcopy(cfg)
    for layer in out["layers"]:
        if layer["type"] == kind:
            m = layer["mixer"]
            if key in ("size", "pool"):
                m["mask"][key] += value
            elif key in ("dims", "base"):
                m["rot"][key] = value
            else:
                m[key] = value
    return out


@pytest.mark.parametrize("fault", ["window + 1", "window - 1", "pool + 1", "no score bias", "no gate", "no key bias",
                                   "fewer rotated dimensions", "tau", "one norm group", "a wider window now and then"])
def test_the_tests_weights_show_a_fault(fault, monkeypatch):
    """A mistake planted in the plain implementation is far above the GPU tests' tolerances."""
    cfg = C.CONFIGS["odd"]
    w, toks = C.weights(cfg), C.tokens(cfg, 90)
    want = O.forward(cfg, w, toks)
    bad, bw = cfg, dict(w)
    if fault.startswith("window"):
        bad = mutated(cfg, "size", 1 if "+" in fault else -1)
    elif fault == "pool + 1":
        bad = mutated(cfg, "pool", 1)
    elif fault == "fewer rotated dimensions":
        bad = mutated(cfg, "dims", 16)
    elif fault == "tau":
        bad = mutated(cfg, "tau", 4.0, "gla")
    elif fault == "one norm group":
        bad = dict(cfg, norm=dict(groups=1, eps=cfg["norm"]["eps"]))
    elif fault == "a wider window now and then":
        # the rotation is relative and would hide it; the window and the blocks do not
        monkeypatch.setattr(O, "visible_tokens", lambda i, size: range(max(0, i - size), i + 1) if i % 7 == 0 else range(max(0, i - size + 1), i + 1))
    else:
        part = {"no score bias": ".pb", "no gate": ".mix.g", "no key bias": ".k.b"}[fault]
        for n in w:
            if n.endswith(part) and not (fault == "no gate" and "l1." in n):
                bw[n] = torch.zeros_like(w[n])
    err = C.logit_error(O.forward(bad, bw, toks), want)
    assert err.max() > 0.05          # 32-bit runs are held to 5e-5


# ---------------------------------------------------------------------------------------------- configuration, loading
def test_registry_and_config(tmp_path):
    from tinyllmforge_amd.models.gitopel import GitopelForCausalLM
    from tinyllmforge_amd.models.qwen3 import Qwen3ForCausalLM
    from tinyllmforge_amd.models.registry import model_class
    cfg = copy.deepcopy(C.CONFIGS["odd"])
    for layer in cfg["layers"]:
        layer["mixer"].pop("rank", None)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    from safetensors.torch import save_file
    save_file(C.weights(C.CONFIGS["odd"]), str(tmp_path / "model.safetensors"))
    hf = model_config(str(tmp_path))
    assert isinstance(hf, GitopelConfig) and model_class(hf) is GitopelForCausalLM
    assert hf.layers[1]["mixer"]["rank"] == 5                 # from the tensor's shape
    assert hf.hidden_size == 90 and hf.vocab_size == 203 and hf.portioned and not hf.position_quirk
    q = model_config(dict(architectures=["Qwen3ForCausalLM"], hidden_size=64, num_hidden_layers=1, num_attention_heads=1,
                          num_key_value_heads=1, intermediate_size=64))
    assert isinstance(q, ModelConfig) and model_class(q) is Qwen3ForCausalLM
    with pytest.raises(ValueError, match="architecture"):
        model_config(dict(architecture="Nothing"))
    c = Config(str(tmp_path), max_model_len=300, kvcache_block_size=64, max_num_batched_tokens=64, dtype="float32")
    assert c.hf_config.torch_dtype == torch.float32 and c.hf_config.max_position_embeddings == 300
    assert not c.decode_position_quirk and c.num_state_slots == c.max_num_seqs
    with pytest.raises(ValueError, match="kernels"):
        Config(dict(hidden_size=64, num_hidden_layers=1, num_attention_heads=1, num_key_value_heads=1,
                    intermediate_size=64), dtype="float32")


def test_loading_fills_every_parameter(tmp_path):
    from safetensors.torch import save_file
    from tinyllmforge_amd.models.gitopel import GitopelForCausalLM
    from tinyllmforge_amd.utils.loader import load_model, load_state_dict
    cfg = C.CONFIGS["odd"]
    w = C.weights(cfg)
    hf = model_config(cfg)
    hf.max_position_embeddings = 32
    torch.set_default_dtype(torch.bfloat16)
    try:
        model = GitopelForCausalLM(hf)
        other = GitopelForCausalLM(hf)
    finally:
        torch.set_default_dtype(torch.float32)
    save_file(w, str(tmp_path / "model.safetensors"))
    load_model(model, str(tmp_path))
    att, mlp = model.layers[0].mix, model.layers[1].mlp
    assert torch.equal(att.qkg.weight[:240, :90], w["l0.mix.q"]) and torch.equal(att.qkg.weight[320:326, :90], w["l0.mix.g"])
    assert att.qkg.weight.shape == (336, 128) and not att.qkg.weight[326:].any() and not att.qkg.weight[:, 90:].any()
    assert torch.equal(mlp.gate_up.weight[128:228, :90], w["l1.mlp.up"]) and not mlp.gate_up.weight[100:128].any()
    assert torch.equal(att.attn.score_bias, w["l0.mix.pb"])
    load_state_dict(other, w)
    assert all(torch.equal(a, b) for a, b in zip(model.parameters(), other.parameters()))
    short = {k: v for k, v in w.items() if k != "l2.mix.o.b"}
    fresh = GitopelForCausalLM(hf)
    with pytest.raises(ValueError, match="l2.mix.o.b"):
        load_state_dict(fresh, short)
    with pytest.raises(KeyError):
        model.route_tensor("l9.norm1")


# ---------------------------------------------------------------------------------------------- portions on the host
def seq_of(n, computed, scheduled, table, slot):
    s = Sequence(list(range(100, 100 + n)))
    s.num_computed, s.num_scheduled, s.block_table, s.state_slot = computed, scheduled, table, slot
    return s


def test_portion_inputs():
    seqs = [seq_of(70, 69, 1, [4, 9], 2), seq_of(3, 2, 1, [1], 0), seq_of(100, 60, 40, [7, 3], 1), seq_of(2, 0, 2, [5], 3)]
    d = I.portion_inputs(seqs, 64)
    assert d["num_single"] == 2 and d["max_portion"] == 40
    assert d["cu_seqlens_q"].tolist() == [0, 1, 2, 42, 44] and d["seq_starts"].tolist() == [69, 2, 60, 0]
    assert d["state_slots"].tolist() == [2, 0, 1, 3]
    pos = [69, 2] + list(range(60, 100)) + [0, 1]
    assert d["positions"].tolist() == pos and d["input_ids"].tolist() == [100 + p for p in pos]
    want = [9 * 64 + 5, 64 + 2] + [7 * 64 + p if p < 64 else 3 * 64 + p - 64 for p in range(60, 100)] + [320, 321]
    assert d["slot_mapping"].tolist() == want
    assert d["row_seq"].tolist() == [0, 1] + [2] * 40 + [3] * 2
    assert d["chunk_rows"].tolist() == [0, 16, 32, 40] and d["chunk_lens"].tolist() == [16, 16, 8, 2]
    assert d["cu_chunks"].tolist() == [0, 3, 4]
    only = I.portion_inputs(seqs[:2], 64)
    assert only["chunk_rows"].size == 0 and only["cu_chunks"].tolist() == [0]


def scheduler(blocks=8, slots=3, budget=32, max_seqs=4):
    cfg = Config(C.config(64, 1, 50, [C.gla(1, 16, 16)]), max_model_len=512, kvcache_block_size=64,
                 max_num_batched_tokens=budget, max_num_seqs=max_seqs, num_state_slots=slots, num_kvcache_blocks=blocks)
    Sequence.block_size = 64
    return Scheduler(cfg)


def finish_step(s, seqs, tok=7):
    ends = [q.num_computed + q.num_scheduled == len(q) for q in seqs]
    s.postprocess(seqs, [tok if e else None for e in ends])


def test_scheduler_mixes_portions_with_decoded_tokens():
    s = scheduler()
    a, b = Sequence([1] * 5, SamplingParams(0.0, 8, True)), Sequence([2] * 70, SamplingParams(0.0, 4, True))
    s.add(a)
    s.add(b)
    batch, portions = s.schedule()
    assert [(q is a, q.num_scheduled) for q in batch] == [(True, 5), (False, 27)] and portions
    finish_step(s, batch)
    assert len(a) == 6 and len(b) == 70 and b.num_computed == 27
    batch, portions = s.schedule()                        # a decodes beside b's next portion, within the budget
    assert [(q is a, q.num_scheduled) for q in batch] == [(True, 1), (False, 31)] and portions
    assert not s.can_run_ahead()
    finish_step(s, batch)
    batch, _ = s.schedule()
    assert [q.num_scheduled for q in batch] == [1, 12]
    finish_step(s, batch)
    assert len(b) == 71 and s.can_run_ahead()
    batch, portions = s.schedule()
    assert [q.num_scheduled for q in batch] == [1, 1] and not portions
    while not s.is_finished():
        finish_step(s, batch)
        if not s.is_finished():
            batch, _ = s.schedule()
    assert len(s.block_manager.free_block_ids) == 8 and len(s.state_slots.free) == 3
    assert a.completion_token_ids == [7] * 8 and b.completion_token_ids == [7] * 4


def test_scheduler_preempts_the_newest_and_restarts_it_from_its_first_token():
    s = scheduler(blocks=2, budget=128)
    a, b = Sequence([1] * 64, SamplingParams(0.0, 4, True)), Sequence([2] * 3, SamplingParams(0.0, 4, True))
    s.add(a)
    s.add(b)
    batch, _ = s.schedule()
    finish_step(s, batch)
    assert a.state_slot == 0 and b.state_slot == 1
    batch, _ = s.schedule()                               # a needs a second block: b gives up its own
    assert batch == [a] and b.state_slot == -1 and b.num_computed == 0 and not b.block_table
    finish_step(s, batch)
    for _ in range(2):
        batch, _ = s.schedule()
        assert batch == [a]
        finish_step(s, batch)
    assert a.is_finished
    batch, _ = s.schedule()
    assert batch == [b] and b.num_scheduled == 4           # its prompt and the token it had
    assert b.state_slot >= 0


def test_scheduler_waits_for_a_state_slot():
    s = scheduler(slots=1)
    a, b = (Sequence([1] * 4, SamplingParams(0.0, 1, True)) for _ in range(2))
    s.add(a)
    s.add(b)
    batch, _ = s.schedule()
    assert batch == [a]
    finish_step(s, batch)
    batch, _ = s.schedule()
    assert batch == [b] and b.state_slot == 0


# ---------------------------------------------------------------------------------------------- argument checks
def test_entry_points_reject_bad_arguments_on_the_host():
    from tinyllmforge_amd import _lib
    lib, a = _lib.load(), 4096
    norm = lambda **k: lib.tlf_group_rmsnorm_add(*[{**dict(y=a, s=64, p=None, sp=1, sc=None, b=None, w=a, x=a, n=a, h=a, rows=2, width=64, groups=4, eps=1e-6, dt=0, st=None), **k}[n]
                                                   for n in ("y", "s", "p", "sp", "sc", "b", "w", "x", "n", "h", "rows", "width", "groups", "eps", "dt", "st")])
    assert norm(y=None) == -1 and norm(sp=3) == -1 and norm(p=a + 4, sp=3) == -3 and norm(p=a, sp=3, dt=1) == -5 and norm(groups=3) == -2 and norm(s=32) == -2 and norm(dt=7) == -5 and norm(rows=0) == 0
    assert lib.tlf_embed_group_rmsnorm(a, a, 0, a, a, 0.0, a, 1, 64, 1, 1e-6, 0, None) == -2
    assert lib.tlf_attn_prep(a, 100, None, 1, None, None, None, a, a, 10, 32, a, 64, a, a, a, a, 1, 1, 1, 300, 320, 1e-6, 0, None) == -2  # head too wide
    assert lib.tlf_attn_prep(a, 60, None, 1, None, None, None, a, a, 10, 32, a, 64, a, a, a, a, 1, 1, 1, 32, 32, 1e-6, 0, None) == -2    # row too short
    assert lib.tlf_attn_prep(a, 80, None, 1, None, None, None, a, a, 10, 32, a, 64, a, a, a, None, 1, 1, 1, 32, 32, 1e-6, 0, None) == -1
    rows = lambda bs=64, pool=4, win=8, ws=a, wsb=1 << 30, dim=32, n=2: lib.tlf_pooled_attn_rows(
        a, a, a, a, a, a, a, a, 4, a, a, None, a, 64, n, 2, 1, dim, bs, pool, win, 100, 10, 0.1, 1, 0, ws, wsb, None)
    assert rows(bs=100) == -2 and rows(pool=0) == -2 and rows(win=0) == -2 and rows(n=0) == 0 and rows(dim=64) == -2
    assert lib.tlf_pooled_attn_prefill(a, a, a, a, a, a, a, a, 4, a, None, 0, 1, 8, a, 64, 2, 1, 32, 64, 4, 8, 10, 0.1, None) == -1
    assert lib.tlf_pool_blocks(a, a, a, a, a, 4, a, a, 0, 0, 8, 1, 32, 64, 4, 8, 10, 0, None) == 0
    gla = lambda dk=16, dv=16, r=4, ld=132, tau=2.0: lib.tlf_gla_decode(a, ld, None, 1, None, a, a, a, a, a, 4, a, a, 64, 2, 2, dk, dv, r, tau, 1.0, 1e-6, 0, None)
    assert gla(dk=300, ld=4000) == -2 and gla(ld=131) == -2 and gla(tau=0.0) == -2 and gla(dv=1000, ld=8000) == -2
    assert lib.tlf_gla_portions(a, 132, a, a, a, a, a, 4, a, a, a, a, 1, 0, 1, a, 64, 8, 2, 16, 16, 4, 2.0, 1.0, 1e-6, 0, None, 0, None) == -4
    assert lib.tlf_f32_gemm(a, 8, a, a, 2, 4, 16, None) == -2 and lib.tlf_f32_argmax(a, 4, a, 1, 8, None) == -2


def test_interleaved_table_is_exact_to_fp32():
    from tinyllmforge_amd.layers.rotary_embedding import rotation_table
    t = rotation_table(6, 5000, 10000.0)
    for p in (0, 1, 4999):
        for i in range(3):
            a = p * 10000.0 ** (-2 * i / 6)
            assert t[p, i].item() == np.float32(math.cos(a)) and t[p, 3 + i].item() == np.float32(math.sin(a))
