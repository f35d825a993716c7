"""Zuzunex on the GPU: every kernel against the plain implementation, then the model through the engine."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import zuzunex as O
from tests import zuzunex_cases as C
from tests.test_gpu_gitopel import run_trace

pytestmark = pytest.mark.gpu
DTYPES = {"bf16": torch.bfloat16, "f32": torch.float32}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def rel(got, want):
    return ((got.double().cpu() - want.double()).norm() / want.double().norm().clamp(min=1e-30)).item()


# ---------------------------------------------------------------------------------------------- single kernels
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,top", [(5, 90, 0), (3, 64, 2), (7, 1024, 1), (130, 4096, 3), (2, 20, 5), (9, 8192, 2), (4, 1, 1)])
def test_residual_layer_norm(dtype, rows, width, top):
    from tinyllmforge_amd import ops as P
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(0)
    tol = 3e-3 if dtype == "bf16" else 2e-6
    r = lambda *s: torch.randn(*s, generator=g)
    y, w, b, x = r(rows, width + 8).to(dt), r(width).to(dt), r(width).to(dt), 3 * r(rows, width) + 40      # a mean far from zero
    extra, own = r(rows * max(top, 1), width).to(dt), r(rows, width + 8).to(dt)
    index = torch.randperm(rows * max(top, 1), generator=g).view(rows, -1).to(torch.int32)
    index[torch.rand(index.shape, generator=g) < 0.3] = -1                           # rows that stand for `own`
    f = torch.rand(index.shape, generator=g)
    for scale, factors in ((1.0, f), (0.37, None)):
        xd = x.cuda()
        args = (extra.cuda(), index.cuda(), factors.cuda() if factors is not None else None, own.cuda()) if top else ()
        h = P.residual_layer_norm(y.cuda(), xd, w.cuda(), b.cuda(), 1e-3, scale, *args)
        rows_of = torch.where(index[..., None] < 0, own.double()[:, None, :width], extra.double()[index.long().clamp(min=0)])
        add = (rows_of * (factors.double()[..., None] if factors is not None else 1)).sum(1) if top else 0
        want = x.double() + y[:, :width].double() + add
        assert rel(xd, want) < 1e-6
        assert rel(h, scale * O.layer_norm(want, w.double(), b.double(), 1e-3)) < tol
        xd = x.cuda()
        h = P.residual_layer_norm(None, xd, w.cuda(), b.cuda(), 1e-3, scale, *args)  # nothing but the extra rows
        assert rel(xd, x.double() + add) < 1e-6 and rel(h, scale * O.layer_norm(x.double() + add, w.double(), b.double(), 1e-3)) < tol
    table, ids = r(11, width).to(dt), torch.tensor([i * 3 % 11 for i in range(rows)])
    xe, he = P.embed_layer_norm(ids.cuda(), table.cuda(), w.cuda(), b.cuda(), 1e-3, 0.5)
    assert torch.equal(xe.cpu(), table[ids].float())
    assert rel(he, 0.5 * O.layer_norm(table[ids].double(), w.double(), b.double(), 1e-3)) < tol


@pytest.mark.parametrize("rows,N,K", [(48, 1024, 4096), (33, 192, 4096), (64, 1024, 4096)])
def test_norm_adds_up_a_split_projection(rows, N, K):
    """Where the projection is split over K the norm sums the partials itself: the same bits as from finished rows."""
    from tinyllmforge_amd import ops as P
    g = torch.Generator().manual_seed(rows)
    a, w = torch.randn(rows, K, generator=g).bfloat16().cuda(), torch.randn(N, K, generator=g).bfloat16().cuda() * K ** -0.5
    nw, nb, x = torch.randn(N, generator=g).bfloat16().cuda(), torch.randn(N, generator=g).bfloat16().cuda(), torch.randn(rows, N, generator=g).cuda()
    x1, x2 = x.clone(), x.clone()
    h1 = P.residual_layer_norm(P.bf16_linear(a, w), x1, nw, nb, 1e-5)
    y = P.linear_deferred(a, w)
    h2 = P.residual_layer_norm(y, x2, nw, nb, 1e-5)
    assert y.splits > 1 and torch.equal(x1, x2) and torch.equal(h1, h2)


@pytest.mark.parametrize("rows,taps,D,V", [(40, 3, 64, 48), (64, 4, 128, 128), (33, 0, 192, 64), (64, 6, 32, 32)])
def test_preparation_adds_up_a_split_projection(rows, taps, D, V):
    """Decoded rows whose projection is split over K: the preparation sums the partials, the same bits as from finished rows."""
    from tinyllmforge_amd import ops as P
    H, G, K, g = 4, 2, 4096, torch.Generator().manual_seed(rows)
    b = lambda *s: torch.randn(*s, generator=g).bfloat16().cuda()
    chan = (H + G) * D + G * V
    a, w = b(rows, K), b(chan + H * V, K) * K ** -0.5
    pos = torch.randint(0, 90, (rows,), generator=g).cuda()
    slots = torch.randperm(64 * 4, generator=g)[:rows].to(torch.int32).cuda()
    states = torch.randperm(rows + 2, generator=g)[:rows].to(torch.int32).cuda()
    slots[3], states[3] = -1, -1                                 # a padding row
    temps, nw, bias, conv, ring = torch.rand(100, generator=g).cuda(), b(D), b(chan), b(taps, chan), b(rows + 2, taps, chan)
    cos = torch.rand(100, 16, generator=g).cuda()
    res = []
    for proj in (P.bf16_linear(a, w), P.linear_deferred(a, w)):
        kv, r = P.SinkKV(4, 64, G, D, V, torch.bfloat16, "cuda"), ring.clone()
        args = (bias, conv, r, states) if taps else (bias,)
        q, gate = P.sink_prep(proj, kv, H, pos, slots, 1e-5, 0.2, None, *args, q_norm=nw, k_norm=nw, cos_sin=cos, rot_dims=16, q_mult=temps)
        res.append((q, gate.contiguous(), kv.k, kv.v, r))
    assert proj.splits > 1 and all(torch.equal(x, y) for x, y in zip(*res))
    assert not torch.equal(res[0][4], ring) or not taps


class Attention:
    """A layer of sink attention with a few sequences in shuffled pages, run step by step as the engine does."""

    def __init__(self, sizes, lens, dt, seed=0, bs=64, scale=None, long_portion=16, cap=None, second=True, taps=3, rot=None, temps=None,
                 sink=None, runs=1, slots=(3, 0, 5)):
        from tinyllmforge_amd.engine.sequence import Sequence
        from tinyllmforge_amd.layers.rotary_embedding import rotation_table
        from tinyllmforge_amd.layers.sink_attention import SinkAttention, query_temperatures
        Sequence.block_size = bs
        H, G, D, V = self.sizes = sizes
        self.lens, self.dt, self.bs, self.long, self.taps, self.second = lens, dt, bs, long_portion, taps, second
        self.scale, self.cap, self.eps, self.rot, self.temps = scale or 2.0 / D ** 0.5, cap, 1e-4, rot, temps
        g = torch.Generator().manual_seed(seed)
        rnd = lambda *s: torch.randn(*s, generator=g)
        most = max(lens) + 1
        torch.set_default_dtype(dt)
        self.layer = SinkAttention(H, G, D, V, self.scale, self.eps, dt, cap=cap, bias=second, taps=taps if second else 0,
                                   weighted_norm=second, rot_dims=rot["dims"] if rot else 0,
                                   rope=rotation_table(rot["dims"], most, rot["base"], **(rot.get("scaling") or {})) if rot else None,
                                   temperatures=query_temperatures(*temps, most) if temps else None, runs=runs).cuda()
        torch.set_default_dtype(torch.float32)
        self.sink = (2 + rnd(H) if sink is None else sink).to(dt)
        self.layer.sink.data.copy_(self.sink)
        self.w = {}
        if second:
            for part, rows in list(self.layer.parts.items())[:3]:
                self.w[part + ".b"] = (0.5 * rnd(rows)).to(dt)
                self.w[part + ".conv"] = (0.6 * rnd(rows, taps)).to(dt)
                self.layer.load_channels(self.layer.bias, self.w[part + ".b"], part)
                self.layer.load_channels(self.layer.conv, self.w[part + ".conv"], part)
            for part in ("q", "k"):
                self.w[part + ".norm"] = (1 + 0.3 * rnd(D)).to(dt)
                getattr(self.layer, part + "_norm").weight.data.copy_(self.w[part + ".norm"])
        need = [-(-n // bs) for n in lens]
        perm = torch.randperm(sum(need) + 2, generator=g).tolist()
        self.layer.bind_pages(sum(need) + 2, bs, "cuda")
        self.layer.bind_slots(6, "cuda")
        for kv in self.layer.kv:                                 # stale contents of reused pages and slots
            kv.k[..., :D].fill_(3.0)
            kv.v[..., :V].fill_(3.0)
        for ring in self.layer.rings:
            if ring is not None:
                ring.fill_(5.0)
        self.seqs = []
        for i, (n, k) in enumerate(zip(lens, need)):
            s = Sequence([0] * n)
            s.block_table, s.state_slot = [perm.pop() for _ in range(k)], slots[i % len(slots)]
            self.seqs.append(s)
        self.columns = sum(self.layer.parts.values())

    def step(self, proj, parts, run=0):
        """``parts``: (sequence, tokens), in the engine's order of kinds.  Returns ``{sequence: [tokens, H * V]}``."""
        from tinyllmforge_amd.engine import inputs as I
        from tinyllmforge_amd.utils.context import reset_context, set_portions_context
        parts = sorted(parts, key=lambda x: I.portion_kind(x[1], self.long))
        seqs = [self.seqs[s] for s, _ in parts]
        for s, (_, n) in zip(seqs, parts):
            s.num_scheduled = n
        d = I.portion_inputs(seqs, self.bs, self.long)
        d = {k: torch.from_numpy(v).cuda() if hasattr(v, "dtype") else v for k, v in d.items()}
        d.pop("input_ids")
        pos = d.pop("positions")
        rows = torch.cat([proj[i][s.num_computed:s.num_computed + n] for s, (i, n) in zip(seqs, parts)]).to(self.dt)
        padded = torch.full((rows.shape[0], -(-self.columns // 16) * 16), 9.0, dtype=self.dt)
        padded[:, :self.columns] = rows
        set_portions_context(max_len=max(self.lens), **d)
        out = self.layer(padded.cuda(), pos, run).cpu()
        reset_context()
        got, at = {}, 0
        for s, (i, n) in zip(seqs, parts):
            got[i] = out[at:at + n]
            at += n
            s.num_computed += n
        return got

    def want(self, proj):
        p = proj.to(self.dt).double()
        T, (H, G, D, V) = p.shape[0], self.sizes
        q, k, v, gate = p.split([H * D, G * D, G * V, H * V], dim=1)
        if self.second:
            f = lambda u, n: O.causal_conv(u + self.w[n + ".b"].double(), self.w[n + ".conv"].double())
            q, k, v = f(q, "q"), f(k, "k"), f(v, "v")
        q, k = O.unit_rms(q.reshape(T, H, D), self.eps), O.unit_rms(k.reshape(T, G, D), self.eps)
        if self.second:
            q, k = q * self.w["q.norm"].double(), k * self.w["k.norm"].double()
        if self.temps:
            q = q * torch.tensor([O.query_temperature(i, *self.temps) for i in range(T)], dtype=q.dtype).view(T, 1, 1)
        if self.rot:
            q, k = O.rotate_halves(q, range(T), self.rot), O.rotate_halves(k, range(T), self.rot)
        o = O.sink_attention(q, k, v.reshape(T, G, V), self.scale, self.sink.double(), self.cap)
        return o.reshape(T, -1) * O.sigmoid(gate)


YARN = dict(factor=3.0, original=40, fast=6.0, slow=0.5)
# heads, kv heads, dim, value dim; cap; convolution taps (0: the mixer without biases, convolution, weights and rotation);
# rotated dims.  Every instantiated width, groups of one to many passes, sizes no vector divides, heads beyond the tiles
ATTN = [((3, 1, 20, 13), None, 3, 12), ((4, 2, 64, 64), 5.0, 0, 0), ((1, 1, 1, 1), 1.5, 0, 0), ((4, 4, 32, 128), None, 4, 32),
        ((20, 1, 128, 32), None, 2, 64), ((40, 2, 16, 24), 9.0, 0, 0), ((12, 2, 128, 128), None, 3, 128), ((12, 4, 128, 128), 25.0, 0, 0),
        ((6, 3, 192, 128), None, 4, 64), ((2, 1, 256, 256), None, 3, 48), ((70, 1, 40, 72), 4.0, 0, 0), ((5, 5, 96, 200), None, 1, 6),
        ((4, 2, 176, 88), None, 6, 176), ((2, 1, 270, 60), None, 3, 100), ((6, 2, 48, 400), 3.0, 0, 0), ((3, 3, 2, 2), None, 2, 2)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes,cap,taps,rot", ATTN)
def test_attention_over_portions_singles_and_mixtures(dtype, sizes, cap, taps, rot):
    dt, lens = DTYPES[dtype], [150, 67, 210]
    tol = 1.2e-2 if dtype == "bf16" else 4e-6
    schedules = {
        "whole": [[(0, 150), (1, 67), (2, 210)]],
        "portions": [[(0, 2), (1, 3)], [(0, 62), (2, 130)], [(0, 1), (1, 2), (2, 2)], [(0, 85), (1, 62), (2, 78)]],
        "mixed": [[(0, 100), (2, 64)], [(0, 1), (1, 20), (2, 1)]] + [[(0, 1), (1, 1), (2, 29)], [(0, 1), (2, 2)]] * 3 +
                 [[(0, 43), (1, 1)], [(1, 43), (2, 52)]],
        "single": [[(0, 1), (1, 1), (2, 1)] for _ in range(67)] + [[(0, 1), (2, 1)] for _ in range(83)] + [[(2, 1)] for _ in range(60)],
    }
    want, kw = None, dict(cap=cap, second=taps > 0, taps=taps, temps=(0.35, 50) if not taps else None,
                          rot=dict(dims=rot, base=500.0, scaling=YARN) if rot else None)
    for name, steps in schedules.items():
        a = Attention(sizes, lens, dt, **kw)
        g = torch.Generator().manual_seed(5)
        proj = [torch.randn(n, a.columns, generator=g) for n in lens]
        if want is None:
            want = [a.want(p) for p in proj]
        got = [[], [], []]
        for parts in steps:
            for s, o in a.step(proj, parts).items():
                got[s].append(o)
        for s in range(3):
            assert rel(torch.cat(got[s]), want[s]) < tol, (name, s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_preparation_of_many_rows(dtype):
    """More than 1024 rows: a lane group walks several tokens, across the ends of sequences."""
    lens = [501, 3, 2, 700, 1, 64, 9]
    a = Attention((3, 1, 24, 16), lens, DTYPES[dtype], taps=4, rot=dict(dims=16, base=300.0), slots=(0, 1, 2, 3, 4, 5, 0))
    g = torch.Generator().manual_seed(2)
    proj = [torch.randn(n, a.columns, generator=g) for n in lens]
    got = a.step(proj, list(enumerate(lens))[:6])
    for i in range(6):
        assert rel(got[i], a.want(proj[i])) < (1.2e-2 if dtype == "bf16" else 4e-6), i


@pytest.mark.parametrize("dtype", DTYPES)
def test_runs_of_a_loop_do_not_mix(dtype):
    a = Attention((4, 2, 32, 24), [90], DTYPES[dtype], runs=2, rot=dict(dims=8, base=90.0))
    g = torch.Generator().manual_seed(1)
    proj = [torch.randn(90, a.columns, generator=g) for _ in range(2)]
    got = [[], []]
    for n in (30, 1, 2, 40, 1, 16):
        for run in (0, 1):
            got[run].append(a.step([proj[run]], [(0, n)], run)[0])
            a.seqs[0].num_computed -= n * (run == 0)
    for run in (0, 1):
        assert rel(torch.cat(got[run]), a.want(proj[run])) < (1.2e-2 if dtype == "bf16" else 4e-6), run


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,cap", [(140, None), (300, 40.0), (65, 40.0)])
def test_one_key_stands_out(dtype, n, cap):
    """One token takes all the weight of whoever sees it, and its value tells it apart: the output says who saw it."""
    dt, (H, G, D, V) = DTYPES[dtype], (2, 1, 8, 4)
    for j in sorted({0, 1, 31, 32, 62, 63, 64, 127, 128, 129, n - 3, n - 2} & set(range(n - 1))):
        for cuts in ([n], [n - 3, 1, 1, 1], [2] * (n // 2) + [1] * (n % 2), [j + 1, n - j - 1], [j, n - j]):
            a = Attention((H, G, D, V), [n], dt, scale=8.0, cap=cap, second=False, sink=torch.full((H,), -5.0))
            proj = torch.zeros(n, a.columns)
            proj[:, :H * D:D] = 1.0                              # every query asks for channel 0
            proj[:, H * D + 1] = 1.0
            proj[j, H * D:H * D + 2] = torch.tensor([1.0, 0.0])
            proj[:, H * D + D] = 1.0                             # the value of all ...
            proj[j, H * D + D:H * D + D + 2] = torch.tensor([0.0, 1.0])   # ... but the one
            want = a.want(proj)
            got = torch.cat([a.step([proj], [(0, c)])[0] for c in cuts if c > 0])
            err = (got.double() - want).abs().amax(dim=1)
            assert err.max() < 0.02 * want.abs().max(), (j, cuts[:2], int(err.argmax()), err.max().item())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cap", [None, 7.0])
def test_sinks_of_every_size(dtype, cap):
    """Absent, small, as large as the scores and far above them; scores that lie far above and far below zero."""
    dt, n, (H, G, D, V) = DTYPES[dtype], 150, (5, 1, 16, 8)
    sink = torch.tensor([-1e30, -9.0, 0.0, 6.0, 60.0])
    for sign in (1.0, -1.0):
        for cuts in ([n], [100] + [1] * 50, [7] * 21 + [3]):
            a = Attention((H, G, D, V), [n], dt, scale=1.0, cap=cap, second=False, sink=sink)
            g = torch.Generator().manual_seed(3)
            proj = torch.randn(n, a.columns, generator=g)
            proj[:, :(H + G) * D] += 1.5 * torch.cat([torch.ones(H * D), sign * torch.ones(G * D)])
            want = a.want(proj).view(n, H, V)
            got = torch.cat([a.step([proj], [(0, c)])[0] for c in cuts]).view(n, H, V)
            for h in range(4):
                assert rel(got[:, h], want[:, h]) < (1.2e-2 if dtype == "bf16" else 1e-5), (sign, h)
            assert got[:, 4].abs().max() < 1e-15


@pytest.mark.parametrize("dtype", DTYPES)
def test_rows_of_many_unequal_sequences(dtype):
    """Decoded rows with contexts from one key to thousands, padding rows between them, several splits."""
    from tinyllmforge_amd import ops as P
    dt, g, (H, G, D, V), bs = DTYPES[dtype], torch.Generator().manual_seed(3), (6, 2, 40, 24), 64
    for B, longest in ((300, 700), (5, 4000), (1, 2500)):
        lens = torch.randint(1, 90, (B,), generator=g)
        lens[torch.randperm(B, generator=g)[:4]] = torch.tensor([longest, longest // 2 // 64 * 64, 65, 64])[:min(B, 4)]
        need = (lens + bs - 1) // bs
        bt = torch.full((B, int(need.max()) + 3), -1, dtype=torch.int32)
        perm, at = torch.randperm(int(need.sum()), generator=g), 0
        kv = P.SinkKV(int(need.sum()), bs, G, D, V, dt, "cuda")
        kv.k[..., :D] = torch.randn(kv.k.shape[:3] + (D,), generator=g).to(dt).cuda()
        kv.v[..., :V] = torch.randn(kv.v.shape[:3] + (V,), generator=g).to(dt).cuda()
        for i in range(B):
            bt[i, :need[i]] = perm[at:at + int(need[i])].to(torch.int32)
            at += int(need[i])
        q = torch.zeros(B, H, 64)
        q[..., :D] = torch.randn(B, H, D, generator=g)
        q = q * 0.4 * 1.4426950408889634                         # the scale and the base of the exponential are in q
        q, gate, sink = q.to(dt), torch.randn(B, H * V, generator=g).to(dt), torch.randn(H, generator=g).to(dt)
        slots = torch.zeros(B, dtype=torch.int32)
        slots[B // 2] = -1 if B > 1 else 0
        out = torch.full((B, H * V + 8), 7.0, dtype=dt, device="cuda")
        P.sink_attention_rows(q.cuda(), kv, bt.cuda(), (lens - 1).cuda(), slots.cuda(), sink.cuda(), gate.cuda(), None, 10 ** 6,
                              out[:, :H * V])
        assert (out[:, H * V:] == 7).all()
        k, v = kv.k.double().cpu(), kv.v.double().cpu()
        for i in range(B):
            n = int(lens[i])
            if slots[i] < 0:
                assert not out[i, :H * V].any()
                continue
            ki = k[bt[i, :need[i]].long()].transpose(1, 2).reshape(-1, G, 64)[:n, :, :D]
            vi = v[bt[i, :need[i]].long()].transpose(1, 2).reshape(-1, G, 32)[:n, :, :V]
            s = torch.einsum("gpd,ngd->gpn", q[i, :, :D].double().view(G, H // G, D), ki) / 1.4426950408889634
            e = torch.exp(s)
            o = torch.einsum("gpn,ngv->gpv", e / (e.sum(-1) + torch.exp(sink.double()).view(G, -1))[..., None], vi)
            want = o.reshape(-1) * O.sigmoid(gate[i].double())
            assert rel(out[i, :H * V], want) < (6e-3 if dtype == "bf16" else 4e-6), (B, i, n)


# ---------------------------------------------------------------------------------------------- experts
@pytest.mark.parametrize("corr_dtype", DTYPES)
@pytest.mark.parametrize("n,E,ident,top,splits", [(1, 5, 2, 2, 1), (64, 70, 7, 6, 3), (500, 16, 1, 1, 2), (1500, 33, 3, 4, 1), (9, 500, 12, 20, 1),
                                                  (5, 1, 0, 1, 1), (5000, 200, 0, 2, 1), (40, 2, 6, 8, 1)])
def test_choice_by_corrected_softmax(corr_dtype, n, E, ident, top, splits):
    from tinyllmforge_amd import ops as P
    g, every = torch.Generator().manual_seed(n), E + ident
    z = torch.randn(splits, n, -(-every // 16) * 16, generator=g)
    z[..., every:] = 50.0                                        # pads are never chosen and enter no sum
    corr = (0.1 * torch.randn(every, generator=g)).to(DTYPES[corr_dtype])
    corr[every // 2] = 2.0                                       # always chosen, whatever its score
    for tile in (32, 128):
        r = P.moe_group(z.cuda(), E, top, tile, corr.cuda(), ident)
        ids, scores, row_of = r.ids.cpu().long(), r.scores.cpu(), r.row_of.cpu().long()
        s = torch.softmax(z.double().sum(0)[:, :every], -1)
        best = (s + corr.double()).sort(dim=-1, descending=True)
        sure = (best.values[:, :top] - torch.cat([best.values[:, 1:], torch.full((n, 1), -9.0)], 1)[:, :top]).min(1).values > 1e-6
        assert sure.float().mean() > 0.9
        assert torch.equal(ids[sure], best.indices[sure, :top]) and (ids == every // 2).any(1).all()
        want = s.gather(1, ids)
        assert rel(scores, want / want.sum(1, keepdim=True)) < 1e-5
        own = ids >= E                                           # identity experts have no row
        assert (row_of[own] == -1).all()
        rows = int((~own).sum())
        assert torch.equal(row_of[~own].sort().values, torch.arange(rows))
        entry = torch.arange(n * top).view(n, top)[~own]
        assert torch.equal(r.src.cpu().long()[row_of[~own]], entry // top)
        by_row = torch.empty(rows, dtype=torch.long)
        by_row[row_of[~own]] = ids[~own]
        covered = []
        for e, first, count, _ in r.tiles.cpu()[:int(r.num_tiles)].tolist():
            assert 0 < count <= tile and (by_row[first:first + count] == e).all()
            covered += range(first, first + count)
        assert covered == list(range(rows))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,width,E,ident,top,ff", [(1, 90, 5, 1, 2, 20), (7, 64, 1, 1, 1, 1), (64, 192, 33, 4, 6, 72), (700, 128, 8, 2, 3, 64),
                                                    (300, 320, 4, 0, 2, 136), (33, 256, 16, 3, 19, 128), (2100, 64, 4, 2, 1, 40),
                                                    (129, 592, 8, 1, 1, 264), (9, 4096, 3, 1, 2, 16)])
def test_mixture_of_experts(dtype, n, width, E, ident, top, ff):
    from tinyllmforge_amd import ops as P
    from tinyllmforge_amd.layers.moe import SwiGLUExperts
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(n)
    torch.set_default_dtype(dt)
    m = SwiGLUExperts(width, E, top, ff, ident)
    torch.set_default_dtype(torch.float32)
    w = {"router": (2 * torch.randn(E + ident, width, generator=g) * width ** -0.5).to(dt), "correction": (0.1 * torch.randn(E + ident, generator=g)).to(dt)}
    for e in range(E):
        for k, shape in (("gate", (ff, width)), ("up", (ff, width)), ("down", (width, ff))):
            w[f"e{e}.{k}"] = (torch.randn(shape, generator=g) * 1.5 * shape[1] ** -0.5).to(dt)
    for name, (target, part) in m.routes().items():
        p = m.get_parameter(target)
        if part is None:
            p.data.copy_(w[name])
        else:
            p.weight_loader(p, w[name], part)
    m = m.cuda()
    h = torch.randn(n, width, generator=g).to(dt)
    extra = m(h.cuda())
    x = torch.zeros(n, width, device="cuda")
    one = torch.ones(width, dtype=dt, device="cuda")
    P.residual_layer_norm(None, x, one, one, 1e-5, 1.0, *extra)
    rows, index, scores, own = extra
    w = {k: v.double() for k, v in w.items()}
    ids, f = O.route(h.double(), w["router"], w["correction"], top)
    z = (torch.softmax(h.double() @ w["router"].T, -1) + w["correction"]).sort(dim=-1, descending=True).values
    sure = z[:, top - 1] - (z[:, top] if top < E + ident else -9) > 1e-4
    assert sure.float().mean() > 0.9
    want = torch.zeros(n, width, dtype=torch.float64)
    for t in range(n):
        for e, k in zip(ids[t].tolist(), f[t]):
            y = h[t].double() if e >= E else O.gated_mlp(h[t].double(), w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
            want[t] += k * y
    assert rel(x.cpu()[sure], want[sure]) < (6e-3 if dtype == "bf16" else 2e-6)


# ---------------------------------------------------------------------------------------------- the model
def engine(cfg, dtype, seed=0, blocks=12, seqs=4, max_len=256, **kw):
    from tinyllmforge_amd.engine.llm_engine import LLMEngine
    return LLMEngine(cfg, state_dict=C.weights(cfg, seed), dtype={"bf16": "bfloat16", "f32": "float32"}[dtype],
                     kvcache_block_size=64, num_kvcache_blocks=blocks, max_num_seqs=seqs, max_model_len=max_len,
                     **{"max_num_batched_tokens": 1024, **kw})


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", C.CONFIGS)
def test_model_under_every_schedule(dtype, name):
    from tinyllmforge_amd.engine.replay import Replay
    cfg = C.CONFIGS[name]
    prompts = {r: C.tokens(cfg, n, i) for i, (r, n) in enumerate({"a": 171, "b": 66, "c": 130, "d": 23, "e": 64}.items())}
    w = C.weights(cfg)
    want = {r: O.forward(cfg, w, t, torch.float64) for r, t in prompts.items()}
    e = engine(cfg, dtype)
    tol = 0.06 if dtype == "bf16" else 5e-5
    replay = Replay(e)
    schedules = {
        "whole": [[(r, len(t))] for r, t in prompts.items()],
        "decode": [s for r, t in prompts.items() for s in [[(r, len(t) - 20)]] + [[(r, 1)]] * 20],
        "tokens": [[("d", 1)]] * 23,
        "portions": [[("a", 2)], [("a", 61)], [("a", 3)], [("a", 64)], [("a", 41)], [("b", 64)], [("b", 2)], [("c", 129)], [("c", 1)]],
        # four live requests, portions beside single tokens, requests that pause; e takes over d's pages and slot
        "mixed": [[("a", 2), ("b", 29)], [("a", 100), ("b", 1), ("c", 16)], [("d", 20), ("b", 1), ("a", 1), ("c", 64)],
                  [("d", 1), ("c", 1)], [("d", 1), ("b", 3), ("a", 1)], [("d", 1), ("a", 65)], [("e", 33), ("a", 1), ("c", 1), ("b", 31)],
                  [("e", 1), ("c", 1), ("b", 1)], [("c", 47), ("e", 2), ("a", 1)], [("e", 28)]],
    }
    alone = None
    for kind, steps in schedules.items():
        used = {r for parts in steps for r, _ in parts}
        got = run_trace(replay, {r: prompts[r] for r in used}, steps)
        for r in used:
            err = C.logit_error(got[r], want[r][:len(got[r])])
            assert err.max() < tol, (kind, r, int(err.argmax()), err.max().item())
        if kind == "whole":
            alone = got
        else:                                # the cut and the company change rounding only
            for r in used:
                assert C.logit_error(got[r], alone[r][:len(got[r])]).max() < tol, (kind, r)
        if not replay.live:
            assert len(e.scheduler.block_manager.free_block_ids) == 12
        for r in list(replay.live):
            e.scheduler.release(replay.live.pop(r))
    e.exit()


def greedy(cfg, w, prompt, n):
    toks, gaps = list(prompt), []
    for _ in range(n):
        top = O.forward(cfg, w, toks, torch.float32)[-1].topk(2)
        gaps.append((top.values[0] - top.values[1]).item())
        toks.append(int(top.indices[0]))
    return toks[len(prompt):], gaps


@pytest.mark.parametrize("eager", [False, True])
def test_greedy_generation_through_the_scheduler(eager):
    """32-bit: portions of 24 rows, five requests of which three run, a pool that forces preemption, run-ahead decoding."""
    from tinyllmforge_amd.sampling_params import SamplingParams
    cfg = C.config(90, 203, [C.attention_2(3, 1, 20, 13, 12, C.dense(50)), C.attention(4, 2, 9, 21, C.moe(5, 1, 2, 20, 30))], loop=(0, 2, 2), eps=1e-3)
    w = C.weights(cfg)
    prompts = [C.tokens(cfg, n, 50 + n) for n in (50, 61, 9, 1, 33)]
    e = engine(cfg, "f32", blocks=4, seqs=3, max_num_batched_tokens=24, enforce_eager=eager)
    out = e.generate(prompts, SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True))
    for p, o in zip(prompts, out):
        want, gaps = greedy(cfg, w, p, 20)
        got = o["token_ids"]
        first = next((i for i in range(20) if got[i] != want[i]), None)
        assert len(got) == 20 and (first is None or gaps[first] < 1e-4), (len(p), first)
    assert eager or e.steps_ahead > 0
    assert len(e.scheduler.block_manager.free_block_ids) == 4 and len(e.scheduler.state_slots.free) == 3
    e.exit()


def test_bf16_generation_graphs_eager_and_sampling_agree():
    from tinyllmforge_amd.sampling_params import SamplingParams
    cfg = C.CONFIGS["even"]
    prompts = [C.tokens(cfg, n, n) for n in (70, 5, 140)]
    sp = SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True)
    runs = []
    for kw in (dict(), dict(enforce_eager=True), dict(run_ahead=False), dict(blocks=40, max_num_batched_tokens=64)):
        e = engine(cfg, "bf16", **kw)
        runs.append([o["token_ids"] for o in e.generate(prompts, sp)])
        if not kw:
            drawn = e.generate(prompts, SamplingParams(temperature=0.8, max_tokens=6, ignore_eos=True))
            assert all(len(o["token_ids"]) == 6 and max(o["token_ids"]) < cfg["vocab"] for o in drawn)
        e.exit()
    assert runs[0] == runs[2]
    for other, least in ((runs[1], 60), (runs[3], 60)):     # other cuts and splits, other rounding: near ties may go the other way
        assert sum(x == y for a, b in zip(runs[0], other) for x, y in zip(a, b)) > least


@pytest.mark.parametrize("name", ["even", "wide"])
def test_graph_replays_match_eager_steps(name):
    """Captured decode steps, replayed with eager work in between, against eager ones, every replay."""
    from tinyllmforge_amd.engine.replay import Replay
    cfg = C.CONFIGS[name]
    prompts = {"a": C.tokens(cfg, 90, 1), "b": C.tokens(cfg, 60, 2), "c": C.tokens(cfg, 75, 3)}
    steps = [[("a", 60), ("b", 40)]] + [[("a", 1), ("b", 1)]] * 8 + [[("c", 50)]] + [[("c", 1), ("a", 1), ("b", 1)]] * 12
    got = []
    for eager in (False, True):
        e = engine(cfg, "bf16", enforce_eager=eager, max_len=128)
        got.append(run_trace(Replay(e), prompts, steps))
        e.exit()
    for r in prompts:
        assert torch.equal(got[0][r], got[1][r]), r


def test_int8_linears():
    from tinyllmforge_amd.engine.replay import Replay
    cfg = C.CONFIGS["odd"]
    prompt = C.tokens(cfg, 70, 4)
    e = engine(cfg, "bf16", quantization="w8a16")
    got = run_trace(Replay(e), {"a": prompt}, [[("a", 60)]] + [[("a", 1)]] * 10)["a"]
    e.exit()
    assert C.logit_error(got, O.forward(cfg, C.weights(cfg), prompt)).median() < 0.15


def test_long_decoding():
    from tinyllmforge_amd.engine.replay import Replay
    cfg = C.config(64, 80, [C.attention_2(2, 1, 16, 24, 8, C.dense(64)), C.attention(4, 2, 16, 8, C.moe(4, 1, 2, 32, 16), every=100)], loop=(0, 1, 2))
    toks = C.tokens(cfg, 700, 5)
    w = C.weights(cfg)
    want = O.forward(cfg, w, toks, torch.float64)
    for dtype, tol in (("f32", 5e-5), ("bf16", 0.06)):
        e = engine(cfg, dtype, max_len=768)
        got = run_trace(Replay(e), {"a": toks}, [[("a", 1)]] * 700)["a"]
        e.exit()
        err = C.logit_error(got, want)
        assert err.max() < tol, (dtype, int(err.argmax()), err.max().item())


def test_trace_run_program(tmp_path):
    """The command line: its own process, steps on standard input, one file of logits per step."""
    from safetensors.torch import save_file
    cfg = C.config(64, 70, [C.attention_2(2, 1, 16, 12, 8, C.dense(40)), C.attention(3, 3, 8, 16, C.moe(3, 1, 2, 16, 8))], loop=(0, 1, 2))
    w = C.weights(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    a, b = C.tokens(cfg, 30, 1), C.tokens(cfg, 12, 2)
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:25], want=[0, 24])], end=[]),
             dict(step=1, entries=[dict(id="b", tokens=b, want=[]), dict(id="a", tokens=a[25:26], want=[])], end=["b"]),
             dict(step=2, entries=[dict(id="a", tokens=a[26:27], want=[0])], end=["a"])]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "128"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = O.forward(cfg, w, a, torch.float64)
    got = torch.frombuffer(bytearray((tmp_path / "0.f32").read_bytes()), dtype=torch.float32).view(2, 70)
    assert C.logit_error(got, want[[0, 24]]).max() < 5e-5
    got = torch.frombuffer(bytearray((tmp_path / "2.f32").read_bytes()), dtype=torch.float32).view(1, 70)
    assert C.logit_error(got, want[26:27]).max() < 5e-5
    assert not (tmp_path / "1.f32").exists()
