"""Gitopel on the GPU: every kernel against the plain implementation, then the model through the engine."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import gitopel as O
from tests import gitopel_cases as C

pytestmark = pytest.mark.gpu
DTYPES = {"bf16": torch.bfloat16, "f32": torch.float32}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def rel(got, want):
    return ((got.double().cpu() - want.double()).norm() / want.double().norm()).item()


# ---------------------------------------------------------------------------------------------- single kernels
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,groups", [(5, 90, 3), (3, 64, 1), (7, 1024, 4), (2, 4096, 1), (130, 4096, 4), (3, 1500, 2), (1, 20000, 4)])
def test_group_norms(dtype, rows, width, groups):
    from tinyllmforge_amd import ops as P
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g)
    y, bias, wp, wn = (t.to(dt) for t in (r(rows, width + 8), r(width), r(width), r(width)))
    x = 3 * r(rows, width)
    xd = x.cuda()
    eps = 1e-3
    h = P.group_rms_norm_add(y.cuda(), bias.cuda(), wp.cuda(), xd, wn.cuda(), groups, eps)
    want_x = x.double() + O.grouped_rms_norm(y[:, :width].double() + bias.double(), wp.double(), groups, eps)
    assert rel(xd, want_x) < 1e-6
    want_h = O.grouped_rms_norm(want_x, wn.double(), groups, eps)
    assert rel(h, want_h) < (3e-3 if dtype == "bf16" else 1e-6)
    no_bias = P.group_rms_norm_add(y.cuda(), None, wp.cuda(), x.cuda(), wn.cuda(), groups, eps)
    assert rel(no_bias, O.grouped_rms_norm(x.double() + O.grouped_rms_norm(y[:, :width].double(), wp.double(), groups, eps),
                                           wn.double(), groups, eps)) < (3e-3 if dtype == "bf16" else 1e-6)
    ids = torch.tensor([i * 3 % 11 for i in range(rows)])
    table = r(11, width).to(dt)
    xe, he = P.embed_group_rms_norm(ids.cuda(), table.cuda(), wn.cuda(), groups, eps)
    assert torch.equal(xe.cpu(), table[ids].float())
    assert rel(he, O.grouped_rms_norm(table[ids].double(), wn.double(), groups, eps)) < (3e-3 if dtype == "bf16" else 1e-6)


@pytest.mark.parametrize("M,N,K", [(1, 16, 16), (5, 203, 90), (130, 64, 256), (64, 100, 33)])
def test_f32_dense_operations(M, N, K):
    from tinyllmforge_amd import ops as P
    g = torch.Generator().manual_seed(M)
    x, w = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g)
    y = P.linear(x.cuda(), w.cuda())
    assert rel(y, x.double() @ w.double().T) < 1e-6
    z = torch.randn(M, 2 * N, generator=g)
    assert rel(P.silu_and_mul(z.cuda()), O.silu(z[:, :N].double()) * z[:, N:].double()) < 1e-6
    z[:, 0] = z[:, 1] = 9.0
    assert P.argmax(z.cuda()).tolist() == [0] * M
    assert P.argmax((-z.abs()).cuda()).cpu().equal((-z.abs()).argmax(-1))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,rot", [(6, 2, 40, 24), (8, 8, 128, 128), (3, 1, 32, 0), (2, 1, 256, 64), (4, 2, 18, 18), (3, 3, 33, 20)])
def test_attention_preparation(dtype, H, G, D, rot):
    from tinyllmforge_amd import ops as P
    from tinyllmforge_amd.layers.rotary_embedding import rotation_table
    dt, g, n, eps = DTYPES[dtype], torch.Generator().manual_seed(1), 21, 1e-4
    width = (H + G) * D + H
    proj = torch.randn(n, -(-width // 16) * 16, generator=g).to(dt)
    qb, kb = torch.randn(H * D, generator=g).to(dt), torch.randn(G * D, generator=g).to(dt)
    pos = torch.randint(0, 900, (n,), generator=g)
    kv = P.PooledKV(3, 64, G, D, 8, 8, dt, "cuda")
    slots = torch.randperm(3 * 64, generator=g)[:n].to(torch.int32)
    slots[4] = -1
    table = rotation_table(rot, 900, 777.0)
    q, gate = P.attn_prep(proj.cuda(), qb.cuda(), kb.cuda(), pos.cuda(), table.cuda(), rot, slots.cuda(), kv.k, kv.v, H, D, eps)
    qr = (proj[:, :H * D].double() + qb.double()).view(n, H, D)
    kr = (proj[:, H * D:(H + G) * D].double() + kb.double()).view(n, G, D)
    turn = lambda x: O.unit_rms(O.rotate_interleaved_fast(x, pos.tolist(), rot, 777.0), eps)
    tol = 4e-3 if dtype == "bf16" else 2e-6
    assert rel(q[..., :D], turn(qr)) < tol and not q[..., D:].any()
    assert rel(gate, torch.sigmoid(proj[:, (H + G) * D:width].double())) < 1e-5
    live = slots >= 0
    rows = slots[live].long()
    dp = kv.k.shape[3]
    kc, vc = kv.k.view(-1, G, dp).cpu(), kv.v.view(-1, G, dp).cpu()
    assert rel(kc[rows][..., :D], turn(kr)[live]) < tol and rel(vc[rows][..., :D], kr[live]) < tol
    assert not kc[..., D:].any() and not vc[..., D:].any()
    rest = torch.ones(3 * 64, dtype=torch.bool)
    rest[rows] = False
    assert not kc[rest].any() and not vc[rest].any()


class Pages:
    """Caches of a few sequences in shuffled pages, and the calls of one step as the layer makes them."""

    def __init__(self, lens, H, G, D, size, pool, dt, bs=64, seed=0):
        from tinyllmforge_amd import ops as P
        self.P, self.H, self.G, self.D, self.size, self.pool, self.dt, self.bs = P, H, G, D, size, pool, dt, bs
        g = torch.Generator().manual_seed(seed)
        need = [-(-n // bs) for n in lens]
        perm = torch.randperm(sum(need) + 2, generator=g).tolist()
        self.bt = torch.full((len(lens), max(need)), -1, dtype=torch.int32)
        for s, n in enumerate(need):
            self.bt[s, :n] = torch.tensor([perm.pop() for _ in range(n)], dtype=torch.int32)
        self.kv = P.PooledKV(sum(need) + 2, bs, G, D, pool, size, dt, "cuda")
        for t in (self.kv.k, self.kv.v, self.kv.pk, self.kv.pv):
            t.fill_(3.0)                                    # stale contents of reused pages
            t[..., D:] = 0
        self.done = [0] * len(lens)

    def step(self, parts, q, k, v, bias, scale, gate=None):
        """``parts``: (sequence, tokens); single tokens first.  Returns ``{sequence: [tokens, H, D]}``."""
        P, bs = self.P, self.bs
        parts = sorted(parts, key=lambda x: x[1] > 1)
        single = sum(n == 1 for _, n in parts)
        pos = torch.cat([torch.arange(self.done[s], self.done[s] + n) for s, n in parts])
        row = torch.cat([torch.full((n,), i) for i, (_, n) in enumerate(parts)])
        bt = self.bt[[s for s, _ in parts]]
        slots = (bt[row, pos // bs].long() * bs + pos % bs).to(torch.int32)
        dp = self.kv.k.shape[3]
        pad = lambda x: torch.nn.functional.pad(x, (0, dp - self.D)).to(self.dt).cuda()
        take = lambda x: torch.cat([x[s][self.done[s]:self.done[s] + n] for s, n in parts])
        self.kv.k.view(-1, self.G, dp)[slots.long().cuda()] = pad(take(k))
        self.kv.v.view(-1, self.G, dp)[slots.long().cuda()] = pad(take(v))
        qd = pad(take(q))
        n = len(pos)
        cu = torch.tensor([0] + torch.tensor([m for _, m in parts]).cumsum(0).tolist(), dtype=torch.int32).cuda()
        starts = torch.tensor([self.done[s] for s, _ in parts], dtype=torch.int32).cuda()
        ones = torch.ones(n, self.H, device="cuda") if gate is None else take(gate).float().cuda()
        out = torch.full((n, self.H * self.D), 7.0, dtype=self.dt, device="cuda")
        b, btd, posd, sd, rowd = bias.to(self.dt).cuda(), bt.cuda(), pos.cuda(), slots.cuda(), row.to(torch.int32).cuda()
        most = max(m for _, m in parts)
        if single:
            P.pooled_attention_rows(qd[:single], b, ones[:single], self.kv, btd, posd[:single], sd[:single], scale, 2048,
                                    out[:single], pool_new=True)
        if single < n:
            P.pool_blocks(self.kv, btd, cu, starts, single, len(parts) - single, most)
            if self.dt == torch.bfloat16:
                P.pooled_attention_prefill(qd, b, ones, self.kv, btd, cu, starts, single, len(parts) - single, most, scale, out)
            else:
                P.pooled_attention_rows(qd[single:], b, ones[single:], self.kv, btd, posd[single:], sd[single:], scale,
                                        2048, out[single:], row_seq=rowd[single:])
        res, at = {}, 0
        for s, m in parts:
            res[s] = out[at:at + m].view(m, self.H, self.D).cpu()
            at += m
            self.done[s] += m
        return res


ATTN = [(4, 2, 40, 37, 5), (8, 2, 64, 80, 16), (1, 1, 32, 1, 1), (6, 6, 96, 64, 64), (20, 1, 128, 130, 100), (3, 1, 256, 9, 3), (2, 2, 160, 200, 7), (4, 2, 27, 30, 6)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,size,pool", ATTN)
def test_attention_over_portions_singles_and_mixtures(dtype, H, G, D, size, pool):
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(D)
    lens = [150, 67, 210]
    rnd = lambda n, h: torch.randn(n, h, D, generator=g).to(dt).float()
    q, k, v = [rnd(n, H) for n in lens], [rnd(n, G) for n in lens], [rnd(n, G) for n in lens]
    gate = [torch.rand(n, H, generator=g) for n in lens]
    bias, scale = (torch.randn(H, generator=g) - 2).to(dt).float(), 1.5 / D ** 0.5
    want = [O.sigmoid_attention(q[s].double(), k[s].double(), v[s].double(), bias.double(), scale, size, pool) * gate[s].double()[..., None]
            for s in range(3)]
    schedules = {
        "whole": [[(0, 150), (1, 67), (2, 210)]],
        "portions": [[(0, 2), (1, 3)], [(0, 62), (2, 130)], [(0, 1), (1, 2), (2, 2)], [(0, 85), (1, 62), (2, 78)]],
        "mixed": [[(0, 100), (2, 64)], [(0, 1), (1, 20), (2, 1)]] + [[(0, 1), (1, 1), (2, 29)], [(0, 1), (2, 2)]] * 3 +
                 [[(0, 43), (1, 1)], [(1, 43), (2, 52)]],
        "single": [[(0, 1), (1, 1), (2, 1)] for _ in range(67)] + [[(0, 1), (2, 1)] for _ in range(83)] + [[(2, 1)] for _ in range(60)],
    }
    tol = 6e-3 if dtype == "bf16" else 3e-6
    for name, steps in schedules.items():
        if name == "single" and dtype == "f32" and D > 64:
            continue
        pages = Pages(lens, H, G, D, size, pool, dt)
        got = [[], [], []]
        for parts in steps:
            for s, o in pages.step(parts, q, k, v, bias, scale, gate).items():
                got[s].append(o)
        for s in range(3):
            assert rel(torch.cat(got[s]), want[s]) < tol, (name, s)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size,pool,n", [(37, 5, 140), (64, 16, 300), (100, 12, 260), (20, 70, 200), (1, 1, 70)])
def test_one_key_stands_out_at_every_edge(dtype, size, pool, n):
    """All weights but those of one token (and of its block's mean) vanish: the output names the keys a position saw."""
    dt, H, G, D = DTYPES[dtype], 2, 1, 32
    scale, bias = 1.0, torch.full((H,), -40.0)
    edges = sorted({0, 1, pool - 1, pool, 63, 64, n - size - 1, n - size, n - size + 1, (n - size) // pool * pool,
                    (n - size) // pool * pool - 1, n - 2} & set(range(n - 1)))
    for j in edges:
        q, k = torch.zeros(n, H, D), torch.zeros(n, G, D)
        q[:, :, 0] = 8.0
        k[j, :, 0] = 8.0 * max(pool, 2)                 # the block's mean still scores far above the bias
        v = torch.zeros(n, G, D)
        v[:, 0, :] = torch.arange(n)[:, None] % 50 + 1.0
        v = v.to(dt).float()
        want = O.sigmoid_attention(q.double(), k.double(), v.double(), bias.double(), scale, size, pool)
        for cuts in ([n], [n - 3, 1, 1, 1], [2] * (n // 2) + [1] * (n % 2), [size, n - size]):
            pages = Pages([n], H, G, D, size, pool, dt)
            got = torch.cat([pages.step([(0, c)], [q], [k], [v], bias, scale)[0] for c in cuts if c > 0])
            err = (got.double() - want).abs().amax(dim=(1, 2))
            assert err.max() < 0.25, (j, cuts[:2], int(err.argmax()), err.max().item())
    # a difference of one key is at least 1 (values are whole numbers), of one block's mean at least the mean itself


GLA = [(3, 24, 20, 5), (2, 64, 64, 16), (1, 16, 16, 1), (2, 128, 256, 16), (1, 256, 512, 33), (2, 100, 50, 7), (1, 5, 3, 2)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv,rank", GLA)
@pytest.mark.parametrize("decay", ["usual", "none", "harsh"])
def test_gated_linear_attention(dtype, H, dk, dv, rank, decay):
    from tinyllmforge_amd import ops as P
    from tinyllmforge_amd.engine import inputs as I
    dt, g, eps = DTYPES[dtype], torch.Generator().manual_seed(dk + dv), 1e-5
    tau = {"usual": 8.0, "none": 1e4, "harsh": 0.5}[decay]
    lens = [61, 18]
    width = 2 * H * (dk + dv) + rank
    proj = [torch.randn(n, width, generator=g).to(dt) for n in lens]
    a2 = (torch.randn(H * dk, rank, generator=g) * (8 if decay == "harsh" else 1)).to(dt)
    a2b, nw = torch.randn(H * dk, generator=g).to(dt), torch.randn(dv, generator=g).to(dt)

    def plain(p):
        p = p.double()
        q, k, v, gt, r = p.split([H * dk, H * dk, H * dv, H * dv, rank], dim=1)
        z = (r @ a2.double().T + a2b.double()).view(-1, H, dk)
        la = -torch.nn.functional.softplus(-z) / tau
        o, s = O.gla_recurrence(q.view(-1, H, dk) * dk ** -0.5, k.view(-1, H, dk), v.view(-1, H, dv), la)
        return (O.unit_rms(o, eps) * nw.double()).reshape(-1, H * dv) * O.silu(gt), s

    want = [plain(p) for p in proj]
    slots = torch.tensor([2, 0])
    schedules = {
        "whole": [[61, 18]], "portions": [[2, 3], [15, 2], [17, 0], [16, 13], [11, 0]],
        "mixed": [[20, 1], [1, 0], [1, 2], [2, 1], [33, 1], [1, 13], [3, 0]], "single": [[1, 1]] * 18 + [[1, 0]] * 43,
    }
    dev = lambda x: x.cuda()
    for name, steps in schedules.items():
        state = torch.full((3, H, dk, dv), 5.0, device="cuda")     # what a finished sequence left behind
        done, got = [0, 0], [[], []]
        for step in steps:
            order = sorted((s for s in (0, 1) if step[s]), key=lambda s: step[s] > 1)
            ns = [step[s] for s in order]
            rows = dev(torch.cat([proj[s][done[s]:done[s] + n] for s, n in zip(order, ns)]))
            pos = dev(torch.cat([torch.arange(done[s], done[s] + n) for s, n in zip(order, ns)]))
            single = sum(n == 1 for n in ns)
            out = torch.full((rows.shape[0], H * dv), 7.0, dtype=dt, device="cuda")
            sl = dev(slots[order].to(torch.int32))
            w = (dev(a2), dev(a2b), dev(nw), state, sl)
            if single:
                P.gla_decode(rows[:single], *w, pos[:single], tau, eps, out[:single])
            if single < rows.shape[0]:
                first, crow, clen, cu = 0, [], [], [0]
                for n in ns[single:]:
                    crow += list(range(first, first + n, I.CHUNK))
                    clen += [min(I.CHUNK, n - c) for c in range(0, n, I.CHUNK)]
                    cu.append(len(crow))
                    first += n
                t = lambda x: torch.tensor(x, dtype=torch.int32, device="cuda")
                P.gla_portions(rows[single:], *w, dev(torch.tensor([done[s] for s in order], dtype=torch.int32)), t(crow),
                               t(clen), t(cu), single, len(ns) - single, tau, eps, out[single:])
            at = 0
            for s, n in zip(order, ns):
                got[s].append(out[at:at + n].cpu())
                done[s] += n
                at += n
        for s in (0, 1):
            assert rel(torch.cat(got[s]), want[s][0]) < (4e-3 if dtype == "bf16" else 2e-5), (name, s)
            assert rel(state[slots[s]], want[s][1]) < 2e-5, (name, s)
        assert (state[1] == 5.0).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lens,start", [([1200], 0), ([700, 515], 0), ([900], 5)])
def test_gated_linear_attention_in_segments(dtype, lens, start):
    """Prompts long enough for the kernels to cut a sequence into segments, from zero and from a state."""
    from tinyllmforge_amd import ops as P
    dt, g, eps, tau = DTYPES[dtype], torch.Generator().manual_seed(7), 1e-5, 16.0
    H, dk, dv, rank = 2, 48, 40, 4
    proj = [torch.randn(n, 2 * H * (dk + dv) + rank, generator=g).to(dt) for n in lens]
    a2, a2b, nw = torch.randn(H * dk, rank, generator=g).to(dt), 3 + torch.randn(H * dk, generator=g).to(dt), torch.randn(dv, generator=g).to(dt)
    first = [torch.randn(H, dk, dv, generator=g) for _ in lens]
    state = torch.stack([torch.full((H, dk, dv), 5.0)] + first).cuda()
    rows = torch.cat(proj).cuda()
    out = torch.empty(rows.shape[0], H * dv, dtype=dt, device="cuda")
    crow, clen, cu, at = [], [], [0], 0
    for n in lens:
        crow += list(range(at, at + n, 16))
        clen += [min(16, n - c) for c in range(0, n, 16)]
        cu.append(len(crow))
        at += n
    t = lambda x: torch.tensor(x, dtype=torch.int32, device="cuda")
    P.gla_portions(rows, a2.cuda(), a2b.cuda(), nw.cuda(), state, t([i + 1 for i in range(len(lens))]), t([start] * len(lens)),
                   t(crow), t(clen), t(cu), 0, len(lens), tau, eps, out)
    at = 0
    for i, n in enumerate(lens):
        p = proj[i].double()
        q, k, v, gt, r = p.split([H * dk, H * dk, H * dv, H * dv, rank], dim=1)
        la = -torch.nn.functional.softplus(-(r @ a2.double().T + a2b.double())).view(-1, H, dk) / tau
        o, s = O.gla_recurrence(q.view(-1, H, dk) * dk ** -0.5, k.view(-1, H, dk), v.view(-1, H, dv), la,
                                first[i].double() if start else None)
        want = (O.unit_rms(o, eps) * nw.double()).reshape(-1, H * dv) * O.silu(gt)
        assert rel(out[at:at + n], want) < (4e-3 if dtype == "bf16" else 2e-5)
        assert rel(state[i + 1], s) < 2e-5
        at += n
    assert (state[0] == 5.0).all()


@pytest.mark.parametrize("quantized", [False, True])
def test_consumers_add_up_split_projections(quantized):
    """A projection left as partial sums gives the bits of the finished one, in every kernel that may read it."""
    from tinyllmforge_amd import ops as P
    from tinyllmforge_amd.layers.linear import quantize_per_channel
    from tinyllmforge_amd.layers.rotary_embedding import rotation_table
    g, n, K = torch.Generator().manual_seed(2), 40, 4096
    bf = lambda *s: torch.randn(*s, generator=g).to(torch.bfloat16).cuda()

    def both(N):
        x, w = bf(n, K), bf(N, K) * K ** -0.5
        if quantized:
            q, scale = quantize_per_channel(w)
            packed = P.pack_w8(q)
            return P.w8a16_linear(x, packed, scale), P.linear_deferred(x, packed, scale)
        return P.bf16_linear(x, w), P.linear_deferred(x, w)

    y, d = both(1024)
    assert d.splits > 1, "this size is meant to split K"
    x, wp, wn, b = torch.randn(n, 1024, generator=g).cuda(), bf(1024), bf(1024), bf(1024)
    x2 = x.clone()
    h2 = P.group_rms_norm_add(d, b, wp, x2, wn, 4, 1e-6)
    h1 = P.group_rms_norm_add(y, b, wp, x, wn, 4, 1e-6)
    assert torch.equal(h1, h2) and torch.equal(x, x2)
    H, G, D = 8, 2, 96
    y, d = both(-(-((H + G) * D + H) // 16) * 16)
    assert d.splits > 1
    tab, pos, slots = rotation_table(64, 100, 1e4).cuda(), torch.arange(n).cuda(), torch.arange(n, dtype=torch.int32).cuda()
    kv = [P.PooledKV(1, 64, G, D, 8, 8, torch.bfloat16, "cuda") for _ in range(2)]
    args = lambda c: (None, None, pos, tab, 64, slots, c.k, c.v, H, D, 1e-6)
    q2, g2 = P.attn_prep(d, *args(kv[1]))
    q1, g1 = P.attn_prep(y, *args(kv[0]))
    assert torch.equal(q1, q2) and torch.equal(g1, g2) and torch.equal(kv[0].k, kv[1].k) and torch.equal(kv[0].v, kv[1].v)
    H, dk, dv, r = 2, 48, 72, 16
    y, d = both(2 * H * (dk + dv) + r)
    assert d.splits > 1
    st = torch.randn(n, H, dk, dv, generator=g).cuda()
    st2 = st.clone()
    a2, a2b, nw, sl = bf(H * dk, r), bf(H * dk), bf(dv), torch.arange(n, dtype=torch.int32).cuda()
    outs = [torch.empty(n, H * dv, dtype=torch.bfloat16, device="cuda") for _ in range(2)]
    P.gla_decode(d, a2, a2b, nw, st2, sl, pos, 8.0, 1e-6, outs[1])
    P.gla_decode(y, a2, a2b, nw, st, sl, pos, 8.0, 1e-6, outs[0])
    assert torch.equal(outs[0], outs[1]) and torch.equal(st, st2)


# ---------------------------------------------------------------------------------------------- the model
def engine(cfg, dtype, seed=0, blocks=12, seqs=4, max_len=256, **kw):
    from tinyllmforge_amd.engine.llm_engine import LLMEngine
    return LLMEngine(cfg, state_dict=C.weights(cfg, seed), dtype={"bf16": "bfloat16", "f32": "float32"}[dtype],
                     kvcache_block_size=64, num_kvcache_blocks=blocks, max_num_seqs=seqs, num_state_slots=seqs,
                     max_model_len=max_len, **{"max_num_batched_tokens": 1024, **kw})


def run_trace(replay, prompts, steps):
    """``steps``: lists of (request, tokens).  Logits of every position, per request."""
    at, got = {r: 0 for r in prompts}, {r: [] for r in prompts}
    for parts in steps:
        entries = [dict(id=r, tokens=prompts[r][at[r]:at[r] + n], want=list(range(n))) for r, n in parts]
        for r, n in parts:
            at[r] += n
        logits = replay.step(entries, [r for r, _ in parts if at[r] == len(prompts[r])])
        lo = 0
        for r, n in parts:
            got[r].append(logits[lo:lo + n])
            lo += n
    return {r: torch.cat(x) for r, x in got.items()}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", C.CONFIGS)
def test_model_under_every_schedule(dtype, name):
    from tinyllmforge_amd.engine.replay import Replay
    cfg = C.CONFIGS[name]
    prompts = {r: C.tokens(cfg, n, i) for i, (r, n) in enumerate({"a": 171, "b": 66, "c": 130, "d": 23, "e": 64}.items())}
    w = C.weights(cfg)
    want = {r: O.forward(cfg, w, t, torch.float64) for r, t in prompts.items()}
    e = engine(cfg, dtype)
    # the plain implementation with its weights as they are is exact; bf16 runs differ by rounding
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
            assert len(e.scheduler.block_manager.free_block_ids) == 12 and len(e.scheduler.state_slots.free) == 4
        for r in list(replay.live):
            e.scheduler.release(replay.live.pop(r))
    e.exit()


def greedy(cfg, w, prompt, n, dtype=torch.float32):
    toks = list(prompt)
    gaps = []
    for _ in range(n):
        top = O.forward(cfg, w, toks, dtype)[-1].topk(2)
        gaps.append((top.values[0] - top.values[1]).item())
        toks.append(int(top.indices[0]))
    return toks[len(prompt):], gaps


@pytest.mark.parametrize("eager", [False, True])
def test_greedy_generation_through_the_scheduler(eager):
    """32-bit: portions of 24 rows, five requests for three slots, a pool that forces preemption, run-ahead decoding."""
    from tinyllmforge_amd.sampling_params import SamplingParams
    cfg = C.CONFIGS["odd"]
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
    prompts = [C.tokens(cfg, n, n) for n in (70, 5, 128)]
    sp = SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True)
    runs = []
    for kw in (dict(), dict(enforce_eager=True), dict(run_ahead=False), dict(blocks=40, max_num_batched_tokens=64)):
        e = engine(cfg, "bf16", **kw)
        runs.append([o["token_ids"] for o in e.generate(prompts, sp)])
        if not kw:
            drawn = e.generate(prompts, SamplingParams(temperature=0.8, max_tokens=6, ignore_eos=True))
            assert all(len(o["token_ids"]) == 6 and max(o["token_ids"]) < cfg["vocab"] for o in drawn)
        e.exit()
    assert runs[0] == runs[1] == runs[2]
    same = [sum(x == y for x, y in zip(a, b)) for a, b in zip(runs[0], runs[3])]
    assert sum(same) > 60                    # other cuts, other rounding: near ties may go the other way


def test_graph_replays_match_eager_steps():
    """Captured decode steps, replayed with eager work in between, against eager ones: the same logits each time."""
    from tinyllmforge_amd.engine.replay import Replay
    cfg = C.CONFIGS["even"]
    prompts = {"a": C.tokens(cfg, 90, 1), "b": C.tokens(cfg, 60, 2), "c": C.tokens(cfg, 75, 3)}
    steps = [[("a", 60), ("b", 40)]] + [[("a", 1), ("b", 1)]] * 8 + [[("c", 50)]] + [[("c", 1), ("a", 1), ("b", 1)]] * 12
    got = []
    for eager in (False, True):
        e = engine(cfg, "bf16", enforce_eager=eager)
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
    cfg = C.config(64, 2, 80, [C.attention(2, 1, 32, 32, 24, 6), C.gla(2, 32, 32, ff=64)])
    toks = C.tokens(cfg, 700, 5)
    e = engine(cfg, "f32", max_len=768)
    got = run_trace(Replay(e), {"a": toks}, [[("a", 1)]] * 700)["a"]
    e.exit()
    err = C.logit_error(got, O.forward(cfg, C.weights(cfg), toks, torch.float64))
    assert err.max() < 5e-5, (int(err.argmax()), err.max().item())


def test_trace_run_program(tmp_path):
    """The command line: its own process, steps on standard input, one file of logits per step."""
    from safetensors.torch import save_file
    cfg = C.config(64, 2, 70, [C.attention(2, 1, 32, 32, 10, 4, ff=64), C.gla(2, 32, 32, rank=3)])
    w = C.weights(cfg)
    for layer in cfg["layers"]:
        layer["mixer"].pop("rank", None)
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
    cfg["layers"][1]["mixer"]["rank"] = 3
    want = O.forward(cfg, w, a, torch.float64)
    got = torch.frombuffer(bytearray((tmp_path / "0.f32").read_bytes()), dtype=torch.float32).view(2, 70)
    assert C.logit_error(got, want[[0, 24]]).max() < 5e-5
    got = torch.frombuffer(bytearray((tmp_path / "2.f32").read_bytes()), dtype=torch.float32).view(1, 70)
    assert C.logit_error(got, want[26:27]).max() < 5e-5
    assert not (tmp_path / "1.f32").exists()
