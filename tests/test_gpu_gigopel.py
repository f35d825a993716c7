"""Gigopel on the GPU: every kernel against the plain implementation, then the model through the engine."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import gigopel as O
from tests import gigopel_cases as C
from tests.test_gpu_gitopel import run_trace

pytestmark = pytest.mark.gpu
DTYPES = {"bf16": torch.bfloat16, "f32": torch.float32}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def rel(got, want):
    return ((got.double().cpu() - want.double()).norm() / want.double().norm()).item()


# ---------------------------------------------------------------------------------------------- single kernels
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,top", [(5, 90, 0), (3, 64, 2), (7, 1024, 1), (130, 4096, 3), (2, 20, 5)])
def test_residual_norm(dtype, rows, width, top):
    from tinyllmforge_amd import ops as P
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g)
    y, w, x = r(rows, width + 8).to(dt), (0.3 * r(width)).to(dt), 3 * r(rows, width)
    extra, index = r(rows * max(top, 1), width).to(dt), torch.randperm(rows * max(top, 1), generator=g).view(rows, -1).to(torch.int32)
    for offset in (1.0, 0.0):
        xd = x.cuda()
        args = (extra.cuda(), index.cuda()) if top else ()
        h = P.residual_rms_norm(y.cuda(), xd, 0.35, w.cuda(), offset, 1e-3, *args)
        add = y[:, :width].double() + (extra.double()[index.long()].sum(1) if top else 0)
        want = x.double() + 0.35 * add
        assert rel(xd, want) < 1e-6
        assert rel(h, want / O.rms(want, 1e-3) * (offset + w.double())) < (3e-3 if dtype == "bf16" else 1e-6)
    table = r(11, width).to(dt)
    ids = torch.tensor([i * 3 % 11 for i in range(rows)])
    xe, he = P.embed_group_rms_norm(ids.cuda(), table.cuda(), w.cuda(), 1, 1e-3, 1.0)
    assert torch.equal(xe.cpu(), table[ids].float())
    assert rel(he, O.zero_centred_norm(table[ids].double(), w.double(), 1e-3)) < (3e-3 if dtype == "bf16" else 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cols,padded,col,ld", [(50, 64, 7, 90), (192, 192, 64, 256), (1, 64, 3, 5), (1000, 1024, 8, 1008)])
def test_xielu(dtype, cols, padded, col, ld):
    from tinyllmforge_amd import ops as P
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(cols)
    x = (3 * torch.randn(9, ld, generator=g)).to(dt)
    x[0, col] = 0.0
    if cols > 6:
        x[0, col + 1:col + 6] = torch.tensor([-0.06, -0.0626, -1e-3, -40.0, 30.0]).to(dt)
    pq = torch.tensor([0.7, -1.3]).to(dt)
    out = torch.full((9, padded + 64), 7.0, dtype=dt, device="cuda")
    P.xielu(x.cuda(), col, cols, pq.cuda(), out[:, 64:])
    want = O.xielu(x[:, col:col + cols].double(), *pq.double())
    assert rel(out[:, 64:64 + cols], want) < (3e-3 if dtype == "bf16" else 1e-6)
    # near zero the function is z / 2 and a small term that must not drown in cancellation
    small = want.abs() < 0.1
    assert ((out[:, 64:64 + cols].double().cpu() - want).abs()[small] <= 8e-3 * want.abs()[small] + 1e-7).all()
    assert not out[:, 64 + cols:].any() and (out[:, :64] == 7).all()


@pytest.mark.parametrize("M,parts,width,ff_pad", [(600, (40, 72), 128, 128), (513, (24, 50), 192, 64), (3000, (1000, 3000), 256, 3008), (700, (8, 64), 64, 64)])
def test_projection_with_an_activated_part(M, parts, width, ff_pad):
    """Many rows: the stacked product applies the activation itself; as the two kernels do up to the bf16 rounding between."""
    from tinyllmforge_amd import ops as P
    from tinyllmforge_amd.layers.activation import XIELU
    from tinyllmforge_amd.layers.linear import StackedLinear
    g = torch.Generator().manual_seed(M)
    torch.set_default_dtype(torch.bfloat16)
    lin, act = StackedLinear(width, {"a": parts[0], "up": parts[1]}).cuda(), XIELU().cuda()
    torch.set_default_dtype(torch.float32)
    w = (torch.randn(sum(parts), width, generator=g) * 2 * width ** -0.5).to(torch.bfloat16)
    lin.weight.data[:sum(parts), :width] = w.cuda()
    act.pq.data.copy_(torch.tensor([0.4, -0.8]))
    x = torch.randn(M, width, generator=g).to(torch.bfloat16)
    out = torch.full((M, ff_pad + 64), 7.0, dtype=torch.bfloat16, device="cuda")
    y = lin.forward_activated(x.cuda(), "up", act, out[:, 64:])
    assert isinstance(y, torch.Tensor)
    z = x.double() @ w.double().T
    assert rel(y[:, :parts[0]], z[:, :parts[0]]) < 3e-3
    assert rel(out[:, 64:64 + parts[1]], O.xielu(z[:, parts[0]:], *act.pq.double().cpu())) < 3e-3
    assert (out[:, :64] == 7).all()
    few = torch.zeros(100, ff_pad, dtype=torch.bfloat16, device="cuda")
    lin.forward_activated(x[:100].cuda(), "up", act, few)                  # too few rows for it: two kernels
    assert rel(few[:, :parts[1]], O.xielu(z[:100, parts[0]:], *act.pq.double().cpu())) < 6e-3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,H,N,K", [(1, 3, 64, 32), (5, 2, 48, 96), (130, 4, 576, 192), (67, 1, 16, 64)])
def test_head_products(dtype, rows, H, N, K):
    from tinyllmforge_amd import ops as P
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(rows)
    x, w = torch.randn(rows, H, K, generator=g).to(dt), torch.randn(H, N, K, generator=g).to(dt)
    tol = 3e-3 if dtype == "bf16" else 1e-6
    assert rel(P.head_gemm(x.cuda(), w.cuda()), torch.einsum("rhk,hnk->rhn", x.double(), w.double())) < tol
    w[:, :32, 32:] = 0            # rows below n_main read k_main columns
    assert rel(P.head_gemm(x.cuda(), w.cuda(), 32, 32), torch.einsum("rhk,hnk->rhn", x.double(), w.double())) < tol


class Attention:
    """A layer of latent attention with a few sequences in shuffled pages, run step by step as the engine does."""

    def __init__(self, sizes, window, lens, dt, seed=0, bs=64, scale=None, long_portion=128, uk=None, uv=None):
        from tinyllmforge_amd.engine.sequence import Sequence
        from tinyllmforge_amd.layers.latent_attention import LatentAttention
        from tinyllmforge_amd.layers.rotary_embedding import rotation_table
        Sequence.block_size = bs
        self.H, self.D, self.R, self.V, self.rank = sizes
        self.window, self.lens, self.dt, self.bs, self.long = window, lens, dt, bs, long_portion
        self.base, self.eps, self.scale = 500.0, 1e-5, scale or 2.0 / (self.D + self.R) ** 0.5
        g = torch.Generator().manual_seed(seed)
        rnd = lambda *s: torch.randn(*s, generator=g)
        self.uk = (rnd(self.H * self.D, self.rank) * self.rank ** -0.5 if uk is None else uk).to(dt)
        self.uv = (rnd(self.H * self.V, self.rank) * self.rank ** -0.5 if uv is None else uv).to(dt)
        self.norm = (1 + 0.2 * rnd(self.rank) if uk is None else torch.ones(self.rank)).to(dt)
        torch.set_default_dtype(dt)
        self.layer = LatentAttention(self.H, self.D, self.R, self.rank, self.V, self.scale, window, 0,
                                     rotation_table(self.R, max(lens) + 1, self.base), self.eps, dt).cuda()
        torch.set_default_dtype(torch.float32)
        for p, v in ((self.layer.uk, self.uk), (self.layer.uv, self.uv), (self.layer.norm.weight, self.norm)):
            p.data.copy_(v)
        self.layer.pack_()
        need = [-(-n // bs) for n in lens]
        perm = torch.randperm(sum(need) + 2, generator=g).tolist()
        self.layer.bind_pages(sum(need) + 2, bs, "cuda")
        self.layer.cache.fill_(3.0)                              # stale contents of reused pages
        self.seqs = []
        for n, k in zip(lens, need):
            s = Sequence([0] * n)
            s.block_table = [perm.pop() for _ in range(k)]
            self.seqs.append(s)
        self.col = self.H * (self.D + self.R) + 3 * (self.D % 8 != 0)
        self.width = self.col + self.rank + self.R + 5

    def step(self, proj, parts):
        """``parts``: (sequence, tokens), in the engine's order of kinds.  Returns ``{sequence: [tokens, H * V]}``."""
        from tinyllmforge_amd.engine import inputs as I
        from tinyllmforge_amd.utils.context import reset_context, set_portions_context
        parts = sorted(parts, key=lambda x: I.portion_kind(x[1], self.long))
        seqs = [self.seqs[s] for s, _ in parts]
        for s, (_, n) in zip(seqs, parts):
            s.num_scheduled = n
        d = I.portion_inputs(seqs, self.bs, self.long, (self.window,))
        d = {k: torch.from_numpy(v).cuda() if hasattr(v, "dtype") else v for k, v in d.items()}
        d.pop("input_ids")
        pos = d.pop("positions")
        rows = torch.cat([proj[i][s.num_computed:s.num_computed + n] for s, (i, n) in zip(seqs, parts)]).to(self.dt).cuda()
        set_portions_context(max_len=max(self.lens), **d)
        out = torch.full((rows.shape[0], self.H * self.V + 8), 7.0, dtype=self.dt, device="cuda")
        self.layer(self.layer.prepare(rows, self.col, pos), pos, out)
        reset_context()
        assert (out[:, self.H * self.V:] == 7).all()
        got, at = {}, 0
        for s, (i, n) in zip(seqs, parts):
            got[i] = out[at:at + n, :self.H * self.V].cpu()
            at += n
            s.num_computed += n
        return got

    def want(self, proj):
        p = proj.to(self.dt).double()
        T, H, D, R = p.shape[0], self.H, self.D, self.R
        turn = lambda x: O.rotate_interleaved_fast(x, list(range(T)), R, self.base)
        q = p[:, :H * (D + R)].reshape(T, H, D + R)
        q = torch.cat([q[..., :D], turn(q[..., D:])], dim=-1)
        low = p[:, self.col:self.col + self.rank + R]
        c = O.plain_norm(low[:, :self.rank], self.norm.double(), self.eps)
        k, v = O.latent_keys_values(c, turn(low[:, None, self.rank:])[:, 0], self.uk.double(), self.uv.double(), H)
        return O.softmax_attention(q, k, v, self.scale, self.window).reshape(T, -1)


# heads, dim, rotated dim, value dim, latent; window.  Every width of the tile kernel (64 ... 576), one and two column tiles,
# several passes over the heads; beyond its sizes in the last two
ATTN = [((3, 20, 6, 13, 27), 37), ((4, 64, 32, 64, 96), 80), ((1, 1, 2, 1, 1), 1), ((20, 32, 16, 48, 176), 64), ((5, 24, 8, 8, 200), 130),
        ((40, 16, 8, 24, 300), 200), ((2, 96, 48, 72, 384), 7), ((17, 40, 24, 128, 440), 100), ((2, 130, 64, 40, 512), 90),
        ((16, 128, 62, 128, 500), 65), ((6, 200, 40, 33, 64), 30), ((2, 48, 16, 150, 130), 50), ((2, 40, 8, 16, 700), 40)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes,window", ATTN)
def test_attention_over_portions_singles_and_mixtures(dtype, sizes, window):
    dt = DTYPES[dtype]
    lens = [150, 67, 210]
    tol = 1.2e-2 if dtype == "bf16" else 4e-6
    schedules = {
        "whole": [[(0, 150), (1, 67), (2, 210)]],
        "portions": [[(0, 2), (1, 3)], [(0, 62), (2, 130)], [(0, 1), (1, 2), (2, 2)], [(0, 85), (1, 62), (2, 78)]],
        "mixed": [[(0, 100), (2, 64)], [(0, 1), (1, 20), (2, 1)]] + [[(0, 1), (1, 1), (2, 29)], [(0, 1), (2, 2)]] * 3 +
                 [[(0, 43), (1, 1)], [(1, 43), (2, 52)]],
        "single": [[(0, 1), (1, 1), (2, 1)] for _ in range(67)] + [[(0, 1), (2, 1)] for _ in range(83)] + [[(2, 1)] for _ in range(60)],
    }
    want = None
    for long_portion in (128, 20) if dtype == "bf16" else (128,):
        for name, steps in schedules.items():
            if name == "single" and long_portion == 20:
                continue
            a = Attention(sizes, window, lens, dt, long_portion=long_portion)
            g = torch.Generator().manual_seed(5)
            proj = [torch.randn(n, a.width, generator=g) for n in lens]
            if want is None:
                want = [a.want(p) for p in proj]
            got = [[], [], []]
            for parts in steps:
                for s, o in a.step(proj, parts).items():
                    got[s].append(o)
            for s in range(3):
                assert rel(torch.cat(got[s]), want[s]) < tol, (name, long_portion, s)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,n", [(37, 140), (64, 300), (100, 260), (1, 70), (129, 200)])
def test_one_key_stands_out_at_every_edge(dtype, window, n):
    """One token takes all the weight of whoever sees it, and its value tells it apart: the output says who saw it."""
    dt, (H, D, R, V, rank) = DTYPES[dtype], (2, 8, 2, 4, 40)
    # latents of equal norm: two channels for the score, the rest for the value
    uk, uv = torch.zeros(H * D, rank), torch.zeros(H * V, rank)
    uk[::D, 0] = 1.0                                             # own key of a head: channel 0 alone
    uv.view(H, V, rank)[:, torch.arange(V), 2 + torch.arange(V)] = 1.0
    for j in sorted({0, 1, 62, 63, 64, n - window - 1, n - window, n - window + 1, n - 2} & set(range(n - 1))):
        for cuts in ([n], [n - 3, 1, 1, 1], [2] * (n // 2) + [1] * (n % 2), [window, n - window]):
            a = Attention((H, D, R, V, rank), window, [n], dt, scale=1.0, uk=uk, uv=uv, long_portion=50)
            proj = torch.zeros(n, a.width)
            proj[:, :H * (D + R):D + R] = 20.0                   # every query asks for channel 0
            proj[:, a.col + 1] = 4.0
            proj[j, a.col:a.col + 2] = torch.tensor([4.0, 0.0])
            proj[:, a.col + 2] = 1.0                             # the value of all ...
            proj[j, a.col + 2:a.col + 4] = torch.tensor([0.0, 1.0])   # ... but the one
            want = a.want(proj)
            got = torch.cat([a.step([proj], [(0, c)])[0] for c in cuts if c > 0])
            err = (got.double() - want).abs().amax(dim=1)
            assert err.max() < 0.03 * want.abs().max(), (j, cuts[:2], int(err.argmax()), err.max().item())


def test_attention_of_many_unequal_sequences():
    """More jobs than one pass of the plan's scan, empty rows between them, and a few long sequences."""
    from tinyllmforge_amd import ops as P
    g, (H, D, R, V, rank), window, bs = torch.Generator().manual_seed(3), (3, 16, 8, 16, 48), 700, 64
    B = 1100
    lens = torch.randint(1, 90, (B,), generator=g)
    lens[torch.randperm(B, generator=g)[:6]] = torch.tensor([2000, 700, 701, 1500, 64, 65])
    s = P.LatentShape(H, D, R, rank, V)
    need = (lens + bs - 1) // bs
    bt = torch.full((B, int(need.max())), -1, dtype=torch.int32)
    perm = torch.randperm(int(need.sum()), generator=g)
    at = 0
    for b in range(B):
        bt[b, :need[b]] = perm[at:at + need[b]].to(torch.int32)
        at += int(need[b])
    cache = torch.randn(at, bs, s.lp, generator=g).to(torch.bfloat16)
    cache[..., rank + R:] = 0
    q = torch.randn(B, H, s.lp, generator=g).to(torch.bfloat16)
    q[..., rank + R:] = 0
    uv = torch.randn(H, 16, s.rp, generator=g).to(torch.bfloat16)
    slots = torch.zeros(B, dtype=torch.int32)
    dead = torch.randperm(B, generator=g)[:40]
    slots[dead] = -1
    batch = P.LatentBatch(B, positions=(lens - 1).cuda(), slot_mapping=slots.cuda())
    plan = P.latent_plan(batch, H, s.lp, window)
    part, ml = P.latent_attention(q.cuda(), cache.cuda(), bt.cuda(), window, 0.1, s, batch, plan)
    out = torch.full((B, H * V), 7.0, dtype=torch.bfloat16, device="cuda")
    P.latent_values(part, ml, uv.cuda(), out, s, batch, plan)
    # every tile of every live sequence is in just one piece
    tiles = [0 if slots[b] < 0 else (int(lens[b]) - 1) // 64 - max(0, int(lens[b]) - window) // 64 + 1 for b in range(B)]
    per, pieces = plan[:2].tolist()
    seen = [[] for _ in range(B)]
    for count, job, tile, start in plan[4:4 + 4 * pieces].view(-1, 4).tolist():
        assert 0 < count <= per and start == int(lens[job]) - 1
        seen[job] += range(tile, tile + count)
    assert seen == [list(range(t)) for t in tiles]
    for b in range(B):
        if slots[b] < 0:
            assert not out[b].any()
            continue
        j = torch.arange(max(0, int(lens[b]) - window), int(lens[b]))
        rows = cache[bt[b, j // bs].long(), j % bs].double()
        p = torch.softmax(0.1 * q[b].double() @ rows.T, dim=-1)
        want = torch.einsum("hr,hvr->hv", p @ rows[:, :rank], uv.double()[..., :rank]).reshape(-1)
        assert rel(out[b], want) < 1.5e-2, b


# ---------------------------------------------------------------------------------------------- experts
@pytest.mark.parametrize("n,E,top,splits", [(1, 5, 2, 1), (64, 70, 6, 3), (500, 16, 1, 2), (1500, 33, 4, 1), (9, 512, 20, 1), (5, 1, 1, 1), (5000, 200, 2, 1)])
def test_grouping_by_expert(n, E, top, splits):
    from tinyllmforge_amd import ops as P
    g = torch.Generator().manual_seed(n)
    z = torch.randn(splits, n, -(-E // 16) * 16, generator=g)
    z[..., E:] = 50.0                                            # pads are never chosen
    if n > 2:
        z[:, 0, :E] = 0.0                                        # ties: the smaller index first
        z[:, 1, :E] = -1e30
        z[:, 2] = float("nan")                                   # still `top` different experts
    for tile in (32, 128):
        r = P.moe_group(z.cuda(), E, top, tile)
        ids, scores = r.ids.cpu().long(), r.scores.cpu()
        total = z.sum(0)[:, :E]
        sound = torch.tensor([i for i in range(n) if n <= 2 or i > 2])
        want = total.double().sort(dim=-1, descending=True, stable=True)
        assert torch.equal(ids[sound], want.indices[sound, :top])
        assert rel(scores[sound], torch.sigmoid(want.values[sound, :top])) < 1e-6
        assert all(len(set(row)) == top and max(row) < E for row in ids.tolist())
        if n > 2:
            assert ids[0].tolist() == list(range(top)) and (scores[0] == 0.5).all()
        row_of = r.row_of.cpu().long().flatten()
        assert torch.equal(row_of.sort().values, torch.arange(n * top))
        assert torch.equal(r.src.cpu().long()[row_of], torch.arange(n * top) // top)
        assert torch.equal(r.weight.cpu()[row_of], scores.flatten()) or n > 2
        by_row = torch.empty(n * top, dtype=torch.long)
        by_row[row_of] = ids.flatten()
        assert (by_row[1:] >= by_row[:-1]).all()
        covered = []
        for e, first, rows, _ in r.tiles.cpu()[:int(r.num_tiles)].tolist():
            assert 0 < rows <= tile and (by_row[first:first + rows] == e).all()
            covered += range(first, first + rows)
        assert covered == list(range(n * top))


def experts(dt, width, E, top, ff, limit, seed=0):
    from tinyllmforge_amd.layers.moe import ClippedGLUExperts
    g = torch.Generator().manual_seed(seed)
    w = {"router": torch.randn(E, width, generator=g) * width ** -0.5}
    for e in range(E):
        for k, shape in (("gate", (ff, width)), ("up", (ff, width)), ("down", (width, ff))):
            w[f"e{e}.{k}"] = torch.randn(shape, generator=g) * shape[1] ** -0.5
    w = {k: v.to(dt) for k, v in w.items()}
    torch.set_default_dtype(dt)
    m = ClippedGLUExperts(width, E, top, ff, limit)
    torch.set_default_dtype(torch.float32)
    for k, v in w.items():
        e, _, kind = k.partition(".")
        m.weight_loader(getattr(m, "router" if k == "router" else "down" if kind == "down" else "gate_up"), v,
                        "router" if k == "router" else (int(e[1:]), kind))
    return m.cuda(), {k: v.double() for k, v in w.items()}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,width,E,top,ff,limit", [(1, 90, 5, 2, 20, 0.7), (7, 64, 1, 1, 1, 1.0), (64, 192, 33, 6, 72, 0.5), (700, 128, 8, 3, 64, 0.6),
                                                    (300, 320, 4, 2, 136, 0.4), (33, 256, 16, 16, 128, 0.8),
                                                    (2100, 64, 4, 1, 40, 0.6), (129, 592, 8, 1, 264, 0.5), (9, 4096, 3, 1, 16, 0.5)])
def test_mixture_of_experts(dtype, n, width, E, top, ff, limit):
    dt = DTYPES[dtype]
    m, w = experts(dt, width, E, top, ff, limit)
    g = torch.Generator().manual_seed(n)
    for kind in ("spread", "all alike"):                         # every token to the same experts: one long group
        h = torch.randn(n, width, generator=g)
        if kind == "all alike":
            h = h[:1] + 0.01 * h
        h = h.to(dt)
        rows, index = m(h.cuda())
        got = rows.double().cpu()[index.cpu().long()].sum(1)[:, :width]
        z = (h.double() @ w["router"].T).sort(dim=-1, descending=True).values
        clear = (z[:, top - 1] - z[:, top] > 1e-3) if top < E else torch.ones(n, dtype=torch.bool)
        want = O.moe_mlp(h.double(), w, dict(expert=dict(limit=limit), router=dict(experts=E, top=top)))
        assert clear.float().mean() > 0.5 and rel(got[clear], want[clear]) < (6e-3 if dtype == "bf16" else 2e-6), kind


def test_consumers_add_up_split_projections():
    """A projection left as partial sums gives the bits of the finished one, in every kernel that may read it."""
    from tinyllmforge_amd import ops as P
    from tinyllmforge_amd.layers.rotary_embedding import rotation_table
    g, n, K = torch.Generator().manual_seed(2), 40, 4096
    bf = lambda *s: torch.randn(*s, generator=g).to(torch.bfloat16).cuda()

    def both(N):
        x, w = bf(n, K), bf(N, K) * K ** -0.5
        d = P.linear_deferred(x, w)
        assert d.splits > 1, "this size is meant to split K"
        return x, w, d
    for H, D, R, V, rank, ff in ((4, 64, 32, 64, 192, 128), (3, 20, 6, 8, 27, 50)):
        s = P.LatentShape(H, D, R, rank, V)
        col = H * (D + R)
        N = -(-(col + rank + R + ff) // 16) * 16
        tab, pos, slots = rotation_table(R, 100, 1e4).cuda(), torch.arange(n).cuda(), torch.arange(n, dtype=torch.int32).cuda()
        nw, pq = bf(rank), bf(2)
        cache = torch.zeros(2, 1, 64, s.lp, dtype=torch.bfloat16, device="cuda")
        out = torch.zeros(2, n, -(-ff // 64) * 64, dtype=torch.bfloat16, device="cuda")
        x, w, d = both(N)
        q2 = P.latent_prep(d, col, nw, pos, tab, slots, cache[1], s, 1e-6)
        P.xielu(d, col + rank + R, ff, pq, out[1])
        y = P.bf16_linear(x, w)
        q1 = P.latent_prep(y, col, nw, pos, tab, slots, cache[0], s, 1e-6)
        P.xielu(y, col + rank + R, ff, pq, out[0])
        assert torch.equal(q1, q2) and torch.equal(cache[0], cache[1]) and torch.equal(out[0], out[1])
    x, w, d = both(1024)
    r, nw, extra = torch.randn(n, 1024, generator=g).cuda(), bf(1024), bf(2 * n, 1024)
    index = torch.randperm(2 * n, generator=g).view(n, 2).to(torch.int32).cuda()
    r2 = r.clone()
    h2 = P.residual_rms_norm(d, r2, 0.4, nw, 1.0, 1e-6, extra, index)
    h1 = P.residual_rms_norm(P.bf16_linear(x, w), r, 0.4, nw, 1.0, 1e-6, extra, index)
    assert torch.equal(h1, h2) and torch.equal(r, r2)


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
        # four live requests, portions beside single tokens, requests that pause; e takes over d's pages
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
    assert len(e.scheduler.block_manager.free_block_ids) == 4
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
    assert runs[0] == runs[1] == runs[2]
    same = [sum(x == y for x, y in zip(a, b)) for a, b in zip(runs[0], runs[3])]
    assert sum(same) > 60                    # other cuts, other rounding: near ties may go the other way


@pytest.mark.parametrize("name", ["even", "wide"])
def test_graph_replays_match_eager_steps(name):
    """Captured decode steps, replayed with eager work in between, against eager ones: the same logits each time."""
    from tinyllmforge_amd.engine.replay import Replay
    cfg = C.CONFIGS[name]
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
    cfg = C.config(64, 80, [C.layer(2, 16, 8, 16, 24, 24, C.dense(64)), C.layer(2, 16, 8, 16, 24, 300, C.moe(4, 2, 32, 1.0))])
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
    cfg = C.config(64, 70, [C.layer(2, 16, 8, 12, 20, 10, C.dense(40)), C.layer(3, 8, 4, 8, 16, 30, C.moe(3, 2, 16, 1.2))])
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
