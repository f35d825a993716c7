"""Tibenex on the GPU: every kernel against the plain implementation, then the mixers and the model under the engine's schedules."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import tibenex as O
from tests import tibenex_cases as C
from tests.test_gpu_gitopel import run_trace

pytestmark = pytest.mark.gpu
DTYPES = {"bf16": torch.bfloat16, "f32": torch.float32}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LOG2E = 1.4426950408889634


def rel(got, want):
    return ((got.double().cpu() - want.double()).norm() / want.double().norm().clamp(min=1e-30)).item()


def i32(*v):
    return torch.tensor(v, dtype=torch.int32).cuda()


# ---------------------------------------------------------------------------------------------- norm behind the sum, token shift
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(5, 90), (3, 64), (70, 1024), (9, 4096), (4, 1), (33, 2050), (2, 8200), (300, 320)])
def test_norm_behind_the_sum(dtype, rows, width):
    from tinyllmforge_amd import ops as P
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(rows)
    tol = 3e-3 if dtype == "bf16" else 2e-6
    r = lambda *s: torch.randn(*s, generator=g)
    y, ls, w, nxt, x = r(rows, width + 8).to(dt), r(width).to(dt), r(width).to(dt), r(width).to(dt), 3 * r(rows, width)
    want = O.post_norm(x.double(), y[:, :width].double(), 1.7, ls.double(), w.double(), 1e-3)
    xd = x.cuda()
    x2, h = P.post_rms_norm(y.cuda(), xd, 1.7, ls.cuda(), w.cuda(), 1e-3)
    assert x2 is xd and rel(x2, want) < 2e-6 and rel(h, want) < tol
    xd = x.cuda()
    x2, h = P.post_rms_norm(y.cuda(), xd, 1.7, ls.cuda(), w.cuda(), 1e-3, None, nxt.cuda())
    assert rel(x2, want) < 2e-6 and rel(h, O.rms_norm(want, nxt.double(), 1e-3)) < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,embed", [(90, False), (1024, False), (64, True), (4096, True), (3000, False), (1, True)])
def test_token_shift_over_steps(dtype, width, embed):
    """Rows of several sequences, whole, in portions and one by one, behind the embedding and behind a sum; a padding row; stale
    states of slots that were used before."""
    from tinyllmforge_amd import ops as P
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(width)
    tol = 3e-3 if dtype == "bf16" else 2e-6
    r = lambda *s: torch.randn(*s, generator=g)
    lens, slots = [37, 9, 20], [3, 0, 2]
    table, mix, ls, w = r(50, width).to(dt), (0.4 + 0.3 * r(width)).to(dt), r(width).to(dt), r(width).to(dt)
    ids = [torch.randint(0, 50, (n,), generator=g) for n in lens]
    x, y = [r(n, width) for n in lens], [r(n, width).to(dt) for n in lens]
    if embed:
        full = [2.5 * table[i].double() for i in ids]
    else:
        full = [O.post_norm(a.double(), b.double(), 1.3, ls.double(), w.double(), 1e-4) for a, b in zip(x, y)]
    want = [O.token_shift(f, mix.double()) for f in full]
    schedules = [[[37, 9, 20]], [[2, 3, 0], [1, 0, 2], [30, 1, 1], [2, 5, 17], [2, 0, 0]], [[1, 1, 1]] * 9 + [[1, 0, 1]] * 11 + [[1, 0, 0]] * 17,
                 [[20, 1, 1]] + [[1, 1, 1]] * 7 + [[10, 1, 12]]]
    for steps in schedules:
        ring = torch.full((5, 2, width), 9.0, device="cuda")
        done, got_x, got_h = [0] * 3, [[], [], []], [[], [], []]
        for step in steps:
            order = sorted((s for s in range(3) if step[s]), key=lambda s: step[s] > 1)
            n = [step[s] for s in order]
            single = sum(k == 1 for k in n)
            take = lambda t: torch.cat([t[s][done[s]:done[s] + step[s]] for s in order])
            pos = torch.cat([torch.arange(done[s], done[s] + step[s]) for s in order])
            st = i32(*[slots[s] for s in order])
            cu = i32(*([0] + torch.tensor(n).cumsum(0).tolist()))
            rows = sum(n)
            pad = int(single == rows)                            # a padding row behind single ones
            pos = torch.cat([pos, torch.zeros(pad, dtype=pos.dtype)]).cuda()
            if pad:
                st = torch.cat([st, i32(-1)])
            seq = torch.repeat_interleave(torch.arange(len(n)), torch.tensor(n)).to(torch.int32).cuda()
            args = P.ShiftArguments(mix.cuda(), ring, st, pos, *(() if pad else (seq, cu)))
            last = lambda t: torch.cat([take(t), take(t)[:1]]) if pad else take(t)
            if embed:
                xs, h = P.embed_shift(last(ids).cuda(), table.cuda(), 2.5, args)
            else:
                xs, h = P.post_rms_norm(last(y).cuda(), last(x).cuda(), 1.3, ls.cuda(), w.cuda(), 1e-4, args)
            if not pad:
                P.conv_tail(xs, ring, st, cu, i32(*[done[s] for s in order]), single, len(n) - single)
            at = 0
            for s, k in zip(order, n):
                got_x[s].append(xs[at:at + k])
                got_h[s].append(h[at:at + k])
                done[s] += k
                at += k
        for s in range(3):
            assert rel(torch.cat(got_x[s]), full[s]) < 2e-6 and rel(torch.cat(got_h[s]), want[s]) < tol, s
            last = lens[s] - 1
            assert rel(ring[slots[s], last % 2], full[s][last]) < 2e-6
        assert (ring[[1, 4]] == 9.0).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,cols,groups,pad", [(5, 60, 4, 64), (3, 64, 1, 1), (40, 4096, 2, 64), (2, 90, 90, 64), (7, 8192, 8, 64), (1, 1, 1, 64), (9, 10000, 1, 1)])
def test_norm_of_row_parts(dtype, rows, cols, groups, pad):
    from tinyllmforge_amd import ops as P
    dt, g = DTYPES[dtype], torch.Generator().manual_seed(cols)
    x, w = (4 * torch.randn(rows, cols, generator=g)).to(dt), torch.randn(cols, generator=g).to(dt)
    x[:, :cols // groups] *= 20                                  # parts of different sizes
    out = P.rows_rms_norm(x.cuda(), w.cuda(), groups, 1e-3, pad)
    assert rel(out[:, :cols], O.grouped_rms_norm(x.double(), w.double(), groups, 1e-3)) < (3e-3 if dtype == "bf16" else 2e-6)
    assert out.shape[1] == -(-cols // pad) * pad and not out[:, cols:].any()


# ---------------------------------------------------------------------------------------------- talking-heads attention
# heads, kv heads, dim, value dim: one of everything, groups of every size, sizes no vector divides, beyond the tiles
TALK = [(1, 1, 2, 1), (6, 3, 20, 13), (8, 4, 64, 64), (16, 4, 64, 128), (16, 8, 128, 128), (32, 8, 128, 128), (32, 1, 32, 64), (12, 12, 96, 80), (5, 5, 17, 100),
        (3, 1, 128, 24), (20, 2, 40, 128), (24, 8, 56, 32), (7, 7, 30, 50), (40, 2, 24, 16), (128, 4, 64, 64), (2, 1, 200, 100), (2, 2, 270, 20), (4, 2, 48, 260),
        (130, 2, 16, 8), (9, 3, 256, 256)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", TALK)
def test_talking_heads_over_paged_rows(dtype, sizes):
    """Portions behind cached keys in shuffled, partly foreign pages: row by row and, where there is a kernel, in tiles."""
    from tinyllmforge_amd import ops as P
    (H, G, D, V), dt, g, bs = sizes, DTYPES[dtype], torch.Generator().manual_seed(sum(sizes)), 64
    starts, lens = [100, 0, 37, 63], [30, 33, 160, 2]
    ends = [a + b for a, b in zip(starts, lens)]
    need = [-(-n // bs) for n in ends]
    perm = torch.randperm(sum(need) + 3, generator=g).to(torch.int32)
    kv = P.SinkKV(sum(need) + 3, bs, G, D, V, dt, "cuda")
    kv.k[..., :D].fill_(30.0)                                    # of whoever had the pages before
    kv.v[..., :V].fill_(30.0)
    bt = torch.full((4, max(need) + 1), -1, dtype=torch.int32)
    keys, values, at = [], [], 0
    for s, n in enumerate(ends):
        bt[s, :need[s]] = perm[at:at + need[s]]
        at += need[s]
        k, v, j = torch.randn(n, G, D, generator=g).to(dt), torch.randn(n, G, V, generator=g).to(dt), torch.arange(n)
        kv.k[bt[s, j // bs].long().cuda(), :, (j % bs).cuda(), :D] = k.cuda()
        kv.v[bt[s, j // bs].long().cuda(), :, (j % bs).cuda(), :V] = v.cuda()
        keys.append(k.double())
        values.append(v.double())
    rows = sum(lens)
    q, talk = torch.zeros(rows, H, kv.k.shape[3]), (torch.randn(H, H, generator=g) * H ** -0.5).to(dt)
    q[..., :D] = torch.randn(rows, H, D, generator=g) * 2.5 * D ** -0.5 * LOG2E
    q = q.to(dt)
    want, lo = [], 0
    for s, n in enumerate(lens):
        wide = torch.zeros(ends[s], H, D, dtype=torch.float64)   # the queries of cached rows do not matter
        wide[starts[s]:] = q[lo:lo + n, :, :D].double() / LOG2E
        want.append(O.talking_attention(wide, keys[s], values[s], 1.0, torch.ones(H, dtype=torch.float64), talk.double())[starts[s]:].reshape(n, H * V))
        lo += n
    want = torch.cat(want)
    pos = torch.cat([torch.arange(a, e) for a, e in zip(starts, ends)])
    seq = torch.repeat_interleave(torch.arange(4), torch.tensor(lens)).to(torch.int32)
    tol = 4e-3 if dtype == "bf16" else 4e-6
    out = torch.full((rows, H * V + 8), 7.0, dtype=dt, device="cuda")
    slots = torch.zeros(rows, dtype=torch.int32)
    slots[lens[0] - 1] = -1                                      # a padding row gives zeros
    P.talk_attention_rows(q.cuda(), kv, bt.cuda(), pos.cuda(), slots.cuda(), talk.cuda(), max(ends), out[:, :H * V], seq.cuda())
    assert not out[lens[0] - 1, :H * V].any() and (out[:, H * V:] == 7).all()
    keep = slots >= 0
    assert rel(out[:, :H * V][keep.cuda()], want[keep]) < tol
    one = [sum(lens[:s + 1]) - 1 for s in range(4)]              # a row of every sequence, without the rows' sequences
    got = torch.empty(4, H * V, dtype=dt, device="cuda")
    P.talk_attention_rows(q[one].cuda(), kv, bt.cuda(), pos[one].cuda(), torch.zeros(4, dtype=torch.int32).cuda(), talk.cuda(), max(ends), got)
    assert rel(got, want[one]) < tol
    small = H <= 32 and max(D, V) <= 128
    assert P.talk_prefill_supported(H, G, D, V) <= small
    if dtype == "bf16" and P.talk_prefill_supported(H, G, D, V):
        cu, out = i32(*([0] + torch.tensor(lens).cumsum(0).tolist())), torch.full((rows, H * V + 8), 7.0, dtype=dt, device="cuda")
        P.talk_attention_prefill(q.cuda(), kv, bt.cuda(), cu, i32(*starts), 1, 3, 160, talk.cuda(), out[:, :H * V])
        assert (out[:lens[0]] == 7).all() and (out[:, H * V:] == 7).all()
        assert rel(out[lens[0]:, :H * V], want[lens[0]:]) < tol


def test_supported_sizes_run_in_tiles():
    from tinyllmforge_amd import ops as P
    for H, G, D, V in ((32, 8, 128, 128), (16, 8, 128, 128), (8, 4, 64, 64), (1, 1, 1, 1), (12, 12, 96, 80), (32, 4, 64, 128)):
        assert P.talk_prefill_supported(H, G, D, V), (H, G, D, V)


@pytest.mark.parametrize("dtype", DTYPES)
def test_talking_heads_of_many_unequal_sequences(dtype):
    """Decoded rows with contexts from one key to thousands, several splits of the keys."""
    from tinyllmforge_amd import ops as P
    dt, g, (H, G, D, V), bs = DTYPES[dtype], torch.Generator().manual_seed(3), (6, 2, 40, 24), 64
    for B, longest in ((200, 500), (4, 4000), (1, 2500)):
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
        q, talk = torch.zeros(B, H, 64), torch.randn(H, H, generator=g).to(dt)
        q[..., :D] = torch.randn(B, H, D, generator=g)
        q = (q * 0.4 * LOG2E).to(dt)
        out = torch.empty(B, H * V, dtype=dt, device="cuda")
        P.talk_attention_rows(q.cuda(), kv, bt.cuda(), (lens - 1).cuda(), torch.zeros(B, dtype=torch.int32).cuda(), talk.cuda(), 10 ** 6, out)
        k, v = kv.k.double().cpu(), kv.v.double().cpu()
        for i in range(B):
            n = int(lens[i])
            ki = k[bt[i, :need[i]].long()].transpose(1, 2).reshape(-1, G, 64)[:n, :, :D]
            vi = v[bt[i, :need[i]].long()].transpose(1, 2).reshape(-1, G, 32)[:n, :, :V]
            s = torch.stack([ki[:, h * G // H] @ q[i, h, :D].double() for h in range(H)]) / LOG2E
            mixed = talk.double() @ torch.softmax(s, -1)
            want = torch.cat([mixed[h] @ vi[:, h * G // H] for h in range(H)])
            assert rel(out[i], want) < (6e-3 if dtype == "bf16" else 4e-6), (B, i, n)


# ---------------------------------------------------------------------------------------------- state-space recurrence
# heads, value dim, state, groups, taps: sizes that no tile divides, one of everything, beyond the matrix cores
SSD = [(6, 10, 13, 3, 3), (1, 1, 1, 1, 1), (4, 64, 64, 1, 4), (8, 64, 128, 2, 4), (2, 128, 256, 2, 5), (12, 24, 40, 12, 2), (3, 200, 96, 1, 4), (2, 300, 280, 1, 2), (5, 16, 300, 5, 3),
       (3, 20, 24, 1, 9)]


def ssd_case(sizes, lens, dt, seed, decay=0.0, step=-1.5):
    H, Pv, N, G, taps = sizes
    g = torch.Generator().manual_seed(seed)
    inner, chan = H * Pv, H * Pv + 2 * G * N
    r = lambda *s: torch.randn(*s, generator=g)
    proj = [r(n, inner + chan + H).to(dt) for n in lens]
    conv = (0.5 * r(chan, taps)).to(dt)
    conv[:, -1] += 0.5
    w = dict(conv=conv, b=(0.3 * r(chan)).to(dt), dt_bias=(step + 1.5 * r(H)).to(dt), A_log=(decay + 0.8 * r(H)).to(dt), D=r(H).to(dt))
    want = []
    for p in proj:
        p = p.double()
        z, xbc, d = p.split([inner, chan, H], dim=1)
        x, B, Cc = O.silu(O.causal_conv(xbc, conv.double(), w["b"].double())).split([inner, G * N, G * N], dim=1)
        T = p.shape[0]
        y = O.state_space_scan(x.reshape(T, H, Pv), B.reshape(T, G, N), Cc.reshape(T, G, N), O.softplus(d + w["dt_bias"].double()), w["A_log"].double(), w["D"].double())
        want.append(y.reshape(T, inner) * O.silu(z))
    return proj, w, want


def run_ssd(sizes, proj, w, steps, dt, slots, stale=5.0):
    """Steps of tokens per sequence; rows of ``proj`` with columns behind them that belong to nobody."""
    from tinyllmforge_amd import ops as P
    H, Pv, N, G, taps = sizes
    inner, chan = H * Pv, H * Pv + 2 * G * N
    weights = P.SsdWeights(w["conv"].T.contiguous().cuda(), w["b"].cuda(), w["dt_bias"].cuda(), w["A_log"].cuda(), w["D"].cuda())
    state = torch.full((max(slots) + 2, H, N, Pv), stale, device="cuda")
    ring = torch.full((max(slots) + 2, taps, chan), stale, dtype=dt, device="cuda")
    done, got = [0] * len(proj), [[] for _ in proj]
    for step in steps:
        order = sorted((s for s in range(len(proj)) if step[s]), key=lambda s: step[s] > 1)
        n = [step[s] for s in order]
        single, rows = sum(k == 1 for k in n), sum(n)
        x = torch.cat([proj[s][done[s]:done[s] + step[s]] for s in order])
        x = torch.nn.functional.pad(x, (0, 16 - x.shape[1] % 16), value=9.0).cuda()
        pos = torch.cat([torch.arange(done[s], done[s] + step[s]) for s in order]).cuda()
        st, start = i32(*[slots[s] for s in order]), i32(*[done[s] for s in order])
        cu = i32(*([0] + torch.tensor(n).cumsum(0).tolist()))
        seq = torch.repeat_interleave(torch.arange(len(n)), torch.tensor(n)).to(torch.int32).cuda()
        out = torch.full((rows, inner), 7.0, dtype=dt, device="cuda")
        if single:
            P.ssd_decode(x[:single], weights, ring, state, st, pos[:single], G, out[:single])
        if single < rows:
            P.ssd_portions(x, weights, ring, state, st, pos, seq, cu, start, single, len(n) - single, single, max(n), G, out)
            P.conv_tail(x[:, inner:], ring, st, cu, start, single, len(n) - single)
        at = 0
        for s, k in zip(order, n):
            got[s].append(out[at:at + k])
            done[s] += k
            at += k
    unused = [i for i in range(max(slots) + 2) if i not in slots]
    assert (state[unused] == stale).all() and (ring[unused] == stale).all()
    return [torch.cat(x) for x in got]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", SSD)
def test_state_space_over_portions_singles_and_mixtures(dtype, sizes):
    dt, lens = DTYPES[dtype], [75, 18]
    schedules = {"whole": [[75, 18]], "portions": [[2, 3], [15, 2], [17, 0], [16, 13], [25, 0]], "single": [[1, 1]] * 18 + [[1, 0]] * 57,
                 "mixed": [[20, 1], [1, 0], [1, 2], [2, 1], [47, 1], [1, 13], [3, 0]]}
    for decay, step in ((0.0, -1.5), (-4.0, -3.0), (3.0, 3.0)):  # states that fade, that stay, that are gone at once
        proj, w, want = ssd_case(sizes, lens, dt, sum(sizes), decay, step)
        for name, steps in schedules.items():
            got = run_ssd(sizes, proj, w, steps, dt, [2, 0])
            for s in (0, 1):
                assert rel(got[s], want[s]) < (6e-3 if dtype == "bf16" else 4e-6), (decay, name, s)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("first", [0, 5, 64])
def test_state_space_in_long_portions(dtype, first):
    """Prompts of many chunks, side by side, from zero and from a state; keys far away still show through a slow decay."""
    sizes, lens, dt = (4, 48, 40, 2, 4), [first + 900, first + 333], DTYPES[dtype]
    proj, w, want = ssd_case(sizes, lens, dt, 7, decay=-5.0, step=-3.0)
    steps = ([[first, first]] if first else []) + [[900, 333]]
    got = run_ssd(sizes, proj, w, steps, dt, [1, 3])
    for s in (0, 1):
        assert rel(got[s], want[s]) < (6e-3 if dtype == "bf16" else 4e-6), s
        assert rel(got[s][-50:], want[s][-50:]) < (8e-3 if dtype == "bf16" else 4e-6), s


@pytest.mark.parametrize("dtype", DTYPES)
def test_one_step_stands_out(dtype):
    """One token writes the state, the others nothing: every later row reads it, whatever lies between."""
    dt, (H, Pv, N, G, taps), n = DTYPES[dtype], (2, 6, 5, 1, 1), 150
    inner = H * Pv
    for j in (0, 1, 31, 32, 63, 64, 65, 127, 128, 140):
        proj = torch.zeros(n, 2 * inner + 2 * G * N + H)
        proj[:, :inner] = 3.0                                    # z
        proj[:, inner:2 * inner] = torch.arange(inner) % 5 + 1.0
        proj[:, 2 * inner:2 * inner + N] = 1.0                   # B
        proj[:, 2 * inner + N:2 * inner + 2 * N] = 1.0           # C
        proj[:, 2 * inner + 2 * N:] = -60.0                      # steps of nothing ...
        proj[j, 2 * inner + 2 * N:] = 2.0                        # ... but one
        proj = proj.to(dt)
        w = dict(conv=torch.ones(inner + 2 * N, 1, dtype=dt), b=torch.zeros(inner + 2 * N, dtype=dt), dt_bias=torch.zeros(H, dtype=dt),
                 A_log=torch.zeros(H, dtype=dt), D=torch.zeros(H, dtype=dt))
        for cuts in ([n], [n - 3, 1, 1, 1], [2] * 75, [j + 1, n - j - 1], [1] * n):
            got = run_ssd((H, Pv, N, G, taps), [proj], w, [[c] for c in cuts], dt, [1])[0].double().cpu()
            assert got[:j].abs().max() < 1e-15 if j else True
            silu = lambda z: z / (1 + torch.exp(-z))
            sb = silu(torch.ones((), dtype=torch.float64))
            y = O.softplus(torch.tensor(2.0, dtype=torch.float64)) * N * sb * sb * silu(proj[0, inner:2 * inner].double()) * silu(torch.tensor(3.0, dtype=torch.float64))
            assert rel(got[j:], y.expand(n - j, -1)) < (8e-3 if dtype == "bf16" else 4e-6), (j, cuts[:3])


# ---------------------------------------------------------------------------------------------- split projections
def test_consumers_add_up_split_projections():
    """A projection left as partial sums gives the bits of the finished one, in every kernel that may read it."""
    from tinyllmforge_amd import ops as P
    from tinyllmforge_amd.layers.rotary_embedding import rotation_table
    g, n, K = torch.Generator().manual_seed(2), 40, 4096
    bf = lambda *s: torch.randn(*s, generator=g).to(torch.bfloat16).cuda()
    pos, slots = torch.arange(n).cuda(), torch.arange(n, dtype=torch.int32).cuda()
    states = torch.randperm(n + 2, generator=g)[:n].to(torch.int32).cuda()
    slots[3], states[3] = -1, -1                                 # a padding row

    def both(N):
        x, w = bf(n, K), bf(-(-N // 16) * 16, K) * K ** -0.5
        d = P.linear_deferred(x, w)
        assert d.splits > 1, "this size is meant to split K"
        return P.bf16_linear(x, w), lambda: P.linear_deferred(x, w)

    def same(N, run):
        rows, deferred = both(N)
        for a, b in zip(run(rows), run(deferred())):
            assert torch.equal(a, b)

    for width in (1024, 200):
        x, ls, nw, nxt, mix, ring = torch.randn(n, width, generator=g).cuda(), bf(width), bf(width), bf(width), bf(width), torch.randn(n + 2, 2, width, generator=g).cuda()
        seq, cu = torch.arange(n, dtype=torch.int32).cuda() // 4, torch.arange(0, n + 1, 4, dtype=torch.int32).cuda()

        def norms(y):
            r = ring.clone()
            one = P.post_rms_norm(y, x.clone(), 1.4, ls, nw, 1e-5, P.ShiftArguments(mix, r, states, pos))
            many = P.post_rms_norm(y, x.clone(), 1.4, ls, nw, 1e-5, P.ShiftArguments(mix, r, states, pos % 4 + 1, seq, cu))
            return (*one, *many, r, *P.post_rms_norm(y, x.clone(), 1.4, ls, nw, 1e-5, None, nxt), *P.post_rms_norm(y, x.clone(), 1.4, ls, nw, 1e-5))
        same(width, norms)
    for H, G, D, V, rot in ((4, 2, 64, 48, 16), (3, 1, 20, 13, 6), (16, 8, 128, 128, 128)):
        qn, kn, temp, tab = bf(H * D), bf(G * D), bf(H), rotation_table(rot, 100, 1e4).cuda()

        def prep(y):
            kv = P.SinkKV(1, 64, G, D, V, torch.bfloat16, "cuda")
            return P.talk_prep(y, kv, H, pos, slots, qn, kn, temp, tab, rot, 1e-5, 0.3), kv.k, kv.v
        same((H + G) * D + G * V, prep)
    for H, Pv, N, G, taps in ((4, 32, 48, 2, 4), (3, 10, 7, 1, 2)):
        chan = H * Pv + 2 * G * N
        w = P.SsdWeights(bf(taps, chan), bf(chan), bf(H), bf(H), bf(H))
        ring, state = bf(n + 2, taps, chan), torch.randn(n + 2, H, N, Pv, generator=g).cuda()

        def step(y):
            r, s, out = ring.clone(), state.clone(), torch.empty(n, H * Pv, dtype=torch.bfloat16, device="cuda")
            return P.ssd_decode(y, w, r, s, states, pos, G, out), r, s
        same(H * Pv + chan + H, step)
    for H, D, R, V, rank, q_rank in ((4, 64, 32, 64, 192, 256), (3, 20, 6, 8, 27, 50)):
        s, tab, nw, qw = P.LatentShape(H, D, R, rank, V), rotation_table(R, 100, 1e4).cuda(), bf(rank), bf(q_rank)

        def down(y):
            cache = torch.zeros(1, 64, s.lp, dtype=torch.bfloat16, device="cuda")
            return (*P.latent_prep_down(y, q_rank, nw, pos, tab, slots, cache, s, 1e-5, True, 0, qw, q_rank + rank + R), cache)
        same(q_rank + rank + R + H, down)
        same(H * (D + R), lambda y: [P.latent_prep_queries(y, pos, tab, s, True)])


# ---------------------------------------------------------------------------------------------- the mixers
class Plain(torch.nn.Module):
    """In the place of an output projection: the rows themselves."""

    def __init__(self, size):
        super().__init__()
        self.input_size = size

    def forward_deferred(self, x):
        return x


class Mixer:
    """A mixer with a few sequences in shuffled pages and slots, run step by step as the engine does; its output is not projected."""

    def __init__(self, layer, lens, dt, width=72, w=None, seed=0, bs=64, slots=(3, 0, 5)):
        from tinyllmforge_amd.config import model_config
        from tinyllmforge_amd.engine.sequence import Sequence
        from tinyllmforge_amd.models.tibenex import TibenexForCausalLM
        from tinyllmforge_amd.utils.loader import load_state_dict
        Sequence.block_size = bs
        cfg = C.config(width, 32, [layer], eps=1e-4)
        self.m, self.kind, self.lens, self.dt, self.bs = layer["mixer"], layer["type"], lens, dt, bs
        all_w = C.weights(cfg, seed) | {"l0.mix." + k: v.to(torch.bfloat16) for k, v in (w or {}).items()}
        self.w = {k[7:]: v.double() for k, v in all_w.items() if k.startswith("l0.mix.")}
        self.out = self.m["heads"] * self.m["vdim"]
        self.w["o"] = torch.eye(self.out, dtype=torch.float64)
        self.hf = hf = model_config(cfg)
        hf.max_position_embeddings, hf.torch_dtype = max(lens) + 1, dt
        torch.set_default_dtype(dt)
        model = TibenexForCausalLM(hf)
        torch.set_default_dtype(torch.float32)
        load_state_dict(model, all_w)
        model = model.cuda().pack_linears_()
        self.mix = model.layers[0].mix
        self.mix.o = Plain(self.out)
        g = torch.Generator().manual_seed(seed)
        need = [-(-n // bs) for n in lens]
        perm = torch.randperm(sum(need) + 2, generator=g).tolist()
        for mod in self.mix.modules():                           # stale contents of pages and slots that are used again
            if hasattr(mod, "bind_pages"):
                mod.bind_pages(sum(need) + 2, bs, "cuda")
                for t in (mod.kv.k, mod.kv.v) if hasattr(mod, "kv") else (mod.cache,):
                    t.fill_(3.0)
                if hasattr(mod, "kv"):                           # pads stay zero
                    mod.kv.k[..., mod.dim:] = 0
                    mod.kv.v[..., mod.value_dim:] = 0
            if hasattr(mod, "bind_slots"):
                mod.bind_slots(6, "cuda")
                mod.state.fill_(5.0)
                mod.ring.fill_(5.0)
        self.seqs = []
        for i, (n, k) in enumerate(zip(lens, need)):
            s = Sequence([0] * n)
            s.block_table, s.state_slot = [perm.pop() for _ in range(k)], slots[i % len(slots)]
            self.seqs.append(s)

    def step(self, h, parts):
        """``parts``: (sequence, tokens).  Returns ``{sequence: [tokens, H * V]}``."""
        from tinyllmforge_amd.engine import inputs as I
        from tinyllmforge_amd.utils.context import reset_context, set_portions_context
        parts = sorted(parts, key=lambda x: I.portion_kind(x[1], self.hf.long_portion))
        seqs = [self.seqs[s] for s, _ in parts]
        for s, (_, n) in zip(seqs, parts):
            s.num_scheduled = n
        d = I.portion_inputs(seqs, self.bs, self.hf.long_portion, self.hf.windows)
        d = {k: torch.from_numpy(v).cuda() if hasattr(v, "dtype") else v for k, v in d.items()}
        d.pop("input_ids")
        pos = d.pop("positions")
        rows = torch.cat([h[i][s.num_computed:s.num_computed + n] for s, (i, n) in zip(seqs, parts)]).to(self.dt)
        set_portions_context(max_len=max(self.lens), plans={}, **d)
        out = self.mix(rows.cuda(), pos)[:, :self.out].cpu()
        reset_context()
        got, at = {}, 0
        for s, (i, n) in zip(seqs, parts):
            got[i] = out[at:at + n]
            at += n
            s.num_computed += n
        return got

    def want(self, h):
        return O.MIXERS[self.kind](h.to(self.dt).double(), self.w, self.m, 1e-4)


MIXERS = [C.attention(6, 3, 20, 13, 12), C.attention(8, 2, 64, 64, 64), C.attention(1, 1, 2, 1, 2), C.attention(16, 16, 32, 128, 6), C.attention(12, 1, 128, 48, 30),
          C.attention(40, 2, 24, 16, 8), C.attention(2, 1, 270, 140, 270), C.latent(3, 11, 6, 9, 17, 21), C.latent(4, 64, 32, 64, 128, 64), C.latent(1, 1, 2, 1, 1, 1),
          C.latent(16, 128, 64, 128, 96, 256), C.latent(5, 20, 4, 23, 40, 9, scaling=None), C.latent(2, 260, 64, 150, 70, 300), C.mamba2(6, 10, 13, 3, 3, 4),
          C.mamba2(8, 64, 64, 2, 4, 2), C.mamba2(1, 1, 1, 1, 1, 1), C.mamba2(4, 30, 96, 4, 5, 8), C.mamba2(2, 300, 280, 1, 2, 1)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layer", MIXERS, ids=lambda la: f"{la['type']}-{la['mixer']['heads']}-{la['mixer'].get('dim', la['mixer'].get('state'))}-{la['mixer']['vdim']}")
def test_mixer_over_portions_singles_and_mixtures(dtype, layer):
    dt, lens = DTYPES[dtype], [150, 67, 210]
    schedules = {
        "whole": [[(0, 150), (1, 67), (2, 210)]],
        "portions": [[(0, 2), (1, 3)], [(0, 62), (2, 130)], [(0, 1), (1, 2), (2, 2)], [(0, 85), (1, 62), (2, 78)]],
        "mixed": [[(0, 100), (2, 64)], [(0, 1), (1, 20), (2, 1)]] + [[(0, 1), (1, 1), (2, 29)], [(0, 1), (2, 2)]] * 3 + [[(0, 43), (1, 1)], [(1, 43), (2, 52)]],
        "single": [[(0, 1), (1, 1), (2, 1)] for _ in range(67)] + [[(0, 1), (2, 1)] for _ in range(83)] + [[(2, 1)] for _ in range(60)],
    }
    g = torch.Generator().manual_seed(5)
    h, want = [torch.randn(n, 72, generator=g) for n in lens], None
    for name, steps in schedules.items():
        a = Mixer(layer, lens, dt)
        want = want or [a.want(x) for x in h]
        got = [[], [], []]
        for parts in steps:
            for s, o in a.step(h, parts).items():
                got[s].append(o)
        for s in range(3):
            assert rel(torch.cat(got[s]), want[s]) < (2e-2 if dtype == "bf16" else 1e-5), (name, s)


def far_key(kind, n, j):
    """``(layer, weights, inputs)``: one token's key takes all the weight of whoever sees it, and its value tells it apart.  Inputs:
    channel 0 is 1, channel 1 marks the ordinary tokens, channel 2 the one; values read channels 1 and 2."""
    width = 72
    h = torch.zeros(n, width)
    h[:, 0] = h[:, 1] = 1.0
    h[j, 1], h[j, 2] = 0.0, 1.0
    z = torch.zeros
    if kind == "attention":                                      # two query heads that see the same and swap their weights
        q, k, v = z(16, width), z(8, width), z(2, width)
        q[4, 0] = q[12, 0] = 1.0
        k[5, 1] = k[4, 2] = 1.0
        v[0, 1] = v[1, 2] = 1.0
        w = dict(q=q, k=k, v=v, temp=torch.ones(2), talk=torch.tensor([[0.0, 1.0], [2.0, 0.0]])) | {"q.norm": torch.ones(16), "k.norm": torch.ones(8)}
        return C.attention(2, 1, 8, 2, 2, scale=3.0), w, h
    dq, uq, dkv, uk, uv, gate = z(3, width), z(2 * 6, 3), z(6, width), z(2 * 4, 4), z(2 * 2, 4), z(2, width)
    dq[0, 0] = dkv[1, 1] = dkv[2, 2] = 1.0
    uq[1, 0] = uq[7, 0] = 1.0                                    # both heads' second dimension
    uk[1, 2] = uk[5, 2] = 1.0
    uv[0, 1] = uv[1, 2] = uv[2, 1] = uv[3, 2] = 1.0
    gate[0, 0], gate[1, 0] = 2.0, -1.0
    w = dict(dq=dq, uq=uq, dkv=dkv, uk=uk, uv=uv, g=gate) | {"dq.norm": torch.ones(3), "dkv.norm": torch.ones(4)}
    return C.latent(2, 4, 2, 2, 3, 4, scale=6.0), w, h


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["attention", "latent"])
@pytest.mark.parametrize("n", [140, 300])
def test_one_key_stands_out(dtype, kind, n):
    for j in sorted({0, 1, 31, 32, 62, 63, 64, 127, 128, 129, n - 3, n - 2} & set(range(n - 1))):
        layer, w, h = far_key(kind, n, j)
        for cuts in ([n], [n - 3, 1, 1, 1], [2] * (n // 2) + [1] * (n % 2), [j + 1, n - j - 1], [j, n - j]):
            a = Mixer(layer, [n], DTYPES[dtype], w=w)
            want = a.want(h)
            assert (want[j:] - want[:1]).abs().amax(1).min() > 0.1 * want.abs().max() or j == 0
            got = torch.cat([a.step([h], [(0, c)])[0] for c in cuts if c > 0])
            err = (got.double() - want).abs().amax(dim=1)
            assert err.max() < 0.02 * want.abs().max(), (j, cuts[:2], int(err.argmax()), err.max().item())


# ---------------------------------------------------------------------------------------------- the model
def engine(cfg, dtype, seed=0, blocks=12, seqs=4, max_len=256, **kw):
    from tinyllmforge_amd.engine.llm_engine import LLMEngine
    return LLMEngine(cfg, state_dict=C.weights(cfg, seed), dtype={"bf16": "bfloat16", "f32": "float32"}[dtype],
                     kvcache_block_size=64, num_kvcache_blocks=blocks, max_num_seqs=seqs, num_state_slots=seqs, max_model_len=max_len,
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
            assert len(e.scheduler.block_manager.free_block_ids) == 12 and len(e.scheduler.state_slots.free) == 4
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
    cfg = C.config(90, 203, [C.attention(6, 3, 20, 13, 12, mlp=50), C.mamba2(6, 10, 13, 3, 3, 2), C.latent(3, 11, 6, 9, 17, 21, mlp=33)], eps=1e-3)
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
    cfg = C.CONFIGS["even"]
    prompt = C.tokens(cfg, 70, 4)
    e = engine(cfg, "bf16", quantization="w8a16")
    got = run_trace(Replay(e), {"a": prompt}, [[("a", 60)]] + [[("a", 1)]] * 10)["a"]
    e.exit()
    assert C.logit_error(got, O.forward(cfg, C.weights(cfg), prompt)).median() < 0.15


def test_long_decoding():
    from tinyllmforge_amd.engine.replay import Replay
    cfg = C.config(64, 80, [C.attention(4, 2, 16, 24, 8, mlp=64), C.mamba2(4, 16, 24, 2, 4, 2), C.latent(2, 16, 8, 12, 24, 32, mlp=40)])
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
    cfg = C.config(64, 70, [C.latent(2, 16, 8, 12, 24, 20, mlp=40), C.mamba2(3, 8, 16, 1, 3, 1), C.attention(3, 3, 8, 16, 4)])
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
