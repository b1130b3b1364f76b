"""GPU: every mechanism of the Galirax layers alone, each kernel form (fast, plain, fp32) against the plain float64 reference on the same rounded inputs.
Where many keys would hide a fault, one key of a sequence is scaled to take the whole softmax, at every border it could be lost or seen by mistake."""
import math

import pytest
import torch

from oracle import galirax_ref as G
from paged_cases import BF16, F32, Pages, close, f64, randn, standout_places

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------------------------------------ attention
def attend_ref(q, k, v, pos, scale, window, keep, sink):
    """q [heads, dim] at position pos over k, v [n, kvh, .]"""
    heads, kvh = q.shape[0], k.shape[1]
    j = torch.arange(k.shape[0])
    ok = (j <= pos) & ((pos - j < window) | (j < keep) if window else j >= 0)
    out = []
    for h in range(heads):
        g = h // (heads // kvh)
        s = ((f64(k)[:, g] @ f64(q)[h]) * scale).masked_fill(~ok, float("-inf"))
        p = G.sink_softmax(s[None], f64(sink)[h])[0] if sink is not None else torch.softmax(s, 0)
        out.append(p @ f64(v)[:, g])
    return torch.stack(out)


SHAPES = [(8, 2, 64, 64), (3, 3, 40, 100), (20, 2, 128, 128), (6, 2, 96, 64), (4, 1, 192, 128), (2, 2, 256, 256), (9, 1, 128, 60), (2, 1, 200, 30), (5, 5, 250, 120),
          (2, 1, 270, 300)]
MASKS = [(0, 0), (1, 0), (64, 3), (100, 70), (65, 64), (7, 130)]


@pytest.mark.parametrize("dtype,generic", [(BF16, False), (BF16, True), (F32, False)])
@pytest.mark.parametrize("heads,kvh,dim,vdim", SHAPES)
def test_rows(heads, kvh, dim, vdim, dtype, generic):
    from nanovllm_hip import ops
    lengths = [1, 2, 64, 65, 129, 300]
    pg = Pages(lengths, kvh, dim, vdim, dtype)
    cache, tables = pg.cache(), pg.tables.cuda()
    q = randn(len(lengths), heads, dim, seed=5, dtype=dtype)
    sink = randn(heads, seed=6, dtype=F32)
    pos = torch.tensor([n - 1 for n in lengths])
    for window, keep in MASKS:
        for use_sink in (True, False):
            want = torch.stack([attend_ref(q[i], pg.k[i], pg.v[i], n - 1, 0.2, window, keep, sink if use_sink else None) for i, n in enumerate(lengths)])
            for splits in (None, 1, 3, 5):
                got = ops.paged_attend_rows(pg.pad_q(q), cache, tables, pos.cuda(), heads, kvh, pg.dk, pg.dv, 0.2, 300, window, keep, sink.cuda() if use_sink else None,
                                            splits=splits, generic=generic)
                close(pg.unpad(got, heads), want, dtype, f"window {window} keep {keep} splits {splits}")


def test_rows_packed_output_and_row_seq():
    from nanovllm_hip import ops
    heads, kvh, dim, vdim = 4, 2, 64, 128
    pg = Pages([70, 200, 5], kvh, dim, vdim, BF16)
    cache, tables = pg.cache(), pg.tables.cuda()
    q = randn(3, heads, dim, seed=5)
    pos = torch.tensor([69, 199, 4]).cuda()
    args = (heads, kvh, pg.dk, pg.dv, 0.3, 200, 50, 2)
    rows = ops.paged_attend_rows(pg.pad_q(q), cache, tables, pos, *args)
    packed = torch.zeros(16 * heads * vdim, dtype=BF16, device="cuda")
    assert ops.paged_attend_rows(pg.pad_q(q), cache, tables, pos, *args, out_packed=packed, want_out=False, splits=2) is None
    close(ops.unpack_rows(packed, 3, heads * vdim), f64(rows), BF16)
    seq = torch.tensor([2, 0, 1], dtype=torch.int32).cuda()              # rows of other sequences, in another order
    got = ops.paged_attend_rows(pg.pad_q(q[[2, 0, 1]]), cache, tables, pos[[2, 0, 1]], *args, row_seq=seq)
    close(got, f64(rows)[[2, 0, 1]], BF16)


@pytest.mark.parametrize("dtype,generic", [(BF16, False), (F32, False)])
@pytest.mark.parametrize("window,keep", [(0, 0), (64, 0), (65, 1), (130, 4), (40, 70)])
def test_rows_one_key_stands_out(window, keep, dtype, generic):
    """A key whose score dwarfs the others' takes the output where it is seen, and changes nothing where it is not."""
    from nanovllm_hip import ops
    heads, kvh, dim, vdim = 4, 2, 64, 64
    for pos in (199, 192, 255):
        places = standout_places(pos, window, keep)
        pg = Pages([pos + 1] * len(places), kvh, dim, vdim, dtype)
        q = randn(len(places), kvh, dim, seed=7, dtype=dtype).repeat_interleave(heads // kvh, dim=1)
        for i, a in enumerate(places):
            pg.k[i] = pg.k[i] * 0.3
            pg.k[i][a] = q[i, ::heads // kvh] * 2
        want = torch.stack([attend_ref(q[i], pg.k[i], pg.v[i], pos, 0.2, window, keep, None) for i in range(len(places))])
        for i, a in enumerate(places):
            seen = not window or pos - a < window or a < keep
            assert ((want[i, 0] - f64(pg.v[i])[a, 0]).abs().max() < 0.05) == seen
        for splits in (1, 4):
            got = ops.paged_attend_rows(pg.pad_q(q), pg.cache(), pg.tables.cuda(), torch.full((len(places),), pos).cuda(), heads, kvh, pg.dk, pg.dv, 0.2, 256, window, keep,
                                        splits=splits)
            close(pg.unpad(got, heads), want, dtype, f"pos {pos}", slack=2)


PORTIONS = [(2, 2), (64, 64), (2, 65), (65, 129), (130, 300), (300, 300), (3, 400), (57, 190)]


@pytest.mark.parametrize("window,keep", MASKS + [(200, 1)])
@pytest.mark.parametrize("heads,kvh,dim,vdim", [s for s in SHAPES if max(s[2:]) <= 256])
def test_prompt(heads, kvh, dim, vdim, window, keep):
    """Portions of several sequences (rows, keys) in one launch; long portions take the two-tile form."""
    from nanovllm_hip import ops
    sink = randn(heads, seed=6, dtype=F32)
    for portions in (PORTIONS[:5], PORTIONS[3:]) if dim <= 128 else (PORTIONS[2:6],):
        pg = Pages([k for _, k in portions], kvh, dim, vdim, BF16, seed=3)
        rows = sum(r for r, _ in portions)
        q = randn(rows, heads, dim, seed=8)
        cu_q = torch.tensor([0] + [r for r, _ in portions]).cumsum(0).int().cuda()
        cu_k = torch.tensor([0] + [k for _, k in portions]).cumsum(0).int().cuda()
        got = pg.unpad(ops.paged_attend_prompt(pg.pad_q(q), pg.cache(), pg.tables.cuda(), cu_q, cu_k, max(r for r, _ in portions), heads, kvh, pg.dk, pg.dv, 0.2, window,
                                               keep, sink.cuda()), heads)
        at = 0
        for i, (r, k) in enumerate(portions):
            for t in sorted({0, 1, r // 2, r - 2, r - 1, min(63, r - 1), min(64, r - 1)}):
                want = attend_ref(q[at + t], pg.k[i], pg.v[i], k - r + t, 0.2, window, keep, sink)
                close(got[at + t], want, BF16, f"portion {i} row {t}")
            at += r


@pytest.mark.parametrize("window,keep", [(0, 0), (64, 0), (65, 1), (130, 4), (40, 70)])
@pytest.mark.parametrize("portion", [2, 40, 200])
def test_prompt_one_key_stands_out(window, keep, portion):
    from nanovllm_hip import ops
    heads, kvh, dim, vdim, n = 2, 1, 64, 64, 200
    places = sorted({a for pos in (n - 1, n - 2, n - portion) for a in standout_places(pos, window, keep)})
    pg = Pages([n] * len(places), kvh, dim, vdim, BF16)
    q1 = randn(len(places), kvh, dim, seed=7)
    for i, a in enumerate(places):
        pg.k[i] = pg.k[i] * 0.3
        pg.k[i][a] = q1[i] * 2
    q = q1.repeat_interleave(portion, dim=0).repeat_interleave(heads, dim=1)              # every row of a portion asks for the same key
    cu_q = (torch.arange(len(places) + 1) * portion).int().cuda()
    cu_k = (torch.arange(len(places) + 1) * n).int().cuda()
    got = pg.unpad(ops.paged_attend_prompt(pg.pad_q(q), pg.cache(), pg.tables.cuda(), cu_q, cu_k, portion, heads, kvh, pg.dk, pg.dv, 0.2, window, keep), heads)
    for i, a in enumerate(places):
        for t in sorted({0, 1, portion // 2, portion - 2, portion - 1} | {x - (n - portion) for x in (a, a - 1, a + window - 1, a + window) if 0 <= x - (n - portion) < portion}):
            want = attend_ref(q[i * portion + t], pg.k[i], pg.v[i], n - portion + t, 0.2, window, keep, None)
            close(got[i * portion + t], want, BF16, f"key {a} row {t}", slack=2)


def test_sink_takes_its_share():
    """A large sink leaves almost nothing, a hugely negative one changes nothing; both forms."""
    from nanovllm_hip import ops
    pg = Pages([150], 1, 64, 64, BF16)
    cache, tables = pg.cache(), pg.tables.cuda()
    q = randn(150, 2, 64, seed=1)
    sink = torch.tensor([30.0, -1e4])
    cu = torch.tensor([0, 150], dtype=torch.int32).cuda()
    prompt = pg.unpad(ops.paged_attend_prompt(pg.pad_q(q), cache, tables, cu, cu, 150, 2, 1, 64, 64, 0.1, sink=sink.cuda()), 2)
    rows = pg.unpad(ops.paged_attend_rows(pg.pad_q(q[-1:]), cache, tables, torch.tensor([149]).cuda(), 2, 1, 64, 64, 0.1, 150, sink=sink.cuda()), 2)
    bare = attend_ref(q[-1], pg.k[0], pg.v[0], 149, 0.1, 0, 0, None)
    for o in (prompt[-1], rows[0]):
        assert o[0].abs().max() < 1e-6 and (o[1] - bare[1]).abs().max() < 0.02


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("norm", [False, True])
@pytest.mark.parametrize("heads,kvh,dim,vdim,rot", [(4, 2, 64, 64, 64), (3, 1, 20, 36, 12), (6, 6, 72, 130, 2), (40, 8, 128, 128, 96), (2, 2, 24, 16, 0)])
def test_prep(heads, kvh, dim, vdim, rot, norm, dtype):
    from nanovllm_hip import ops
    from nanovllm_hip.layers.paged_attention import padded_widths
    from nanovllm_hip.layers.rotary import rotation_table
    dk, dv = padded_widths(dim, vdim)
    rows, bs, pages = 9, 64, 3
    parts = [randn(rows, h, w, seed=i, dtype=dtype) for i, (h, w) in enumerate(((heads, dim), (kvh, dim), (kvh, vdim)))]

    def pad(t, width):
        out = torch.zeros(*t.shape[:-1], width, dtype=t.dtype)
        out[..., :t.shape[-1]] = t
        return out
    qkv = torch.cat([pad(t, w).reshape(rows, -1) for t, w in zip(parts, (dk, dk, dv))], dim=1).cuda()
    qw, kw = 1 + randn(heads, dim, seed=7, scale=0.3, dtype=F32), 1 + randn(kvh, dim, seed=8, scale=0.3, dtype=F32)
    pos = torch.tensor([0, 1, 2, 63, 64, 65, 500, 4000, 8191])
    slots = torch.tensor([5, 63, 64, 65, 130, -1, 191, 0, 100], dtype=torch.int32)
    table = rotation_table(rot, 5000.0, 8192, "cuda", dict(factor=8.0, low=1.0, high=4.0, original=256)) if rot else torch.zeros(8192, 0, device="cuda")
    cache = torch.full((pages, bs, kvh * (dk + dv)), 7.0, dtype=dtype, device="cuda")
    kw_args = dict(q_weight=pad(qw, dk).reshape(-1).cuda(), k_weight=pad(kw, dk).reshape(-1).cuda(), q_n=heads * dim, k_n=kvh * dim, eps=1e-3) if norm else {}
    ops.attn_prep(qkv, heads, kvh, dk, dv, pos.cuda(), table, cache, slots.cuda(), **kw_args)
    q, k, v = (f64(t) for t in parts)
    if norm:
        q = G.rms_norm(q.reshape(rows, -1), f64(qw).reshape(-1), 1e-3).view(rows, heads, dim)
        k = G.rms_norm(k.reshape(rows, -1), f64(kw).reshape(-1), 1e-3).view(rows, kvh, dim)
    freqs = G.frequencies(dict(dims=rot, base=5000.0, scaling=dict(factor=8.0, low=1.0, high=4.0, original=256)))
    q, k = G.rotate_pairs(q, pos, freqs), G.rotate_pairs(k, pos, freqs)
    close(qkv[:, :heads * dk].reshape(rows, heads, dk)[..., :dim], q, dtype, "queries", slack=20 if dtype == F32 else 1)
    flat = cache.view(pages, kvh, bs * (dk + dv))
    keys, vals = flat[:, :, :bs * dk].view(pages, kvh, bs, dk), flat[:, :, bs * dk:].view(pages, kvh, bs, dv)
    for i, s in enumerate(slots.tolist()):
        if s >= 0:
            close(keys[s // bs, :, s % bs, :dim], k[i], dtype, f"key {i}", slack=20 if dtype == F32 else 1)
            assert torch.equal(f64(vals[s // bs, :, s % bs, :vdim]), v[i])
    assert (keys == 7.0).all(-1).sum() == kvh * (pages * bs - 8)         # nothing else was written


def test_frequency_scaling_has_three_ranges():
    from nanovllm_hip.layers.rotary import frequencies
    scaling = dict(factor=8.0, low=1.0, high=4.0, original=512)
    got = frequencies(64, 10000.0, scaling)
    want = torch.tensor(G.frequencies(dict(dims=64, base=10000.0, scaling=scaling)), dtype=torch.float64)
    assert torch.allclose(got, want, rtol=1e-12)
    ratio = got / frequencies(64, 10000.0)
    assert (ratio == 1).any() and torch.isclose(ratio, torch.tensor(1 / 8, dtype=torch.float64)).any() and ((ratio > 0.13) & (ratio < 0.99)).any()


# ------------------------------------------------------------------------------------------------ lightning attention
def lightning_ref(x, heads, dim, vdim, decay, dtype, state=None):
    """x [T, q | k | v]; silu rounded to the activation type.  Returns (o [T, heads * vdim], states)"""
    act = G.silu(f64(x)).to(dtype).double()
    a, outs, states = heads * dim, [], []
    for h in range(heads):
        q, k, v = act[:, h * dim:(h + 1) * dim], act[:, a + h * dim:a + (h + 1) * dim], act[:, 2 * a + h * vdim:2 * a + (h + 1) * vdim]
        o, s = G.lightning_recurrence(q, k, v, float(torch.tensor(decay[h], dtype=F32)), None if state is None else f64(state[h]))
        outs.append(o)
        states.append(s)
    return torch.cat(outs, dim=1), torch.stack(states)


DECAYS = [0.6, 0.97, 0.999, 1.0, 0.0, 0.9]


@pytest.mark.parametrize("dtype,generic", [(BF16, False), (BF16, True), (F32, False)])
@pytest.mark.parametrize("heads,dk,dv,segment", [(2, 64, 64, 64), (3, 64, 128, 128), (6, 128, 128, 64), (2, 128, 64, 192), (1, 256, 128, 64)])
def test_lightning_portions(heads, dk, dv, segment, dtype, generic):
    """Portions of several sequences in one launch, whole and in pieces; a first portion ignores what its slot holds; more than one segment per portion."""
    from nanovllm_hip import ops
    from nanovllm_hip.engine.model_runner import recurrence_chunks
    decay = DECAYS[:heads]
    d = torch.tensor(decay, dtype=F32).cuda()
    slots = torch.tensor([3, 0, 2], dtype=torch.int32)
    pieces = [[200, 1, 2, 63], [64, 65, 70, 3], [2, 130, 1, 129]]
    xs = [randn(sum(p), heads * (2 * dk + dv), seed=i, dtype=dtype) for i, p in enumerate(pieces)]
    refs = [lightning_ref(x, heads, dk, dv, decay, dtype) for x in xs]
    state = torch.full((4, heads, dk, dv), 1e4, device="cuda")
    at = [0, 0, 0]
    for step in range(4):
        rows, pos, chunks = [], [], []
        for i, p in enumerate(pieces):
            chunks += recurrence_chunks(sum(r.shape[0] for r in rows), p[step], i, segment)
            rows.append(xs[i][at[i]:at[i] + p[step]])
            pos += range(at[i], at[i] + p[step])
        got = ops.lightning_chunks(torch.cat(rows).cuda(), d, torch.tensor(pos).cuda(), slots.cuda(), torch.tensor(chunks, dtype=torch.int32).cuda(),
                                   any(c[3] for c in chunks), state, generic=generic)
        for i, g in enumerate(got.split([p[step] for p in pieces])):
            close(g, refs[i][0][at[i]:at[i] + pieces[i][step]], dtype, f"sequence {i} step {step}", slack=4)
            at[i] += pieces[i][step]
    for i in range(3):
        close(state[slots[i]], refs[i][1], F32 if dtype == F32 or generic else BF16, f"state {i}", slack=4 if dtype == F32 or generic else 0.05)
    assert (state[1] == 1e4).all()


@pytest.mark.parametrize("heads,dk,dv,rows", [(3, 64, 64, 4), (2, 128, 128, 5), (4, 256, 64, 2), (16, 64, 64, 40)])
def test_lightning_step(heads, dk, dv, rows):
    """Token by token: the step form against the recurrence, from garbage-filled slots on; long enough that a slow head remembers and a fast one forgets."""
    from nanovllm_hip import ops
    decay = [DECAYS[h % len(DECAYS)] for h in range(heads)]
    d = torch.tensor(decay, dtype=F32).cuda()
    steps = 70 if heads < 16 else 3
    x = randn(steps, rows, heads * (2 * dk + dv), seed=1)
    slots = torch.randperm(rows + 2, generator=torch.Generator().manual_seed(2))[:rows].int().cuda()
    state = torch.full((rows + 2, heads, dk, dv), float("nan"), device="cuda")
    outs = [ops.lightning_step(x[t].cuda(), d, torch.full((rows,), t).cuda(), slots, state) for t in range(steps)]
    for r in range(min(rows, 5)):
        o, s = lightning_ref(x[:, r], heads, dk, dv, decay, BF16)
        close(torch.stack([out[r] for out in outs]), o, BF16, f"row {r}", slack=2)
        close(state[slots[r]], s, F32, f"state {r}", slack=4)
    assert torch.isnan(state).all(-1).all(-1).all(-1).sum() == 2


def test_lightning_remembers_and_forgets_the_same_in_every_form():
    """One token a thousand back, everything behind it zero: portions with and without segments and decoding carry it alike (constant decay 0.999)."""
    from nanovllm_hip import ops
    from nanovllm_hip.engine.model_runner import recurrence_chunks
    heads, dk, dv, n = 1, 64, 64, 1000
    x = torch.zeros(n, 2 * dk + dv, dtype=BF16)
    x[0], x[-1, :dk] = randn(2 * dk + dv, seed=1) * 2, 3.0
    want = lightning_ref(x, heads, dk, dv, [0.999], BF16)[0][-1]
    d, slot = torch.tensor([0.999]).cuda(), torch.zeros(1, dtype=torch.int32).cuda()
    assert want.abs().max() > 1
    for segment in (64, 256, 1024):
        state = torch.zeros(1, heads, dk, dv, device="cuda")
        chunks = torch.tensor(recurrence_chunks(0, n - 1, 0, segment), dtype=torch.int32).cuda()
        ops.lightning_chunks(x[:-1].cuda(), d, torch.arange(n - 1).cuda(), slot, chunks, len(chunks) > 1, state)
        got = ops.lightning_step(x[-1:].cuda(), d, torch.tensor([n - 1]).cuda(), slot, state)
        assert (f64(got)[0] - want).abs().max() < 0.01 * want.abs().max()


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("rows,cols,n", [(5, 64, 50), (3, 2048, 2048), (2, 5184, 5180)])
def test_norm_gate(rows, cols, n, dtype):
    from nanovllm_hip import ops
    a = randn(rows, 2 * cols, seed=1, dtype=dtype)
    x, gate = a[:, :cols].clone(), a[:, cols:].clone()
    x[:, n:] = 0
    w = torch.zeros(cols)
    w[:n] = 1 + randn(n, seed=2, scale=0.3, dtype=F32)
    want = torch.zeros(rows, cols, dtype=torch.float64)
    want[:, :n] = G.rms_norm(f64(x)[:, :n], f64(w)[:n], 1e-3) * torch.sigmoid(f64(gate)[:, :n])
    close(ops.norm_gate(x.cuda(), gate.cuda(), w.cuda(), 1e-3, n), want, dtype)
    if dtype == BF16:
        packed = torch.zeros(16 * cols, dtype=BF16, device="cuda")
        ops.norm_gate(x.cuda(), gate.cuda(), w.cuda(), 1e-3, n, packed=packed)
        close(ops.unpack_rows(packed, rows, cols), want, dtype)


# ------------------------------------------------------------------------------------------------ mixture of experts
@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("experts,groups,keep,top", [(8, 2, 1, 4), (6, 3, 2, 3), (9, 1, 1, 1), (70, 7, 3, 5), (64, 64, 9, 9), (256, 8, 4, 8), (100, 10, 10, 33), (3, 3, 3, 3)])
def test_route(experts, groups, keep, top, dtype):
    from nanovllm_hip import ops
    rows, cols = 37, 192
    x, w = randn(rows, cols, seed=1, dtype=dtype), randn(experts, cols, seed=2, scale=cols ** -0.5, dtype=dtype)
    corr = randn(experts, seed=3, scale=0.5, dtype=F32) - 1.0                      # (choice scores of both signs)
    ids, weights = ops.moe_route(x.cuda(), w.cuda(), corr.cuda(), top, groups, keep, 2.5)
    z = f64(x) @ f64(w).T
    r = dict(groups=dict(count=groups, keep=keep), top=top, scale=2.5)
    clear = 0
    for t in range(rows):
        chosen, want, gap = G.route(z[t], f64(corr), r)
        if gap < 1e-5:
            continue
        clear += 1
        got = dict(zip(ids[t].tolist(), weights[t].tolist()))
        assert set(got) == set(chosen), (t, gap)
        assert all(abs(got[e] - g) < 1e-5 for e, g in zip(chosen, want.tolist()))
    assert clear > rows // 2


def test_route_closed_groups_stay_closed():
    """Choice scores far below zero: what a closed group holds still loses to every open expert; the correction never enters a weight."""
    from nanovllm_hip import ops
    x, w = torch.ones(1, 64, dtype=BF16).cuda(), torch.zeros(6, 64, dtype=BF16).cuda()
    corr = torch.tensor([-9.0, -8.0, -2.5, -30.0, -3.0, -3.5]).cuda()              # groups (0 1) (2 3) (4 5): sums -16, -31.5, -5.5 (+ 1 each)
    ids, weights = ops.moe_route(x, w, corr, 4, 3, 2, 1.0)
    assert sorted(ids[0].tolist()) == [0, 1, 4, 5] and torch.allclose(weights, torch.full((1, 4), 0.25, device="cuda"))


@pytest.mark.parametrize("pairs_shape,experts", [((1, 1), 4), ((70, 3), 5), ((1000, 8), 64), ((3000, 2), 300)])
@pytest.mark.parametrize("dtype", [BF16, F32])
def test_dispatch(pairs_shape, experts, dtype):
    from nanovllm_hip import ops
    g = torch.Generator().manual_seed(1)
    ids = torch.stack([torch.randperm(max(experts - 1, pairs_shape[1]), generator=g)[:pairs_shape[1]] for _ in range(pairs_shape[0])]).int()
    slots, tiles, _ = ops.moe_dispatch(ids.cuda(), experts, dtype)
    slots, tiles, flat = slots.cpu(), tiles.cpu(), ids.flatten()
    assert sorted(slots.tolist()) == list(range(ids.numel()))
    seen = torch.zeros(ids.numel(), dtype=torch.bool)
    used = 0
    for e, first, n, count in tiles.tolist():
        used += n > 0
        assert (flat[slots[first:first + n].long()] == e).all() and not seen[first:first + n].any()
        seen[first:first + n] = True
    assert seen.all() and all(t[3] == used for t in tiles.tolist())


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("rows,top,experts,n,k", [(1, 2, 4, 64, 64), (5, 4, 8, 128, 320), (33, 8, 16, 192, 128), (64, 1, 2, 64, 1088), (40, 3, 3, 2112, 192), (65, 2, 9, 64, 128),
                                                  (300, 4, 8, 192, 256), (700, 2, 3, 128, 64)])
def test_expert_products(rows, top, experts, n, k, dtype):
    """Both products against the reference expert by expert; batches of at most 64 rows in the small form and through the sorted tiles."""
    from nanovllm_hip import ops
    g = torch.Generator().manual_seed(rows)
    ids = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(rows)]).int()
    if rows > 2:
        ids[1:rows // 2] = ids[0]                                                  # one expert with many rows
    x = randn(rows, k, seed=1, dtype=dtype)
    gu, dn = randn(experts, 2 * n, k, seed=2, scale=k ** -0.5, dtype=dtype), randn(experts, k, n, seed=3, scale=n ** -0.5, dtype=dtype)
    forms = [ops.moe_dispatch(ids.cuda(), experts, dtype, r) for r in ([64] if dtype == F32 else [None, 128, 256])] + ([None] if dtype == BF16 and rows <= 64 else [])
    flat = ids.flatten().long()
    xr = f64(x).repeat_interleave(top, dim=0)
    for dispatch in forms:
        act = ops.moe_gemm(x.cuda(), gu.cuda(), ids.cuda(), True, dispatch)
        out = ops.moe_gemm(act, dn.cuda(), ids.cuda(), False, dispatch)
        for e in range(experts):
            p = (flat == e).nonzero().flatten()
            if len(p):
                want = G.silu(xr[p] @ f64(gu[e, :n]).T) * (xr[p] @ f64(gu[e, n:]).T)
                close(act[p.cuda()], want, dtype, f"act {e}", slack=2)
                close(out[p.cuda()], f64(act)[p] @ f64(dn[e]).T, dtype, f"out {e}", slack=2)


# ------------------------------------------------------------------------------------------------ residual, norm, cap
@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("rows,cols,n,top", [(3, 64, 64, 0), (5, 320, 300, 4), (17, 2048, 2048, 8), (2, 8192, 8190, 3)])
def test_residual_norm(rows, cols, n, top, dtype):
    from nanovllm_hip import ops
    x, y = randn(rows, cols, seed=1, dtype=F32) + 5.0, randn(rows, cols, seed=2, dtype=dtype)
    x[:, n:], y[:, n:] = 0, 0
    e, ew = randn(rows * max(top, 1), cols, seed=3, dtype=dtype), randn(rows, max(top, 1), seed=4, dtype=F32)
    e[:, n:] = 0
    w, b = torch.zeros(cols), torch.zeros(cols)
    w[:n], b[:n] = 1 + randn(n, seed=5, scale=0.3, dtype=F32), randn(n, seed=6, dtype=F32)
    for use_y, use_e in ((True, top > 0), (False, top > 0), (False, False), (True, False)):
        want = f64(x)
        if use_y:
            want = want + f64(y)
        if use_e:
            want = want + (f64(e).view(rows, top, cols) * f64(ew)[:, :, None]).sum(1)
        gx = x.cuda()
        packed = torch.zeros(32 * cols, dtype=BF16, device="cuda") if dtype == BF16 else None
        h = ops.residual_norm(gx, dtype, y=y.cuda() if use_y else None, experts=(e.cuda(), ew.cuda()) if use_e else None, weight=w.cuda(), bias=b.cuda(), eps=1e-3, n=n,
                              packed=packed)
        close(gx, want, F32, "stream")
        ln = torch.zeros(rows, cols, dtype=torch.float64)
        ln[:, :n] = G.layer_norm(want[:, :n], f64(w)[:n], f64(b)[:n], 1e-3)
        close(h, ln, dtype, "norm")
        if packed is not None:
            assert torch.equal(ops.unpack_rows(packed, rows, cols), h)
    gx = x.cuda()
    assert ops.residual_norm(gx, dtype, y=y.cuda()) is None
    close(gx, f64(x) + f64(y), F32, "addition only")


@pytest.mark.parametrize("dtype", [BF16, F32])
def test_softcap(dtype):
    from nanovllm_hip import ops
    x = randn(7, 130, seed=1, scale=30.0, dtype=dtype)
    buf = x.cuda()
    view = buf[:, :101]
    assert ops.softcap_(view, 15.0) is view
    close(view, G.softcap(f64(x)[:, :101], 15.0), dtype)
    assert torch.equal(buf[:, 101:].cpu(), x[:, 101:]) and not math.isnan(view.float().sum().item())
