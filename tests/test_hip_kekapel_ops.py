"""GPU: every mechanism of the Kekapel layers alone, each kernel form (fast, plain, fp32) against the plain float64 reference on the same rounded inputs.
Where many keys would hide a fault, one key of a sequence is scaled to take the whole softmax, at every border it could be lost or seen by mistake."""
import pytest
import torch

from oracle import kekapel_ref as K
from paged_cases import BF16, F32, Pages, close, f64, randn, standout_places

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------------------------------------ attention
def mixing(heads, seed=9):
    """Not symmetric, some heads swapped for others, negative parts."""
    t = torch.eye(heads) + randn(heads, heads, seed=seed, scale=0.5 * heads ** -0.5, dtype=F32)
    return t.roll(1, 0) * 0.7 + t * 0.5


def attend_ref(q, k, v, talk, pos, scale, cap, window=0, keep=0, sink=None):
    """q [rows, heads, dim] at positions pos over k, v [n, kvh, .]"""
    rows, heads, ratio = q.shape[0], q.shape[1], q.shape[1] // k.shape[1]
    i, j = torch.as_tensor(pos).view(-1, 1), torch.arange(k.shape[0])[None, :]
    ok = (j <= i) & ((i - j < window) | (j < keep) if window else j >= 0)
    s = torch.stack([f64(q)[:, h] @ f64(k)[:, h // ratio].T * scale for h in range(heads)])
    s = K.mix_heads(K.softcap(s, cap) if cap else s, f64(talk)).masked_fill(~ok, float("-inf"))
    if sink is not None:
        s = torch.cat([s, f64(sink).view(heads, 1, 1).expand(heads, rows, 1)], dim=2)
    p = torch.softmax(s, dim=-1)[:, :, :k.shape[0]]
    return torch.stack([p[h] @ f64(v)[:, h // ratio] for h in range(heads)], dim=1)


SHAPES = [(6, 2, 20, 12), (20, 2, 64, 128), (3, 3, 40, 100), (12, 3, 128, 128), (4, 1, 192, 128), (8, 4, 70, 200), (16, 1, 64, 64), (32, 4, 128, 120), (1, 1, 64, 64),
          (17, 17, 60, 64), (14, 14, 128, 128), (32, 8, 128, 128), (9, 3, 256, 250)]
ROWS_ONLY = [(40, 8, 16, 24), (64, 4, 64, 64), (16, 16, 128, 128)]     # more heads, or values of more heads, than the prompt kernel holds
PLAIN = [(2, 1, 270, 300), (70, 10, 8, 8)]
MASKS = [(0, 0), (1, 0), (64, 0), (65, 0), (100, 70), (7, 130)]


def test_supported_shapes():
    from nanovllm_hip import ops
    from nanovllm_hip.layers.paged_attention import padded_widths
    for shapes, rows, prompt in ((SHAPES, True, True), (ROWS_ONLY, True, False), (PLAIN, False, False)):
        for h, g, *w in shapes:
            assert (ops.talk_rows_supported(h, *padded_widths(*w), 64), ops.talk_prompt_supported(h, g, *padded_widths(*w), 64, 5.0)) == (rows, prompt), (h, w)
    for cap in (0.0, 2e4):
        assert not ops.talk_prompt_supported(4, 2, 64, 64, 64, cap)


@pytest.mark.parametrize("dtype,generic", [(BF16, False), (BF16, True), (F32, False)])
@pytest.mark.parametrize("heads,kvh,dim,vdim", SHAPES + ROWS_ONLY + PLAIN)
def test_rows(heads, kvh, dim, vdim, dtype, generic):
    from nanovllm_hip import ops
    lengths = [1, 2, 64, 65, 129, 300]
    pg = Pages(lengths, kvh, dim, vdim, dtype)
    cache, tables = pg.cache(), pg.tables.cuda()
    q, talk = randn(len(lengths), heads, dim, seed=5, dtype=dtype), mixing(heads)
    sink = randn(heads, seed=6, dtype=F32)
    pos = torch.tensor([n - 1 for n in lengths])
    for n_mask, (window, keep) in enumerate(MASKS):
        cap, sk = ((3.0, None), (0.0, sink), (20.0, None))[n_mask % 3]
        want = torch.cat([attend_ref(q[i:i + 1], pg.k[i], pg.v[i], talk, [n - 1], 0.2, cap, window, keep, sk) for i, n in enumerate(lengths)])
        for splits in (None, 1, 3, 5):
            got = ops.talk_rows(pg.pad_q(q), cache, tables, pos.cuda(), heads, kvh, pg.dk, pg.dv, 0.2, 300, talk.cuda(), cap, window, keep,
                                sk.cuda() if sk is not None else None, splits=splits, generic=generic)
            close(pg.unpad(got, heads), want, dtype, f"window {window} keep {keep} splits {splits}", slack=2)


def test_rows_packed_output_row_seq_and_pieces(monkeypatch):
    from nanovllm_hip import ops
    heads, kvh, dim, vdim = 4, 2, 64, 128
    pg = Pages([70, 200, 5], kvh, dim, vdim, BF16)
    cache, tables = pg.cache(), pg.tables.cuda()
    q, talk = randn(3, heads, dim, seed=5), mixing(heads).cuda()
    pos = torch.tensor([69, 199, 4]).cuda()
    args = (heads, kvh, pg.dk, pg.dv, 0.3, 200, talk, 5.0, 50)
    rows = ops.talk_rows(pg.pad_q(q), cache, tables, pos, *args)
    packed = torch.zeros(16 * heads * vdim, dtype=BF16, device="cuda")
    assert ops.talk_rows(pg.pad_q(q), cache, tables, pos, *args, out_packed=packed, want_out=False, splits=2) is None
    close(ops.unpack_rows(packed, 3, heads * vdim), f64(rows), BF16)
    seq = torch.tensor([2, 0, 1], dtype=torch.int32).cuda()              # rows of other sequences, in another order
    moved = (pg.pad_q(q[[2, 0, 1]]), cache, tables, pos[[2, 0, 1]].contiguous(), *args)
    close(ops.talk_rows(*moved, row_seq=seq), f64(rows)[[2, 0, 1]], BF16)
    monkeypatch.setattr(ops, "SCORE_BYTES", 1)                            # one row per launch
    close(ops.talk_rows(*moved, row_seq=seq), f64(rows)[[2, 0, 1]], BF16)
    close(ops.talk_rows(pg.pad_q(q), cache, tables, pos, *args), f64(rows), BF16)


def asking(pg, places, kvh, dtype):
    """Queries that ask for the key at place i of sequence i: it gets a score of about 17, the others about 0.5."""
    q = randn(len(places), kvh, pg.dim, seed=7, dtype=dtype)
    for i, a in enumerate(places):
        pg.k[i] = pg.k[i] * 0.3
        pg.k[i][a] = q[i] * 2
    return q


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("window,keep", [(0, 0), (64, 0), (65, 0), (40, 0), (130, 4), (40, 70)])
def test_rows_one_key_stands_out(window, keep, dtype):
    """A key whose score dwarfs the others' takes the output where it is seen, and changes nothing where it is not."""
    from nanovllm_hip import ops
    heads, kvh, dim, vdim = 4, 2, 64, 64
    talk = torch.eye(heads) + randn(heads, heads, seed=3, scale=0.1, dtype=F32)
    for pos in (199, 192, 255):
        places = standout_places(pos, window, keep)
        pg = Pages([pos + 1] * len(places), kvh, dim, vdim, dtype)
        q = asking(pg, places, kvh, dtype).repeat_interleave(heads // kvh, dim=1)
        want = torch.cat([attend_ref(q[i:i + 1], pg.k[i], pg.v[i], talk, [pos], 0.2, 20.0, window, keep) for i in range(len(places))])
        for i, a in enumerate(places):
            seen = not window or pos - a < window or a < keep
            assert ((want[i, 0] - f64(pg.v[i])[a, 0]).abs().max() < 0.05) == seen
        for splits in (1, 4):
            got = ops.talk_rows(pg.pad_q(q), pg.cache(), pg.tables.cuda(), torch.full((len(places),), pos).cuda(), heads, kvh, pg.dk, pg.dv, 0.2, 256, talk.cuda(), 20.0,
                                window, keep, splits=splits)
            close(pg.unpad(got, heads), want, dtype, f"pos {pos}", slack=2)


PORTIONS = [(2, 2), (64, 64), (2, 65), (65, 129), (130, 300), (300, 300), (3, 400), (57, 190)]


@pytest.mark.parametrize("window,keep", MASKS)
@pytest.mark.parametrize("heads,kvh,dim,vdim", SHAPES)
def test_prompt(heads, kvh, dim, vdim, window, keep):
    """Portions of several sequences (rows, keys) in one launch."""
    from nanovllm_hip import ops
    sink, talk = randn(heads, seed=6, dtype=F32) if keep else None, mixing(heads)
    for cap, portions in ((3.0, PORTIONS[:5]), (50.0, PORTIONS[3:])) if heads <= 12 and dim <= 128 else ((15.0, PORTIONS[2:6]),):
        pg = Pages([k for _, k in portions], kvh, dim, vdim, BF16, seed=3)
        q = randn(sum(r for r, _ in portions), heads, dim, seed=8)
        cu_q = torch.tensor([0] + [r for r, _ in portions]).cumsum(0).int().cuda()
        cu_k = torch.tensor([0] + [k for _, k in portions]).cumsum(0).int().cuda()
        got = pg.unpad(ops.talk_prompt(pg.pad_q(q), pg.cache(), pg.tables.cuda(), cu_q, cu_k, max(r for r, _ in portions), heads, kvh, pg.dk, pg.dv, 0.2, talk.cuda(), cap,
                                       window, keep, sink.cuda() if keep else None), heads)
        at = 0
        for i, (r, k) in enumerate(portions):
            t = torch.tensor(sorted({0, 1, r // 2, r - 2, r - 1, min(15, r - 1), min(16, r - 1), min(63, r - 1), min(64, r - 1)}))
            want = attend_ref(q[at + t], pg.k[i], pg.v[i], talk, k - r + t, 0.2, cap, window, keep, sink)
            close(got[at + t], want, BF16, f"portion {i}", slack=2)
            at += r


@pytest.mark.parametrize("window,keep", [(0, 0), (64, 0), (65, 0), (40, 0), (33, 0), (130, 4), (40, 70)])
@pytest.mark.parametrize("portion", [2, 40, 200])
def test_prompt_one_key_stands_out(window, keep, portion):
    from nanovllm_hip import ops
    heads, kvh, dim, vdim, n = 5, 1, 64, 64, 200
    talk = torch.eye(heads) + randn(heads, heads, seed=3, scale=0.1, dtype=F32)
    places = sorted({a for pos in (n - 1, n - 2, n - portion) for a in standout_places(pos, window, keep)})
    pg = Pages([n] * len(places), kvh, dim, vdim, BF16)
    q = asking(pg, places, kvh, BF16).repeat_interleave(portion, dim=0).repeat_interleave(heads, dim=1)   # every row of a portion asks for the same key
    cu_q = (torch.arange(len(places) + 1) * portion).int().cuda()
    cu_k = (torch.arange(len(places) + 1) * n).int().cuda()
    got = pg.unpad(ops.talk_prompt(pg.pad_q(q), pg.cache(), pg.tables.cuda(), cu_q, cu_k, portion, heads, kvh, pg.dk, pg.dv, 0.2, talk.cuda(), 20.0, window, keep), heads)
    for i, a in enumerate(places):
        t = torch.tensor(sorted({0, 1, portion // 2, portion - 2, portion - 1} |
                                {x - (n - portion) for x in (a, a - 1, a + window - 1, a + window) if 0 <= x - (n - portion) < portion}))
        want = attend_ref(q[i * portion + t], pg.k[i], pg.v[i], talk, n - portion + t, 0.2, 20.0, window, keep)
        close(got[i * portion + t], want, BF16, f"key {a}", slack=2)


@pytest.mark.parametrize("dtype", [BF16, F32])
def test_a_head_sees_where_another_looks(dtype):
    """Permuted heads: head h attends by head h + 1's scores, in rows and in a prompt, though its own query asks for another key."""
    from nanovllm_hip import ops
    heads, kvh, dim, n = 4, 4, 64, 120
    pg = Pages([n], kvh, dim, dim, dtype)
    q, talk, keys = randn(1, heads, dim, seed=7, dtype=dtype), torch.eye(heads).roll(1, 1), [5, 63, 64, 118]
    pg.k[0] = pg.k[0] * 0.3
    for h in range(heads):
        pg.k[0][keys[h], h] = q[0, h] * 2
    want = torch.stack([f64(pg.v[0])[keys[(h + 1) % heads], h] for h in range(heads)])
    got = ops.talk_rows(pg.pad_q(q), pg.cache(), pg.tables.cuda(), torch.tensor([n - 1]).cuda(), heads, kvh, 64, 64, 0.2, n, talk.cuda(), 20.0)
    assert (pg.unpad(got, heads)[0] - want).abs().max() < 0.05
    if dtype == BF16:
        cu_q, cu_k = torch.tensor([0, 2], dtype=torch.int32).cuda(), torch.tensor([0, n], dtype=torch.int32).cuda()
        got = ops.talk_prompt(pg.pad_q(q.repeat(2, 1, 1)), pg.cache(), pg.tables.cuda(), cu_q, cu_k, 2, heads, kvh, 64, 64, 0.2, talk.cuda(), 20.0)
        assert (pg.unpad(got, heads)[1] - want).abs().max() < 0.05


# ------------------------------------------------------------------------------------------------ row ops
def padded(t, width):
    out = torch.zeros(*t.shape[:-1], width, dtype=t.dtype)
    out[..., :t.shape[-1]] = t
    return out


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("heads,kvh,dim,vdim", [(4, 2, 64, 64), (3, 1, 20, 36), (6, 6, 130, 130), (40, 8, 128, 128), (3, 1, 250, 64), (7, 7, 8, 300), (2, 1, 270, 16)])
def test_norm_per_head(heads, kvh, dim, vdim, dtype):
    from nanovllm_hip import ops
    from nanovllm_hip.layers.paged_attention import padded_widths
    dk, dv = padded_widths(dim, vdim)
    rows, bs, pages = 5, 64, 3
    parts = [randn(rows, h, w, seed=i, dtype=dtype) for i, (h, w) in enumerate(((heads, dim), (kvh, dim), (kvh, vdim)))]
    parts[0] = parts[0] * torch.tensor([3.0, 0.1, 1.0] * heads)[:heads, None].to(dtype)                   # heads of unlike size: one's mean must not enter another's
    qkv = torch.cat([padded(t, w).reshape(rows, -1) for t, w in zip(parts, (dk, dk, dv))], dim=1).cuda()
    qw, kw = (1 + randn(dim, seed=s, scale=0.3, dtype=F32) for s in (7, 8))
    slots = torch.tensor([5, 63, 64, -1, 191], dtype=torch.int32)
    cache = torch.full((pages, bs, kvh * (dk + dv)), 7.0, dtype=dtype, device="cuda")
    ops.attn_prep(qkv, heads, kvh, dk, dv, torch.arange(rows).cuda(), None, cache, slots.cuda(), q_weight=padded(qw, dk).cuda(), k_weight=padded(kw, dk).cuda(), q_n=dim, k_n=dim,
                  eps=1e-3, head_norm=True)
    q, k = (K.unit_rms(f64(t), 1e-3) * f64(w) for t, w in zip(parts, (qw, kw)))
    got = qkv[:, :heads * dk].reshape(rows, heads, dk)
    close(got[..., :dim], q, dtype, "queries")
    assert not got[..., dim:].any()
    flat = cache.view(pages, kvh, bs * (dk + dv))
    keys, vals = flat[:, :, :bs * dk].view(pages, kvh, bs, dk), flat[:, :, bs * dk:].view(pages, kvh, bs, dv)
    for i, s in enumerate(slots.tolist()):
        if s >= 0:
            close(keys[s // bs, :, s % bs, :dim], k[i], dtype, f"key {i}")
            assert torch.equal(f64(vals[s // bs, :, s % bs, :vdim]), f64(parts[2])[i])
    assert (keys == 7.0).all(-1).sum() == kvh * (pages * bs - 4)                                          # nothing else was written


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("rows,cols,n", [(1, 64, 50), (5, 320, 300), (17, 3072, 3072), (2, 20480, 20475)])
def test_poly_norm(rows, cols, n, dtype):
    from nanovllm_hip import ops
    z = randn(rows, cols + 64, seed=1, dtype=dtype)[:, :cols].contiguous() * torch.logspace(-2, 1, rows)[:, None].to(dtype)
    z[:, n:] = 0
    coef = torch.tensor([0.7, -0.4, 0.5, 0.2])
    want = torch.zeros(rows, cols, dtype=torch.float64)
    want[:, :n] = K.poly_norm(f64(z)[:, :n], f64(coef), 1e-4)
    close(ops.poly_norm(z.cuda(), coef.cuda(), 1e-4, n), want, dtype)
    if dtype == BF16:
        packed = torch.zeros((rows + 15) // 16 * 16 * cols, dtype=BF16, device="cuda")
        assert ops.poly_norm(z.cuda(), coef.cuda(), 1e-4, n, packed=packed) is None
        close(ops.unpack_rows(packed, rows, cols), want, dtype)


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("rows,cols,n,top", [(3, 64, 64, 0), (5, 320, 300, 4), (17, 2048, 2048, 8), (2, 8192, 8190, 3)])
def test_residual_with_norms_on_both_sides(rows, cols, n, top, dtype):
    """x += mult norm(sublayer), += embedding, += step vector, norm of the result: in every combination a pass uses."""
    from nanovllm_hip import ops
    x, y = randn(rows, cols, seed=1, dtype=F32) + 5.0, randn(rows, cols, seed=2, dtype=dtype) + 2.0
    e, ew = randn(rows * max(top, 1), cols, seed=3, dtype=dtype), randn(rows, max(top, 1), seed=4, dtype=F32)
    base, shift = randn(rows, cols, seed=7, dtype=F32), randn(cols, seed=8, dtype=F32)
    for t in (x, y, e, base):
        t[:, n:] = 0
    shift[n:] = 0
    w, b, pw, pb = (padded(t, cols) for t in (1 + randn(n, seed=5, scale=0.3, dtype=F32), randn(n, seed=6, dtype=F32), 1 + randn(n, seed=9, scale=0.3, dtype=F32),
                                              randn(n, seed=10, dtype=F32)))

    def ln(t, w, b):
        out = torch.zeros_like(t)
        out[:, :n] = K.layer_norm(t[:, :n], f64(w)[:n], f64(b)[:n], 1e-3)
        return out
    for use_y, use_e, first, begins, mult in ((True, False, False, False, 0.6), (False, top > 0, True, True, 0.6), (False, False, False, True, 1.0), (True, False, True, True, 1.0),
                                              (True, False, False, True, 0.3)):
        added = torch.zeros(rows, cols, dtype=torch.float64)
        if use_y:
            added += f64(y)
        if use_e:
            added += (f64(e).view(rows, top, cols) * f64(ew)[:, :, None]).sum(1)
        want = f64(x) + (mult * ln(added, pw, pb) if use_y or use_e else 0.0) + (f64(base) if first else 0.0) + (f64(shift) if begins else 0.0)
        gx = x.cuda()
        packed = torch.zeros(32 * cols, dtype=BF16, device="cuda") if dtype == BF16 else None
        h = ops.residual_norm(gx, dtype, y=y.cuda() if use_y else None, experts=(e.cuda(), ew.cuda()) if use_e else None, weight=w.cuda(), bias=b.cuda(), eps=1e-3, n=n,
                              packed=packed, post=(pw.cuda(), pb.cuda()) if use_y or use_e else None, mult=mult, base=base.cuda() if first else None,
                              shift=shift.cuda() if begins else None)
        close(gx, want, F32, "stream")
        close(h, ln(want, w, b), dtype, "norm")
        if packed is not None:
            assert torch.equal(ops.unpack_rows(packed, rows, cols), h)


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("rows,cols", [(1, 64), (9, 320), (40, 2048)])
def test_embedding_with_positions(rows, cols, dtype):
    from nanovllm_hip import ops
    embed, table = randn(50, cols, seed=1, dtype=dtype), randn(30, cols, seed=2, dtype=F32)
    toks, pos = torch.arange(rows) * 7 % 50, torch.arange(rows) * 11 % 30
    toks[0], pos[-1] = 49, 29
    copy = torch.zeros(rows, cols, device="cuda")
    x, xb = ops.embed_rows(toks.cuda(), embed.cuda(), 3.5, positions=pos.cuda(), table=table.cuda(), copy=copy)
    want = f64(embed)[toks] * 3.5 + f64(table)[pos]
    close(x, want, F32)
    close(xb, want, dtype)
    assert torch.equal(x, copy)


# ------------------------------------------------------------------------------------------------ experts
@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("experts,top", [(4, 1), (6, 3), (70, 5), (64, 9), (256, 8), (33, 33), (1, 1)])
def test_softmax_route(experts, top, dtype):
    from nanovllm_hip import ops
    rows, cols = 37, 192
    x, w = randn(rows, cols, seed=1, dtype=dtype), randn(experts, cols, seed=2, scale=2 * cols ** -0.5, dtype=dtype)
    bias = randn(experts, seed=3, dtype=F32) - 40.0                                # (far below zero, so a sum of exponentials needs its largest entry taken off)
    ids, weights = ops.moe_route(x.cuda(), w.cuda(), bias.cuda(), top, softmax=True)
    z = f64(x) @ f64(w).T + f64(bias)
    clear = 0
    for t in range(rows):
        chosen, want, gap = K.route(z[t], top)
        if gap < 1e-4:
            continue
        clear += 1
        got = dict(zip(ids[t].tolist(), weights[t].tolist()))
        assert set(got) == set(chosen), (t, gap)
        assert all(abs(got[e] - g) < 3e-5 for e, g in zip(chosen, want.tolist()))
    assert clear > rows // 2


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("rows,top,experts,n,k,limit", [(1, 2, 4, 64, 64, 1.0), (5, 4, 8, 128, 320, 0.5), (64, 1, 2, 64, 1088, 2.0), (65, 2, 9, 64, 128, 0.9), (300, 4, 8, 192, 256, 7.0),
                                                        (700, 2, 3, 128, 64, 0.3)])
def test_clamped_expert_products(rows, top, experts, n, k, limit, dtype):
    """The clamped unit in every form of the first product."""
    from nanovllm_hip import ops
    g = torch.Generator().manual_seed(rows)
    ids = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(rows)]).int()
    x, gu = randn(rows, k, seed=1, dtype=dtype), randn(experts, 2 * n, k, seed=2, scale=1.5 * k ** -0.5, dtype=dtype)
    forms = [ops.moe_dispatch(ids.cuda(), experts, dtype, r) for r in ([64] if dtype == F32 else [None, 128, 256])] + ([None] if dtype == BF16 and rows <= 64 else [])
    flat, xr = ids.flatten().long(), f64(x).repeat_interleave(top, dim=0)
    for dispatch in forms:
        act = ops.moe_gemm(x.cuda(), gu.cuda(), ids.cuda(), True, dispatch, (limit, 1.702))
        for e in range(experts):
            p = (flat == e).nonzero().flatten()
            if len(p):
                close(act[p.cuda()], K.clamped_unit(xr[p] @ f64(gu[e, :n]).T, xr[p] @ f64(gu[e, n:]).T, limit), dtype, f"expert {e}", slack=2)
