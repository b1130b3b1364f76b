"""GPU: every mechanism of the Zaposun layers alone, each kernel form (fast, plain, fp32; portions, single tokens) against the plain float64 reference on the same
rounded inputs.  State pools start full of garbage: a sequence's first token must not see it.  Where many keys would hide a fault, one key of a sequence is scaled to take
the whole softmax, at every border it could be lost or seen by mistake."""
import pytest
import torch

from oracle import zaposun_ref as Z
from paged_cases import BF16, F32, Pages, close, f64, randn
from zaposun_cases import Portions, feed_plan

pytestmark = pytest.mark.gpu


def ops():
    from nanovllm_hip import ops
    return ops


def padded(t, *shape):
    from nanovllm_hip.layers.linear import padded
    return padded(t, *shape)


# ------------------------------------------------------------------------------------------------ embedding
@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("buckets,mul_prev,mul_cur", [(31, 7, 5), (1, 3, 2), (100003, 90001, 70001)])
def test_bigram_embed(buckets, mul_prev, mul_cur, dtype):
    vocab, cols = 50, 72
    embed, bigram = randn(vocab, cols, dtype=dtype), randn(min(buckets, 100003) + 1, cols, seed=1, dtype=dtype)
    lengths, cuts, slots = [40, 1, 9, 23], [[3, 1, 1, 7], [1], [2, 1], [1, 12, 2]], [4, 0, 2, 1]
    toks = [torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(n)) for n in lengths]
    want = [f64(embed)[t] + f64(bigram)[torch.tensor(Z.bigram_rows(t.tolist(), buckets, mul_prev, mul_cur))] for t in toks]
    last = torch.full((5,), 17, dtype=torch.int64).cuda()
    got = [[] for _ in lengths]
    for batch in feed_plan(lengths, cuts, slots):
        p = Portions([(a, n, s) for _, a, n, s in batch])
        x = ops().bigram_embed(torch.cat([toks[i][a:a + n] for i, a, n, _ in batch]).cuda(), p.positions, p.meta(), embed.cuda(), bigram.cuda(), mul_prev, mul_cur, last)
        for (i, *_), rows in zip(batch, x.split([n for _, _, n, _ in batch])):
            got[i].append(rows)
    for g, w in zip(got, want):
        close(torch.cat(g), w, F32)
    assert [last[s].item() for s in slots] == [t[-1].item() for t in toks] and last[3].item() == 17


# ------------------------------------------------------------------------------------------------ streams
@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("streams,n,cols,groups", [(1, 64, 64, 1), (2, 72, 128, 3), (3, 136, 192, 8), (4, 352, 384, 2), (4, 2048, 2048, 4), (5, 100, 128, 100), (8, 1000, 1024, 5), (16, 72, 72, 1),
                                                   (4, 4160, 4160, 2), (2, 9000, 9024, 6)])
def test_stream_mix(streams, n, cols, groups, dtype):
    rows, eps = 5, 1e-3
    xs = padded(randn(rows, streams, n, dtype=F32), rows, streams, cols)
    y, y2 = (padded(randn(rows, n, seed=s, dtype=dtype, scale=0.5), rows, cols) for s in (1, 2))
    mix, out, read = randn(streams, streams, seed=3, dtype=F32), randn(streams, seed=4, dtype=F32), randn(streams, seed=5, dtype=F32)
    w, wa, wb = (padded(randn(n, seed=s, dtype=F32), cols) for s in (6, 7, 8))
    x64, y64 = f64(xs).transpose(0, 1)[..., :n], f64(y)[:, :n]
    both = 0.5 * (Z.rms(y64, eps) * f64(wa)[:n] + Z.rms(f64(y2)[:, :n], eps) * f64(wb)[:n])
    for alike in (False, True):
        base = x64 if not alike else x64[:1].expand(streams, -1, -1)
        for post in (False, True):
            new = Z.update_streams(base, f64(mix), f64(out), both if post else y64)
            src = xs.cuda() if not alike else xs[:, 0].contiguous().cuda()
            dst = torch.full((rows, streams, cols), 9.0).cuda() if alike else None
            update = dict(y=y.cuda(), mix=mix.cuda(), out=out.cuda(), eps=eps, post=(y2.cuda(), wa.cuda(), wb.cuda(), 0.5) if post else None)
            packed = torch.zeros(16 * cols, dtype=BF16, device="cuda") if dtype == BF16 and cols % 32 == 0 else None
            h = ops().stream_mix(src, streams, dtype, n, update, read.cuda(), (w.cuda(), groups, eps), packed=packed, out=dst)
            got = dst if alike else src
            close(got[..., :n], new.transpose(0, 1), F32)
            assert not got[..., n:].any() and not h[:, n:].any()
            want = Z.group_norm(Z.read_streams(new, f64(read)), f64(w)[:n], groups, eps)
            close(h[:, :n], want, dtype)
            if packed is not None:
                assert torch.equal(ops().unpack_rows(packed, rows, cols), h)
        u = ops().stream_mix(xs.cuda() if not alike else xs[:, 0].contiguous().cuda(), streams, dtype, n)
        close(u[:, :n], base.sum(0), F32)
        h = ops().stream_mix(xs.cuda() if not alike else xs[:, 0].contiguous().cuda(), streams, dtype, n, None, read.cuda(), (w.cuda(), groups, eps))
        close(h[:, :n], Z.group_norm(Z.read_streams(base, f64(read)), f64(w)[:n], groups, eps), dtype)


# ------------------------------------------------------------------------------------------------ shift, convolution
LENGTHS, SLOTS = [1500, 1, 2, 77, 64], [3, 0, 5, 1, 4]
CUTS = [[700, 1, 2, 1, 1, 300], [1], [1], [2, 1, 3, 1, 1, 40], [64]]


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("mixes", [0, 1, 5])
def test_token_shift(mixes, dtype):
    """Portions down to one token, the first tokens of a sequence, several sequences in one batch (long batches take several rows per thread)."""
    cols = 136
    h = [randn(n, cols, seed=n, dtype=dtype) for n in LENGTHS]
    shift, mu = randn(cols, seed=1, dtype=F32), randn(mixes, cols, seed=2, dtype=F32)
    want = []
    for x in h:
        s = Z.lerp_previous(f64(x), f64(shift))
        want.append(torch.stack([Z.lerp_previous(s, f64(m)) for m in mu]) if mixes else s[None])
    ring = torch.full((6, 3 if mixes else 2, cols), 50.0, dtype=dtype).cuda()
    got = [[] for _ in h]
    for batch in feed_plan(LENGTHS, CUTS, SLOTS):
        p = Portions([(a, n, s) for _, a, n, s in batch])
        rows = torch.cat([h[i][a:a + n] for i, a, n, _ in batch]).cuda()
        out = ops().token_shift(rows, p.positions, p.meta(), shift.cuda(), ring, mu.cuda() if mixes else None)
        for (i, *_), part in zip(batch, out.split([n for _, _, n, _ in batch], dim=1)):
            got[i].append(part)
    for g, w in zip(got, want):
        close(torch.cat(g, dim=1), w, dtype)
    assert (ring[2] == 50).all()                                        # (no sequence has this slot)


def test_token_shift_packed():
    cols, rows = 128, 19
    h, shift, mu = randn(rows, cols), randn(cols, seed=1, dtype=F32), randn(5, cols, seed=2, dtype=F32)
    p = Portions([(7, 1, i) for i in range(rows)])
    ring = randn(rows, 3, cols, seed=3).cuda()
    want = ops().token_shift(h.cuda(), p.positions, p.meta(), shift.cuda(), ring.clone(), mu.cuda())
    packed = torch.zeros(5 * 32 * cols, dtype=BF16, device="cuda")
    assert ops().token_shift(h.cuda(), p.positions, p.meta(), shift.cuda(), ring, mu.cuda(), packed=packed) is None
    for k in range(5):
        assert torch.equal(ops().unpack_rows(packed[k * 32 * cols:(k + 1) * 32 * cols], rows, cols), want[k])


@pytest.mark.parametrize("mixes", [0, 5])
@pytest.mark.parametrize("streams,n,cols", [(1, 64, 64), (3, 100, 128), (4, 2048, 2048)])
def test_shift_inside_the_stream_update(streams, n, cols, mixes):
    """Single tokens: the norm and the shift in one launch give what the two launches give, rows, ring and all; first tokens and second ones too."""
    rows = 19
    x, y = padded(randn(rows, streams, n, dtype=F32), rows, streams, cols).cuda(), padded(randn(rows, n, seed=1), rows, cols).cuda()
    w, shift = (padded(randn(n, seed=s, dtype=F32), cols).cuda() for s in (2, 4))
    read = randn(streams, seed=5, dtype=F32).cuda()
    update = dict(y=y, mix=randn(streams, streams, seed=6, dtype=F32).cuda(), out=randn(streams, seed=7, dtype=F32).cuda())
    norm, mu = (w, 1, 1e-5), randn(mixes, cols, seed=8, dtype=F32).cuda() if mixes else None
    p = Portions([(i % 4 if i < 12 else 700 + i, 1, 18 - i) for i in range(rows)])
    rings = [randn(rows, 3 if mixes else 2, cols, seed=9).cuda() for _ in range(2)]
    xs = [x.clone(), x.clone()]
    packs = [torch.zeros(max(mixes, 1) * 32 * cols, dtype=BF16, device="cuda") for _ in range(2)]
    h = ops().stream_mix(xs[0], streams, BF16, n, update, read, norm)
    ops().token_shift(h, p.positions, p.meta(), shift, rings[0], mu, packed=packs[0])
    assert ops().stream_mix(xs[1], streams, BF16, n, update, read, norm, want_rows=False,
                            shift=dict(positions=p.positions, step=p.meta(), shift=shift, ring=rings[1], mu=mu, packed=packs[1])) is None
    assert torch.equal(xs[0], xs[1]) and torch.equal(rings[0], rings[1])
    close(packs[1], f64(packs[0]), BF16)


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
def test_causal_conv(taps, dtype):
    cols = 72
    x = [randn(n, cols, seed=n, dtype=dtype) for n in LENGTHS]
    w, b = randn(taps, cols, seed=1, dtype=F32), randn(cols, seed=2, dtype=F32)
    want = [Z.silu(Z.causal_conv(f64(t), f64(w).T, f64(b))) for t in x]
    ring = torch.full((6, taps, cols), 50.0, dtype=dtype).cuda()
    got = [[] for _ in x]
    for batch in feed_plan(LENGTHS, CUTS, SLOTS):
        p = Portions([(a, n, s) for _, a, n, s in batch])
        wide = torch.cat([torch.cat([x[i][a:a + n] for i, a, n, _ in batch]), torch.full((p.rows, cols), 9.0, dtype=dtype)], dim=1).cuda()      # (a slice of wider rows)
        out = ops().causal_conv(wide[:, :cols], p.positions, p.meta(), w.cuda(), b.cuda(), ring)
        for (i, *_), part in zip(batch, out.split([n for _, _, n, _ in batch])):
            got[i].append(part)
    for g, t in zip(got, want):
        close(torch.cat(g), t, dtype)


# ------------------------------------------------------------------------------------------------ selective scan
class Scan:
    """Random operands of one scan layer and the plain result for several sequences."""

    def __init__(self, lengths, inner, n, rank, dtype, a_lo=-4.0, a_hi=1.5):
        self.inner, self.n, self.rank, self.dtype, self.kept = inner, n, rank, dtype, ops().scan_states(n)
        self.x, self.z, self.low = ([randn(t, w, seed=10 * t + s, dtype=dtype) for t in lengths] for s, w in ((1, inner), (2, inner), (3, rank)))
        self.bc = [randn(t, 2, n, seed=10 * t + 4, dtype=dtype) for t in lengths]
        gen = torch.Generator().manual_seed(n)
        self.a = -torch.exp(torch.rand(inner, n, generator=gen) * (a_hi - a_lo) + a_lo)
        self.d, self.bias, self.w_dt = randn(inner, seed=5, dtype=F32), torch.rand(inner, generator=gen) * 4 - 5, randn(inner, rank, seed=6, scale=rank ** -0.5, dtype=dtype)
        self.dt = [(f64(t) @ f64(self.w_dt).T).to(dtype) for t in self.low]
        self.want = []
        for x, z, dt, bc in zip(self.x, self.z, self.dt, self.bc):
            y, s = Z.selective_scan(f64(x), Z.softplus(f64(dt) + f64(self.bias)), f64(self.a), f64(bc)[:, 0], f64(bc)[:, 1], f64(self.d))
            self.want.append((y * Z.silu(f64(z)), s))
        self.params = dict(a_log2=padded(self.a * 1.4426950408889634, inner, self.kept).cuda(), d=self.d.cuda(), dt_bias=self.bias.cuda(), w_dt=self.w_dt.cuda())

    def rows(self, what, batch):
        t = torch.cat([getattr(self, what)[i][a:a + k] for i, a, k, _ in batch])
        return (padded(t, t.shape[0], 2, self.kept).reshape(t.shape[0], -1) if what == "bc" else t).cuda()

    def run(self, batch, state, segment=64, step=False):
        p = Portions([(a, k, s) for _, a, k, s in batch])
        x, z, bc = (self.rows(w, batch) for w in ("x", "z", "bc"))
        if step:
            return ops().scan_step(x, self.rows("low", batch), bc, z, self.params, p.positions, p.slots, state)
        chunks, more = p.chunks(segment)
        return ops().scan_chunks(x, self.rows("dt", batch), bc, z, self.params, p.positions, p.slots, chunks, more, state)


def feed_scan(layer, lengths, cuts, slots, segment, steps=False):
    state = torch.full((max(slots) + 1, layer.inner, layer.kept), 30.0).cuda()
    got = [[] for _ in lengths]
    for batch in feed_plan(lengths, cuts, slots):
        singles = [e for e in batch if e[2] == 1] if steps else []
        for part in (singles, [e for e in batch if e not in singles]):
            if part:
                out = layer.run(part, state, segment, step=part is singles)
                for (i, *_), rows in zip(part, out.split([k for _, _, k, _ in part])):
                    got[i].append(rows)
    return [torch.cat(g) for g in got], state


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("inner,n,rank", [(8, 1, 8), (72, 5, 16), (64, 16, 64), (136, 16, 8), (320, 30, 24), (64, 50, 8), (40, 100, 8), (24, 256, 8)])
def test_scan_portions(inner, n, rank, dtype):
    lengths, cuts, slots = [300, 2, 65, 131], [[150, 1, 2, 3, 64], [1], [65], [2, 129]], [2, 0, 3, 4]
    layer = Scan(lengths, inner, n, rank, dtype)
    for segment in (64, 128, 1024):
        got, state = feed_scan(layer, lengths, cuts, slots, segment)
        for i, (y, s) in enumerate(layer.want):
            close(got[i], y, dtype, f"segment {segment} sequence {i}")
            close(state[slots[i], :, :n], s, F32, f"state {i}", slack=4)
            assert not state[slots[i], :, n:].any()
        assert (state[1] == 30).all()


@pytest.mark.parametrize("inner,n,rank", [(72, 5, 16), (64, 16, 64), (8192, 16, 128), (320, 30, 24), (64, 50, 8), (40, 100, 72), (24, 256, 8)])
def test_scan_step(inner, n, rank):
    """Single tokens behind portions; many channels take several rows per workgroup."""
    lengths = [40, 9, 33, 21, 5] if inner > 1000 else [90, 9, 70]
    cuts, slots = [[30, 1, 1, 1], [1], [2, 1, 1], [1], [3, 1]][:len(lengths)], [2, 0, 3, 4, 1][:len(lengths)]
    layer = Scan(lengths, inner, n, rank, BF16)
    got, state = feed_scan(layer, lengths, cuts, slots, 64, steps=True)
    for i, (y, s) in enumerate(layer.want):
        close(got[i], y, BF16, f"sequence {i}", slack=2)                 # (the portions' step sizes are rounded once more)
        close(state[slots[i], :, :n], s, BF16, f"state {i}", slack=2)


@pytest.mark.parametrize("dtype,steps", [(BF16, False), (BF16, True), (F32, False)])
def test_scan_remembers_for_long(dtype, steps):
    """An input a thousand tokens back is still there where the decay is slow, and gone where it is fast; across segments, portions and single tokens."""
    n_tok, inner, n = 1003, 64, 16
    layer = Scan([n_tok], inner, n, 8, dtype)
    a = torch.full((inner, n), -1e-4)
    a[inner // 2:] = -300.0
    layer.params["a_log2"] = (a * 1.4426950408889634).cuda()
    layer.x[0][1:] = 0
    layer.z[0][:] = 1.0
    layer.params["d"] = torch.zeros(inner).cuda()
    y, _ = Z.selective_scan(f64(layer.x[0]), Z.softplus(f64(layer.dt[0]) + f64(layer.bias)), f64(a), f64(layer.bc[0])[:, 0], f64(layer.bc[0])[:, 1], torch.zeros(inner, dtype=torch.float64))
    y = y * Z.silu(f64(layer.z[0]))
    got, _ = feed_scan(layer, [n_tok], [[500, 200] + [1] * 40] if steps else [[n_tok]], [0], 128, steps)
    close(got[0], y, dtype)
    close(got[0][-1], y[-1], dtype, slack=max(y[-1].abs().max().item(), 1e-3))        # (of the last token's own size)
    assert y[-1, :inner // 2].abs().max() > 0.01 and got[0][-1, inner // 2:].abs().max() < 1e-6


# ------------------------------------------------------------------------------------------------ time mixing
class Wkv:
    def __init__(self, lengths, heads, dim, dk, dtype, w0=(-6.0, 0.0), eps=1e-5, rank=16):
        self.heads, self.dim, self.dk, self.dtype, self.eps = heads, dim, dk, dtype, eps
        self.r, self.k, self.v, self.g = ([randn(t, heads, dim, seed=10 * t + s, dtype=dtype) for t in lengths] for s in (1, 2, 3, 4))
        gen = torch.Generator().manual_seed(dim)
        self.low, self.w2 = [randn(t, rank, seed=10 * t + 5, dtype=dtype) for t in lengths], randn(heads * dim, rank, seed=6, scale=0.7 * rank ** -0.5, dtype=dtype)
        self.z = [(torch.tanh(f64(t)) @ f64(self.w2).T).to(dtype).view(-1, heads, dim) for t in self.low]
        self.w0 = torch.rand(heads, dim, generator=gen) * (w0[1] - w0[0]) + w0[0]
        self.u, self.norm = randn(heads, dim, seed=7, dtype=F32), 1 + 0.2 * randn(heads, dim, seed=8, dtype=F32)
        self.want = []
        for r, k, v, g, z in zip(*(map(f64, t) for t in (self.r, self.k, self.v, self.g, self.z))):
            pairs = [Z.wkv_scan(r[:, h], k[:, h], v[:, h], torch.exp(-torch.exp(z[:, h] + f64(self.w0)[h])), f64(self.u)[h]) for h in range(heads)]
            o = torch.stack([p[0] for p in pairs], dim=1)
            self.want.append((Z.rms(o, eps) * f64(self.norm) * Z.silu(g), torch.stack([p[1] for p in pairs])))
        self.params = dict(w2=padded(self.w2.view(heads, dim, rank), heads, dk, rank).reshape(heads * dk, rank).cuda(),
                           **{n: padded(t, heads, dk).reshape(-1).contiguous().cuda() for n, t in (("w0", self.w0), ("u", self.u), ("norm", self.norm))})

    def rows(self, what, batch):
        t = torch.cat([getattr(self, what)[i][a:a + n] for i, a, n, _ in batch])
        return t.cuda() if what == "low" else padded(t, t.shape[0], self.heads, self.dk).reshape(t.shape[0], -1).cuda()

    def run(self, batch, state, segment, step, generic):
        p = Portions([(a, k, s) for _, a, k, s in batch])
        args = [self.rows(w, batch) for w in ("r", "k", "v", "g", "low" if step else "z")]
        if step:
            return ops().wkv_step(*args, self.params, self.eps, self.dim, p.positions, p.slots, state)
        chunks, more = p.chunks(segment)
        return ops().wkv_chunks(*args, self.params, self.eps, self.dim, p.positions, p.slots, chunks, more, state, generic=generic)


def feed_wkv(layer, lengths, cuts, slots, segment=64, steps=False, generic=False):
    state = torch.full((max(slots) + 1, layer.heads, layer.dk, layer.dk), 30.0).cuda()
    got = [[] for _ in lengths]
    for batch in feed_plan(lengths, cuts, slots):
        singles = [e for e in batch if e[2] == 1] if steps else []
        for part in (singles, [e for e in batch if e not in singles]):
            if part:
                out = layer.run(part, state, segment, part is singles, generic).view(-1, layer.heads, layer.dk)
                assert not out[..., layer.dim:].any()
                for (i, *_), rows in zip(part, out[..., :layer.dim].split([k for _, _, k, _ in part])):
                    got[i].append(rows)
    return [torch.cat(g) for g in got], state


WKV_SHAPES = [(3, 64, 64), (2, 128, 128), (2, 40, 64), (1, 100, 128), (5, 8, 64)]
DECAYS = {"usual": (-6.0, 0.0), "slow": (-12.0, -7.0), "strong": (-0.5, 2.5), "some chunks strong": (0.4, 0.9), "gone at once": (4.0, 6.0)}


@pytest.mark.parametrize("decay", sorted(DECAYS))
@pytest.mark.parametrize("heads,dim,dk,dtype,generic", [(*s, BF16, False) for s in WKV_SHAPES] + [(3, 64, 64, BF16, True), (1, 150, 152, BF16, True), (2, 20, 24, F32, True), (3, 64, 64, F32, True)])
def test_wkv_portions(heads, dim, dk, dtype, generic, decay):
    """Decays of every strength (a chunk leaves the matrix form where a channel loses more than 2^100 in half of it), portions and segments of every kind."""
    lengths, cuts, slots = [300, 2, 65, 131], [[150, 1, 2, 3, 64], [1], [65], [2, 129]], [2, 0, 3, 4]
    layer = Wkv(lengths, heads, dim, dk, dtype, DECAYS[decay])
    for segment in (64, 128, 1024):
        got, state = feed_wkv(layer, lengths, cuts, slots, segment, generic=generic)
        for i, (o, s) in enumerate(layer.want):
            close(got[i], o, dtype, f"segment {segment} sequence {i}", slack=2)
            close(state[slots[i], :, :dim, :dim], s, F32, f"state {i}", slack=8 if generic else 64)
            assert not state[slots[i], :, dim:].any() and not state[slots[i], :, :, dim:].any()
        assert (state[1] == 30).all()


@pytest.mark.parametrize("decay", ["usual", "slow", "strong"])
@pytest.mark.parametrize("heads,dim,dk", WKV_SHAPES)
def test_wkv_step(heads, dim, dk, decay):
    lengths, cuts, slots = [90, 9, 70], [[30, 1, 1, 1], [1], [2, 1, 1]], [2, 0, 3]
    layer = Wkv(lengths, heads, dim, dk, BF16, DECAYS[decay])
    got, state = feed_wkv(layer, lengths, cuts, slots, steps=True)
    for i, (o, s) in enumerate(layer.want):
        close(got[i], o, BF16, f"sequence {i}", slack=2)                 # (the portions' decays pass through one more rounding)
        close(state[slots[i], :, :dim, :dim], s, BF16, f"state {i}", slack=2)


def test_wkv_strong_chunks_take_the_other_way():
    """The decays of test_wkv_portions lie on both sides of the matrix form's bound, in one sequence even on both sides from chunk to chunk."""
    def loss(lo_hi):
        layer = Wkv([300], 3, 64, 64, BF16, DECAYS[lo_hi])
        lw = torch.exp(f64(layer.z[0]) + f64(layer.w0)) * 1.4426950408889634
        return [torch.stack([c[:32].sum(0).max(), c[32:].sum(0).max()]).max().item() for c in lw[:256].split(64)]
    assert max(loss("usual")) < 100 < min(loss("strong")) and max(loss("slow")) < 1
    mixed = loss("some chunks strong")
    assert min(loss("gone at once")) > 2000 and 60 < min(mixed) and max(mixed) < 300


def test_wkv_one_token_stands_out():
    """A key far back that the last token asks for wins where the decay is slow; in every form."""
    n, dim = 700, 64
    layer = Wkv([n], 1, dim, dim, BF16, (-14.0, -13.0))
    layer.k[0] *= 0.01
    layer.k[0][3] = 0
    layer.k[0][3, 0, 5] = 100.0
    layer.r[0][-1] = 0
    layer.r[0][-1, 0, 5] = 1.0
    o = Z.wkv_scan(f64(layer.r[0])[:, 0], f64(layer.k[0])[:, 0], f64(layer.v[0])[:, 0], torch.exp(-torch.exp(f64(layer.z[0])[:, 0] + f64(layer.w0)[0])), f64(layer.u)[0])[0]
    assert (Z.rms(o[-1:], 0.0) - Z.rms(f64(layer.v[0])[3], 0.0)).abs().max() < 0.1
    want = Z.rms(o[:, None], layer.eps) * f64(layer.norm) * Z.silu(f64(layer.g[0]))
    for cuts, kw in (([[n]], {}), ([[n]], dict(segment=128)), ([[650, 2, 17]], dict(segment=64)), ([[600] + [1] * 100], dict(steps=True)), ([[n]], dict(generic=True))):
        got, _ = feed_wkv(layer, [n], cuts, [0], **kw)
        close(got[0][-1], want[-1], BF16, str(kw), slack=2)


# ------------------------------------------------------------------------------------------------ attention: chunks, values that turn
def attend_ref(q, k, v, pos, scale, chunk, keep):
    """q [heads, dim] at position pos over k, v [n, kvh, .]"""
    heads, kvh = q.shape[0], k.shape[1]
    j = torch.arange(k.shape[0])
    ok = (j <= pos) & ((j // chunk == pos // chunk) | (j < keep))
    out = []
    for h in range(heads):
        g = h // (heads // kvh)
        p = torch.softmax(((f64(k)[:, g] @ f64(q)[h]) * scale).masked_fill(~ok, float("-inf")), 0)
        out.append(p @ f64(v)[:, g])
    return torch.stack(out)


def turned_back(o, pos, table):
    """Interleaved pairs of o [heads, d] by minus the table's angles."""
    half = table.shape[1] // 2
    c, s = f64(table)[pos, :half], f64(table)[pos, half:]
    o = o.clone()
    x, y = o[:, 0:2 * half:2].clone(), o[:, 1:2 * half:2].clone()
    o[:, 0:2 * half:2], o[:, 1:2 * half:2] = x * c + y * s, y * c - x * s
    return o


def table_of(dims, n=512):
    from nanovllm_hip.layers.rotary import rotation_table
    return rotation_table(dims, 50.0, n, "cuda")


SHAPES = [(8, 2, 64, 64), (3, 3, 40, 100), (20, 2, 128, 128), (6, 2, 96, 30), (2, 2, 256, 256), (9, 1, 128, 60), (2, 1, 270, 300)]


@pytest.mark.parametrize("dtype,generic", [(BF16, False), (BF16, True), (F32, False)])
@pytest.mark.parametrize("heads,kvh,dim,vdim", SHAPES)
def test_rows_in_chunks(heads, kvh, dim, vdim, dtype, generic):
    lengths = [1, 2, 64, 65, 129, 300]
    pg = Pages(lengths, kvh, dim, vdim, dtype)
    cache, tables, table = pg.cache(), pg.tables.cuda(), table_of(vdim)
    q, pos = randn(len(lengths), heads, dim, seed=5, dtype=dtype), torch.tensor([n - 1 for n in lengths])
    for chunk, keep in ((1, 0), (64, 0), (65, 3), (37, 0), (128, 70), (1000, 0)):
        want = torch.stack([attend_ref(q[i], pg.k[i], pg.v[i], n - 1, 0.2, chunk, keep) for i, n in enumerate(lengths)])
        back = torch.stack([turned_back(w, n - 1, table) for w, n in zip(want, lengths)])
        for splits in (None, 1, 3, 5):
            for turn, w in ((None, want), (table, back)):
                got = ops().paged_attend_rows(pg.pad_q(q), cache, tables, pos.cuda(), heads, kvh, pg.dk, pg.dv, 0.2, 300, 0, keep, splits=splits, generic=generic, chunk=chunk, turn=turn)
                close(pg.unpad(got, heads), w, dtype, f"chunk {chunk} keep {keep} splits {splits}")


PORTIONS = [(2, 2), (64, 64), (2, 65), (65, 129), (130, 300), (300, 300), (3, 400), (57, 190)]


@pytest.mark.parametrize("chunk,keep", [(1, 0), (64, 0), (65, 3), (37, 0), (130, 70), (1000, 0)])
@pytest.mark.parametrize("heads,kvh,dim,vdim", [s for s in SHAPES if max(s[2:]) <= 256])
def test_prompt_in_chunks(heads, kvh, dim, vdim, chunk, keep):
    """Portions of several sequences (rows, keys) in one launch; long portions take the two-tile form."""
    table = table_of(vdim)
    for portions in (PORTIONS[:5], PORTIONS[3:]) if dim <= 128 else (PORTIONS[2:6],):
        pg = Pages([k for _, k in portions], kvh, dim, vdim, BF16, seed=3)
        rows = sum(r for r, _ in portions)
        q = randn(rows, heads, dim, seed=8)
        cu_q = torch.tensor([0] + [r for r, _ in portions]).cumsum(0).int().cuda()
        cu_k = torch.tensor([0] + [k for _, k in portions]).cumsum(0).int().cuda()
        got = pg.unpad(ops().paged_attend_prompt(pg.pad_q(q), pg.cache(), pg.tables.cuda(), cu_q, cu_k, max(r for r, _ in portions), heads, kvh, pg.dk, pg.dv, 0.2, 0, keep,
                                                 chunk=chunk, turn=table), heads)
        at = 0
        for i, (r, k) in enumerate(portions):
            borders = {t for t in range(r) if (k - r + t) % chunk in (0, chunk - 1)} if chunk > 30 else set()
            for t in sorted({0, 1, r // 2, r - 2, r - 1, min(63, r - 1), min(64, r - 1)} | borders):
                want = turned_back(attend_ref(q[at + t], pg.k[i], pg.v[i], k - r + t, 0.2, chunk, keep), k - r + t, table)
                close(got[at + t], want, BF16, f"portion {i} row {t}")
            at += r


@pytest.mark.parametrize("chunk", [1, 64, 65, 40, 100, 128])
@pytest.mark.parametrize("portion", [1, 2, 40, 200])
def test_one_key_stands_out_at_chunk_borders(chunk, portion):
    """A key whose score dwarfs the others' takes the output inside its chunk and changes nothing past it: at page borders, at the chunk's first and last place."""
    heads, kvh, dim, vdim, n = 2, 1, 64, 64, 259
    last = (n - 1) // chunk * chunk                                     # first position of the last row's chunk
    places = sorted({a for a in (0, 1, 63, 64, 65, 127, 128, n - 2, n - 1, last - 1, last, last + 1, last - chunk, last - chunk - 1) if 0 <= a < n})
    pg = Pages([n] * len(places), kvh, dim, vdim, BF16)
    q1 = randn(len(places), kvh, dim, seed=7)
    for i, a in enumerate(places):
        pg.k[i] = pg.k[i] * 0.3
        pg.k[i][a] = q1[i] * 2
    q = q1.repeat_interleave(portion, dim=0).repeat_interleave(heads, dim=1)
    args = (heads, kvh, pg.dk, pg.dv, 0.2)
    if portion == 1:
        pos = torch.full((len(places),), n - 1).cuda()
        results = [ops().paged_attend_rows(pg.pad_q(q), pg.cache(), pg.tables.cuda(), pos, *args, n, chunk=chunk, splits=s, generic=g) for s, g in ((1, False), (3, False), (1, True))]
    else:
        cu_q, cu_k = ((torch.arange(len(places) + 1) * t).int().cuda() for t in (portion, n))
        results = [ops().paged_attend_prompt(pg.pad_q(q), pg.cache(), pg.tables.cuda(), cu_q, cu_k, portion, *args, chunk=chunk)]
    for got in results:
        got = pg.unpad(got, heads)
        for i, a in enumerate(places):
            near = {0, 1, portion // 2, portion - 2, portion - 1} | {x - (n - portion) for x in (a - 1, a, a + 1, (a // chunk + 1) * chunk - 1, (a // chunk + 1) * chunk)}
            for t in sorted(x for x in near if 0 <= x < portion):
                p = n - portion + t
                want = attend_ref(q[i * portion + t], pg.k[i], pg.v[i], p, 0.2, chunk, 0)
                close(got[i * portion + t], want, BF16, f"key {a} row {t}", slack=2)
                if p // chunk == a // chunk and a <= p:
                    assert (want[0] - f64(pg.v[i])[a, 0]).abs().max() < 0.05


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("heads,kvh,dim,vdim,rot", [(4, 2, 64, 32, 24), (3, 1, 40, 14, 40), (8, 8, 128, 128, 0), (5, 5, 20, 100, 6)])
def test_prep_with_turned_values(heads, kvh, dim, vdim, rot, dtype):
    from nanovllm_hip.layers.paged_attention import padded_widths
    (dk, dv), rows, bs = padded_widths(dim, vdim), 37, 64
    qkv = torch.cat([padded(randn(rows, n, w, seed=s, dtype=dtype), rows, n, to).reshape(rows, -1) for n, w, to, s in ((heads, dim, dk, 1), (kvh, dim, dk, 2), (kvh, vdim, dv, 3))], dim=1)
    pos = torch.randint(0, 500, (rows,), generator=torch.Generator().manual_seed(1))
    slots = torch.randperm(3 * bs, generator=torch.Generator().manual_seed(2))[:rows].int()
    w = [padded(1 + randn(dim, seed=s, dtype=F32, scale=0.3), dk) for s in (4, 5)]
    table, v_table = table_of(rot) if rot else None, table_of(vdim)
    cache = torch.zeros(3, bs, kvh * (dk + dv), dtype=dtype).cuda()
    before, x = f64(qkv), qkv.cuda()
    ops().attn_prep(x, heads, kvh, dk, dv, pos.cuda(), table, cache, slots.cuda(), w[0].cuda(), w[1].cuda(), dim, dim, 1e-3, head_norm=True, v_cos_sin=v_table)
    flat = f64(cache).view(3, kvh, bs * (dk + dv))

    def turned(t, p, tab):
        return turned_back(t, p, torch.cat([tab[:, :tab.shape[1] // 2], -tab[:, tab.shape[1] // 2:]], dim=1)) if tab is not None else t
    for r in range(rows):
        q, k, v = (t.view(-1, d) for t, d in zip(before[r].split([heads * dk, kvh * dk, kvh * dv]), (dk, dk, dv)))
        nq, nk = (t / torch.sqrt((t * t).sum(-1, keepdim=True) / dim + 1e-3) * f64(g) for t, g in zip((q, k), w))
        close(x[r, :heads * dk].view(heads, dk), turned(nq, pos[r], table), dtype)
        page, off = slots[r].item() // bs, slots[r].item() % bs
        close(flat[page, :, off * dk:(off + 1) * dk], turned(nk, pos[r], table), dtype)
        close(flat[page, :, bs * dk + off * dv:bs * dk + (off + 1) * dv], turned(v, pos[r], v_table), dtype)


# ------------------------------------------------------------------------------------------------ feed-forward, grouped projection
@pytest.mark.parametrize("dtype", [BF16, F32])
def test_gelu_glu(dtype):
    gu = randn(7, 2 * 136, dtype=dtype, scale=3.0)
    close(ops().gelu_glu(gu.cuda()), Z.gelu_tanh(f64(gu)[:, :136]) * f64(gu)[:, 136:], dtype)


@pytest.mark.parametrize("m,k,inter", [(1, 64, 16), (17, 256, 448), (33, 1280, 192), (64, 2048, 6144)])
def test_gelu_epilogue(m, k, inter):
    x, w = randn(m, k), randn(2 * inter, k, seed=1, scale=k ** -0.5)
    ws = torch.zeros(max(16, ops().linear_workspace_bytes(m, 2 * inter, k, "silu_mul")), dtype=torch.uint8, device="cuda")
    a = f64(x) @ f64(w).T
    want = Z.gelu_tanh(a[:, :inter]) * a[:, inter:]
    got = ops().fused_linear(ops().pack_rows(x.cuda()), w.cuda(), x_packed_rows=m, epilogue="silu_mul", glu="gelu", workspace=ws)
    close(got, want, BF16, slack=2)
    close(ops().fused_linear(x.cuda(), w.cuda(), epilogue="silu_mul", glu="gelu", workspace=ws), want, BF16, slack=2)


@pytest.mark.parametrize("m,k,rows,tail", [(1, 64, 64, 16), (19, 192, 384, 64), (32, 2048, 2048, 64), (64, 1280, 128, 192), (5, 128, 16, 16)])
def test_projection_of_several_inputs(m, k, rows, tail):
    """Groups of weight rows, each applied to its own activations; the last group of another size; contractions split over workgroups."""
    xs, w = [randn(m, k, seed=s) for s in range(5)], randn(4 * rows + tail, k, seed=9, scale=k ** -0.5)
    ws = torch.zeros(max(16, ops().linear_workspace_bytes(m, w.shape[0], k)), dtype=torch.uint8, device="cuda")
    packed = torch.cat([ops().pack_rows(x.cuda()) for x in xs])
    want = torch.cat([f64(x) @ f64(p).T for x, p in zip(xs, w.split([rows] * 4 + [tail]))], dim=1)
    for _ in range(2):
        close(ops().fused_linear(packed, w.cuda(), x_packed_rows=m, workspace=ws, x_groups=(5, rows)), want, BF16)


def test_operand_checks():
    """Shapes the kernels do not take are refused on the host."""
    x = torch.zeros(2, 17, 64, device="cuda")
    with pytest.raises(RuntimeError, match="streams"):
        ops().stream_mix(x, 17, BF16, 64)
    with pytest.raises(RuntimeError, match="groups"):
        ops().stream_mix(x[:, 0].contiguous(), 2, F32, 60, None, None, (torch.ones(64, device="cuda"), 7, 1e-5))
    assert [ops().scan_states(n) for n in (1, 8, 9, 256, 257)] == [8, 8, 16, 256, 0] and not ops().wkv_supported(96)
    with pytest.raises(RuntimeError, match="x groups"):
        ops().fused_linear(torch.zeros(5 * 16 * 64, dtype=BF16, device="cuda"), torch.zeros(100, 64, dtype=BF16, device="cuda")[:96], x_packed_rows=1, x_groups=(5, 24))
