"""GPU: the recurrent and latent-attention layer ops, one mechanism at a time, against plain equations on the CPU (oracle/zobasun_ref.py, float64):
bf16 on the MFMA kernels, bf16 and fp32 on the plain ones.  Inputs are given in the compared type, so fp32 results are held to fp32 rounding."""
import pytest
import torch

from oracle import zobasun_ref as Z

pytestmark = pytest.mark.gpu
F64 = torch.float64
TYPES = [torch.bfloat16, torch.float32]


def rnd(*shape, seed=0, scale=1.0, dtype=torch.bfloat16):
    return (torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale).to(dtype)


def close(got, want, dtype, factor=1.0):
    """Largest difference against the scale of the wanted values: a few bf16 roundings, or fp32 ones."""
    got, want = got.detach().to("cpu", F64), want.to(F64)
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-30)
    assert err <= factor * (2.0 ** -7 if dtype == torch.bfloat16 else 3e-6), f"error {err:.3e} of scale"


def pad_cols(t, cols):
    out = t.new_zeros(*t.shape[:-1], cols)
    out[..., :t.shape[-1]] = t
    return out


# ------------------------------------------------------------------------------------------------ row ops
@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("rows,n,cols", [(1, 40, 64), (3, 96, 96), (20, 1000, 1024), (5, 2880, 2880), (2, 5000, 5056)])
def test_norm_residual(dtype, rows, n, cols):
    from nanovllm_hip import ops
    x, y, w = rnd(rows, cols, seed=1, dtype=torch.float32), rnd(rows, n, seed=2, scale=3.0, dtype=dtype), rnd(cols, seed=3, dtype=torch.float32)
    y = pad_cols(y, cols)
    x[:, n:] = 0
    xg = x.cuda()
    packed = torch.zeros((rows + 15) // 16 * 16 * cols, dtype=torch.bfloat16, device="cuda") if dtype == torch.bfloat16 and cols % 32 == 0 else None
    out = ops.norm_residual(xg, w.cuda(), 1e-3, n, dtype, y=y.cuda(), packed=packed)
    want = x.to(F64)
    want[:, :n] += Z.rms_norm(y[:, :n].to(F64), 1e-3) * w[:n].to(F64)
    close(xg, want, torch.float32)
    close(out, want, dtype)
    if packed is not None:
        assert torch.equal(ops.unpack_rows(packed, rows, cols), out)
    before = xg.clone()
    close(ops.norm_residual(xg, w.cuda(), 1e-3, n, dtype)[:, :n], Z.rms_norm(want[:, :n], 1e-3) * w[:n].to(F64), dtype)
    assert torch.equal(xg, before)


@pytest.mark.parametrize("dtype", TYPES)
def test_embed_rows(dtype):
    from nanovllm_hip import ops
    e = rnd(50, 96, dtype=dtype)
    toks = torch.tensor([0, 49, 7, 7, 1])
    x, xb = ops.embed_rows(toks.cuda(), e.cuda(), 5.5)
    want = e[toks].to(F64) * 5.5
    close(x, want, torch.float32)
    close(xb, want, dtype)
    if dtype == torch.bfloat16:
        packed = torch.zeros(16 * 96, dtype=dtype, device="cuda")
        ops.embed_rows(toks.cuda(), e.cuda(), 5.5, packed=packed)
        assert torch.equal(ops.unpack_rows(packed, 5, 96), xb)


@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("limit", [0.5, 1.0, 7.0])
def test_clamped_glu(dtype, limit):
    from nanovllm_hip import ops
    gu = rnd(9, 2 * 72, scale=3.0, dtype=dtype)                              # both sides of every limit
    want = Z.clamped_glu(gu[:, :72].to(F64), gu[:, 72:].to(F64), limit)
    close(ops.clamped_glu(gu.cuda(), limit, 1.702), want, dtype)


@pytest.mark.parametrize("m,k,inter", [(1, 64, 32), (17, 192, 224), (64, 1536, 96), (33, 2048, 8192)])
def test_clamped_glu_epilogue(m, k, inter):
    """The same unit in the gate_up projection's epilogue: row-major and packed, split over K, wide tiles."""
    from nanovllm_hip import ops
    x, w = rnd(m, k, seed=1), rnd(2 * inter, k, seed=2, scale=2.0 * k ** -0.5)
    h = x.to(F64) @ w.to(F64).T
    want = Z.clamped_glu(h[:, :inter].bfloat16().to(F64), h[:, inter:].bfloat16().to(F64), 1.3)
    xg, wg = x.cuda(), w.cuda()
    close(ops.fused_linear(xg, wg, epilogue="silu_mul", glu=(1.3, 1.702)), want, torch.bfloat16, 2)
    ws = torch.zeros(max(16, ops.linear_workspace_bytes(m, 2 * inter, k, "silu_mul")), dtype=torch.uint8, device="cuda")
    packed = torch.zeros((m + 15) // 16 * 16 * inter, dtype=torch.bfloat16, device="cuda")
    out = ops.fused_linear(ops.pack_rows(xg), wg, x_packed_rows=m, epilogue="silu_mul", glu=(1.3, 1.702), out_packed=packed, workspace=ws)
    close(out, want, torch.bfloat16, 2)
    assert torch.equal(ops.unpack_rows(packed, m, inter), out)


def test_rotation_table():
    from nanovllm_hip.layers.rotary import rotation_table
    t = rotation_table(24, 3000.0, 5000, "cuda").cpu().to(F64)
    pos, i = torch.arange(5000, dtype=F64)[:, None], torch.arange(12, dtype=F64)[None]
    ang = pos * 3000.0 ** (-2 * i / 24)
    assert (t[:, :12] - ang.cos()).abs().max() < 1e-7 and (t[:, 12:] - ang.sin()).abs().max() < 1e-7


# ------------------------------------------------------------------------------------------------ recurrence
class Recurrence:
    """Random parameters of one block-diagonal recurrence, its pools, and the plain result."""

    def __init__(self, blocks, size, block, taps, dtype, slots=4, seed=0, lam=None):
        self.blocks, self.size, self.block, self.taps, self.dtype = blocks, size, block, taps, dtype
        self.n, self.cols = blocks * size, blocks * block
        self.conv, self.conv_b = rnd(self.n, taps, seed=seed + 1, dtype=dtype), rnd(self.n, seed=seed + 2, scale=0.3, dtype=dtype)
        self.ra, self.ri = [rnd(blocks, size, size, seed=seed + s, scale=size ** -0.5, dtype=dtype) for s in (3, 4)]
        self.ra_b, self.ri_b = [rnd(blocks, size, seed=seed + s, scale=0.5, dtype=dtype) for s in (5, 6)]
        self.lam = lam if lam is not None else torch.rand(self.n, generator=torch.Generator().manual_seed(seed + 7)) * 8 - 7
        rate = 8.0 * torch.nn.functional.softplus(self.lam.to(F64))
        f32 = dict(conv_w=self.conv.float().t(), conv_b=self.conv_b.float()[None], ra_b=self.ra_b.float().reshape(1, -1), ri_b=self.ri_b.float().reshape(1, -1),
                   rate=rate.float()[None])
        self.params = {k: self.spread(v).contiguous().cuda() for k, v in f32.items()}
        for k in ("conv_b", "ra_b", "ri_b", "rate"):
            self.params[k] = self.params[k].reshape(-1)
        for k, v in (("ra", self.ra), ("ri", self.ri)):
            self.params[k] = pad_cols(pad_cols(v, block).transpose(1, 2), block).transpose(1, 2).contiguous().cuda()
        # pools full of garbage: nothing of an earlier owner may reach a new sequence
        self.state = torch.full((slots, self.cols), 1e6, device="cuda")
        self.conv_state = torch.full((slots, taps, self.cols), 1e4, dtype=dtype, device="cuda")

    def spread(self, t):
        """[rows, blocks * size] -> padded channels."""
        return pad_cols(t.reshape(t.shape[0], self.blocks, self.size), self.block).reshape(t.shape[0], self.cols)

    def unspread(self, t):
        return t.reshape(t.shape[0], self.blocks, self.block)[:, :, :self.size].reshape(t.shape[0], self.n)

    def yx(self, rows, seed):
        y, x = rnd(rows, self.n, seed=100 + seed, dtype=self.dtype), rnd(rows, self.n, seed=200 + seed, dtype=self.dtype)
        return y, x

    def rows(self, y, x):
        return torch.cat([self.spread(y), self.spread(x)], 1).cuda()

    def plain(self, y, x):
        d = lambda t: t.to(F64)
        u = Z.causal_conv(d(x), d(self.conv), d(self.conv_b))
        if self.dtype == torch.bfloat16:
            u = u.bfloat16().to(F64)                                          # the one rounding in front of the recurrence
        r, i = Z.block_gate(u, d(self.ra), d(self.ra_b)), Z.block_gate(u, d(self.ri), d(self.ri_b))
        s, last = Z.rglru_recurrence(u, r, i, d(self.lam))
        return s * Z.gelu_tanh(d(y)), last

    def run(self, portions, generic=False, step=False, segment=64):
        """portions: [(slot, first position, y, x)] as one batch; returns the unpadded rows per portion."""
        from nanovllm_hip import ops
        from nanovllm_hip.engine.model_runner import recurrence_chunks
        yx = torch.cat([self.rows(y, x) for _, _, y, x in portions])
        pos = torch.cat([torch.arange(p, p + y.shape[0]) for _, p, y, _ in portions]).cuda()
        slots = torch.tensor([s for s, *_ in portions], dtype=torch.int32, device="cuda")
        if step:
            packed = torch.zeros((len(portions) + 15) // 16 * 16 * self.cols, dtype=torch.bfloat16, device="cuda")
            out = ops.rglru_step(yx, self.params, pos, slots, self.state, self.conv_state, out_packed=packed)
            assert torch.equal(ops.unpack_rows(packed, len(portions), self.cols), out)
        else:
            table, row = [], 0
            for j, (_, _, y, _) in enumerate(portions):
                table += recurrence_chunks(row, y.shape[0], j, segment)
                row += y.shape[0]
            out = ops.rglru_chunks(yx, self.params, pos, slots, torch.tensor(table, dtype=torch.int32, device="cuda"), segment, any(k for *_, k in table),
                                   self.state, self.conv_state, generic=generic)
        out = self.unspread(out.cpu())
        return out.split([y.shape[0] for _, _, y, _ in portions])


SHAPES = [(1, 32, 64, 1), (3, 44, 64, 4), (2, 96, 96, 2), (4, 256, 256, 4), (1, 640, 640, 5), (5, 13, 64, 7), (2, 160, 160, 9), (2, 224, 224, 12)]
FORMS = [(torch.bfloat16, False), (torch.bfloat16, True), (torch.float32, False)]
WALKS = [(torch.bfloat16, 0), (torch.bfloat16, 1), (torch.bfloat16, 2), (torch.float32, 0)]      # fastest, plain, MFMA without LDS-DMA


@pytest.mark.parametrize("segment", [64, 128, 4096])
@pytest.mark.parametrize("dtype,generic", WALKS)
@pytest.mark.parametrize("blocks,size,block,taps", SHAPES)
def test_recurrence_portions(blocks, size, block, taps, dtype, generic, segment):
    """Two unequal sequences in one batch, then their later portions (down to two tokens, across chunk edges) from the state."""
    r = Recurrence(blocks, size, block, taps, dtype)
    (ya, xa), (yb, xb) = r.yx(341, 1), r.yx(77, 2)
    (wa, la), (wb, lb) = r.plain(ya, xa), r.plain(yb, xb)
    cuts_a, cuts_b = [0, 193, 195, 196, 330, 341], [0, 2, 66, 68, 75, 77]
    for (a0, a1), (b0, b1) in zip(zip(cuts_a, cuts_a[1:]), zip(cuts_b, cuts_b[1:])):
        ga, gb = r.run([(2, a0, ya[a0:a1], xa[a0:a1]), (0, b0, yb[b0:b1], xb[b0:b1])], generic, segment=segment)
        close(ga, wa[a0:a1], dtype)
        close(gb, wb[b0:b1], dtype)
    close(r.unspread(r.state[[2, 0]].cpu()), torch.stack([la, lb]), torch.float32, 40 if dtype == torch.bfloat16 else 3)


@pytest.mark.parametrize("blocks,size,block,taps", SHAPES)
def test_recurrence_step_follows_portions(blocks, size, block, taps):
    """Prompt by the chunked form, then single tokens by the step form (one sequence steps from its very first token)."""
    r = Recurrence(blocks, size, block, taps, torch.bfloat16, slots=40)
    y, x = r.yx(90, 1)
    want, last = r.plain(y, x)
    close(r.run([(3, 0, y[:71], x[:71])])[0], want[:71], torch.bfloat16)
    others = [r.yx(19, 10 + k) for k in range(34)]                             # 35 rows: more than one row tile
    wants = [r.plain(*o)[0] for o in others]
    for t in range(19):
        got = r.run([(3, 71 + t, y[71 + t:72 + t], x[71 + t:72 + t])] + [(5 + k, t, o[0][t:t + 1], o[1][t:t + 1]) for k, o in enumerate(others)], step=True)
        close(got[0], want[71 + t:72 + t], torch.bfloat16)
        close(torch.cat(got[1:]), torch.stack([w[t] for w in wants]), torch.bfloat16)
    close(r.unspread(r.state[3:4].cpu()), last[None], torch.float32, 40)


@pytest.mark.parametrize("dtype,generic", WALKS)
def test_recurrence_remembers_for_long(dtype, generic):
    """Decays within 1e-4 of one: one large input at the start still dominates after 600 tokens and several portions."""
    r = Recurrence(2, 64, 64, 3, dtype, lam=torch.full((128,), -11.0))
    y, x = r.yx(640, 1)
    x = x * 0.05
    x[3] = 40.0
    want, _ = r.plain(y, x)
    zeroed = x.clone()
    zeroed[3] = 0
    assert (want[600:] - r.plain(y, zeroed)[0][600:]).abs().max() > 0.5 * want[600:].abs().max()
    got = torch.cat([r.run([(1, a, y[a:b], x[a:b])], generic, segment=128)[0] for a, b in ((0, 300), (300, 302), (302, 640))])
    close(got, want, dtype, 3)


@pytest.mark.parametrize("dtype", TYPES)
def test_recurrence_skips_negative_slots_and_reuses_slots(dtype):
    r = Recurrence(2, 32, 32, 4, dtype)
    y, x = r.yx(9, 1)
    want, _ = r.plain(y, x)
    before = r.state.clone(), r.conv_state.clone()
    close(r.run([(-1, 0, y, x)])[0], want, dtype)
    assert torch.equal(r.state, before[0]) and torch.equal(r.conv_state, before[1])
    r.run([(1, 0, *r.yx(70, 5))])
    close(r.run([(1, 0, y[:3], x[:3])])[0], want[:3], dtype)                    # the slot's next owner starts from zero
    close(r.run([(1, 3, y[3:], x[3:])])[0], want[3:], dtype)


# ------------------------------------------------------------------------------------------------ latent attention
class Latent:
    """One latent-attention geometry with a paged cache whose pages are dealt in a shuffled order and start as garbage."""

    def __init__(self, heads, dim, dim_cols, rot, vdim, v_cols, kv, kv_cols, rot_cols, dtype, page=64, pages=40, scale=None, seed=0):
        self.__dict__.update(heads=heads, dim=dim, dim_cols=dim_cols, rot=rot, vdim=vdim, v_cols=v_cols, kv=kv, kv_cols=kv_cols, rot_cols=rot_cols, dtype=dtype, page=page)
        self.scale = scale or (dim + rot) ** -0.5
        self.uk, self.uv = rnd(heads, dim, kv, seed=seed + 1, scale=kv ** -0.5, dtype=dtype), rnd(heads, vdim, kv, seed=seed + 2, scale=kv ** -0.5, dtype=dtype)
        self.dk = (dim_cols + rot + 63) // 64 * 64
        w_uk = torch.zeros(heads, kv_cols, dim_cols, dtype=dtype)
        w_uk[:, :kv, :dim] = self.uk.transpose(1, 2)
        w_uv = torch.zeros(heads, v_cols, kv_cols, dtype=dtype)
        w_uv[:, :vdim, :kv] = self.uv
        self.w_uk, self.w_uv = w_uk.cuda(), w_uv.cuda()
        from nanovllm_hip.layers.rotary import rotation_table
        self.table = rotation_table(rot, 700.0, 4096, "cuda")
        self.cache = torch.full((pages, page, kv_cols + rot_cols), 77.0, dtype=dtype, device="cuda")
        self.free = torch.randperm(pages, generator=torch.Generator().manual_seed(seed)).tolist()

    def context(self, n, seed):
        """A sequence of n cached tokens: (latents [n, kv], rotated parts [n, rot] in the compared type, page list)."""
        c, k = rnd(n, self.kv, seed=seed, dtype=self.dtype), rnd(n, self.rot, seed=seed + 1, dtype=self.dtype)
        return c, k, [self.free.pop() for _ in range((n + self.page - 1) // self.page)]

    def store(self, ctx):
        c, k, pages = ctx
        rows = torch.cat([pad_cols(c, self.kv_cols), pad_cols(k, self.rot_cols)], 1).cuda()
        for j in range(0, rows.shape[0], self.page):
            n = min(self.page, rows.shape[0] - j)
            self.cache[pages[j // self.page], :n] = rows[j:j + n]

    def queries(self, n, seed):
        return rnd(n, self.heads, self.dim + self.rot, seed=seed, dtype=self.dtype)

    def q_rows(self, q):
        full = torch.zeros(q.shape[0], self.heads, self.dk, dtype=self.dtype)
        full[:, :, :self.dim], full[:, :, self.dim_cols:self.dim_cols + self.rot] = q[:, :, :self.dim], q[:, :, self.dim:]
        return full.reshape(q.shape[0], -1).cuda()

    def plain(self, q, positions, ctx):
        """Attention of q rows at `positions` over the context, in expanded form."""
        c, k_rot = ctx[0].to(F64), ctx[1].to(F64)
        out = []
        for h in range(self.heads):
            q_rot = Z.rotate_pairs(q[:, h, self.dim:].to(F64), positions, self.rot, 700.0)
            s = (q[:, h, :self.dim].to(F64) @ (c @ self.uk[h].to(F64).T).T + q_rot @ k_rot.T) * self.scale
            s = s.masked_fill(torch.arange(c.shape[0])[None] > positions[:, None], float("-inf"))
            out.append(torch.softmax(s, -1) @ (c @ self.uv[h].to(F64).T))
        return torch.stack(out, 1)

    def tables(self, ctxs):
        w = max(len(c[2]) for c in ctxs)
        return torch.tensor([c[2] + [0] * (w - len(c[2])) for c in ctxs], dtype=torch.int32, device="cuda")

    def attend(self, q, positions, ctxs, row_seq=None, **kw):
        from nanovllm_hip import ops
        rs = None if row_seq is None else torch.tensor(row_seq, dtype=torch.int32, device="cuda")
        out = ops.latent_attention(self.q_rows(q), self.cache, self.tables(ctxs), positions.cuda(), self.table, self.w_uk, self.w_uv, self.scale, self.rot,
                                   int(positions.max()) + 1, row_seq=rs, **kw)
        return out.cpu().view(q.shape[0], self.heads, self.v_cols)[:, :, :self.vdim]


#            heads dim dim_cols rot vdim v_cols kv kv_cols rot_cols
LAT = {"one": (1, 8, 32, 8, 16, 64, 20, 64, 64), "small": (7, 32, 32, 24, 40, 64, 56, 64, 64), "many": (20, 64, 64, 64, 128, 128, 250, 256, 64),
       "big": (16, 128, 128, 64, 128, 128, 512, 512, 64), "three": (3, 40, 64, 24, 50, 64, 129, 192, 64), "heads40": (40, 32, 32, 16, 64, 64, 384, 384, 64), "wide": (2, 70, 96, 90, 130, 192, 600, 640, 128)}


@pytest.mark.parametrize("dtype,generic", FORMS)
@pytest.mark.parametrize("name", sorted(LAT))
def test_latent_rows(name, dtype, generic):
    """Single queries at every kind of place: first token, page borders, one past them, long contexts; unequal contexts in one batch."""
    L = Latent(*LAT[name], dtype)
    lens = [1, 2, 63, 64, 65, 128, 129, 300, 500]
    ctxs = [L.context(n, 10 + n) for n in lens]
    for c in ctxs:
        L.store(c)
    q, pos = L.queries(len(lens), 5), torch.tensor(lens) - 1
    want = torch.cat([L.plain(q[i:i + 1], pos[i:i + 1], c) for i, c in enumerate(ctxs)])
    for splits in (None, 1, 3):
        close(L.attend(q, pos, ctxs, splits=splits, generic=generic), want, dtype, 2 if dtype == torch.bfloat16 else 1)
    got = [L.attend(q[i:i + 1], pos[i:i + 1], ctxs[i:i + 1], generic=generic) for i in range(len(lens))]
    close(torch.cat(got), want, dtype, 2 if dtype == torch.bfloat16 else 1)


@pytest.mark.parametrize("dtype,generic", FORMS)
def test_latent_one_key_stands_out(dtype, generic):
    """One key is scaled to win the softmax wherever it sits: the result is that key's value alone — and not seen one position earlier."""
    L = Latent(*LAT["small"], dtype)
    n = 330
    c, k, pages = L.context(n, 50)
    q = L.queries(1, 6)
    # a latent whose expanded key points along head 0's query
    target = q[0, 0, :32].float() @ L.uk[0].float()
    for at in (0, 1, 63, 64, 65, 127, 128, 191, 256, 319, 320, 328, 329):
        cc = c.clone()
        cc[at] = (target * 60.0 / target.norm()).to(dtype)
        ctx = (cc, k, pages)
        L.store(ctx)
        value = cc[at].to(F64) @ L.uv[0].to(F64).T
        got = L.attend(q, torch.tensor([n - 1]), [ctx], generic=generic)
        close(got, L.plain(q, torch.tensor([n - 1]), ctx), dtype, 2)
        close(got[0, 0], value, dtype, 2)
        if at:
            before = L.attend(q, torch.tensor([at - 1]), [ctx], generic=generic)
            close(before, L.plain(q, torch.tensor([at - 1]), ctx), dtype, 2)
            assert (before[0, 0].to(F64) - value).abs().max() > 0.3 * value.abs().max()


@pytest.mark.parametrize("dtype", TYPES)
def test_latent_rows_of_portions(dtype):
    """The plain kernel on rows of several portions (row_seq): the form fp32 models and unusual widths use for prompts."""
    L = Latent(*LAT["wide"], dtype)
    ctxs = [L.context(n, 20 + n) for n in (70, 131)]
    for c in ctxs:
        L.store(c)
    pos = torch.cat([torch.arange(60, 70), torch.arange(0, 131)])
    seq = [0] * 10 + [1] * 131
    q = L.queries(141, 8)
    want = torch.cat([L.plain(q[:10], pos[:10], ctxs[0]), L.plain(q[10:], pos[10:], ctxs[1])])
    close(L.attend(q, pos, ctxs, row_seq=seq), want, dtype, 2 if dtype == torch.bfloat16 else 1)


@pytest.mark.parametrize("name", ["one", "small", "many", "big", "three"])
@pytest.mark.parametrize("portions", [[(0, 1), (0, 2), (0, 64)], [(0, 65), (63, 65), (64, 66), (100, 300)], [(0, 300), (37, 341)], [(511, 513)]])
def test_latent_prefill(name, portions):
    """Prompt portions in expanded form from gathered pages: whole prompts, two-token portions at page borders, a prefix from earlier steps."""
    from nanovllm_hip import ops
    L = Latent(*LAT[name], torch.bfloat16)
    ctxs = [L.context(hi, 30 + hi) for _, hi in portions]
    for c in ctxs:
        L.store(c)
    cu_q = torch.tensor([0] + [hi - lo for lo, hi in portions], dtype=torch.int32).cumsum(0).int().cuda()
    cu_k = torch.tensor([0] + [hi for _, hi in portions], dtype=torch.int32).cumsum(0).int().cuda()
    pos = torch.cat([torch.arange(lo, hi) for lo, hi in portions])
    q = L.queries(pos.numel(), 9)
    q[-1, 0] *= 3                                                             # one sharp row
    rows = ops.latent_gather(L.cache, cu_k, int(cu_k[-1]), L.tables(ctxs))
    assert torch.equal(rows.cpu(), torch.cat([torch.cat([pad_cols(c, L.kv_cols), pad_cols(k, L.rot_cols)], 1) for c, k, _ in ctxs]))
    k = torch.zeros(rows.shape[0], L.heads, L.dim_cols, dtype=torch.bfloat16)
    v = torch.zeros(rows.shape[0], L.heads, L.v_cols, dtype=torch.bfloat16)
    c_all = torch.cat([c for c, _, _ in ctxs]).float()
    for h in range(L.heads):
        k[:, h, :L.dim], v[:, h, :L.vdim] = c_all @ L.uk[h].float().T, c_all @ L.uv[h].float().T
    out = ops.latent_prefill(L.q_rows(q).view(-1, L.heads, L.dk), k.cuda(), rows[:, L.kv_cols:], v.cuda(), cu_q, cu_k, max(hi - lo for lo, hi in portions),
                             pos.cuda(), L.table, L.scale).cpu().view(-1, L.heads, L.v_cols)[:, :, :L.vdim]
    row = 0
    for (lo, hi), ctx in zip(portions, ctxs):
        close(out[row:row + hi - lo], L.plain(q[row:row + hi - lo], torch.arange(lo, hi), ctx), torch.bfloat16, 2)
        row += hi - lo


@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("shared", [False, True])
def test_latent_prep(dtype, shared):
    """Norms over the true ranks, rotation at the row's position, store at its slot; rows without a slot are not stored; a layer on another's
    cache stores nothing."""
    from nanovllm_hip import ops
    from nanovllm_hip.layers.rotary import rotation_table
    rows, qr, qc, kr, kc, rot, rc = 70, 50, 64, 40, 64, 20, 64
    a = torch.zeros(rows, qc + (0 if shared else kc + rc), dtype=dtype)
    a[:, :qr] = rnd(rows, qr, seed=1, scale=2.0, dtype=dtype)
    qw = pad_cols(rnd(qr, seed=4, dtype=torch.float32), qc)
    pos = torch.randperm(900, generator=torch.Generator().manual_seed(3))[:rows]
    pos[0] = 0
    table = rotation_table(rot, 50.0, 1000, "cuda")
    want_q = Z.rms_norm(a[:, :qr].to(F64), 1e-4) * qw[:qr].to(F64)
    if shared:
        close(ops.latent_prep(a.cuda(), qr, qw.cuda(), 1e-4, pos.cuda(), table)[:, :qr], want_q, dtype)
        return
    a[:, qc:qc + kr], a[:, qc + kc:qc + kc + rot] = rnd(rows, kr, seed=2, dtype=dtype), rnd(rows, rot, seed=5, dtype=dtype)
    kw = pad_cols(rnd(kr, seed=6, dtype=torch.float32), kc)
    cache = torch.zeros(3, 64, kc + rc, dtype=dtype, device="cuda")
    slots = torch.randperm(192, generator=torch.Generator().manual_seed(4))[:rows].int()
    slots[5] = -1
    cq = ops.latent_prep(a.cuda(), qr, qw.cuda(), 1e-4, pos.cuda(), table, kv_rank=kr, kv_weight=kw.cuda(), cache=cache, slots=slots.cuda())
    close(cq[:, :qr], want_q, dtype)
    want = torch.zeros(192, kc + rc, dtype=F64)
    for r in range(rows):
        if slots[r] >= 0:
            want[slots[r], :kr] = Z.rms_norm(a[r, qc:qc + kr].to(F64), 1e-4) * kw[:kr].to(F64)
            want[slots[r], kc:kc + rot] = Z.rotate_pairs(a[r:r + 1, qc + kc:qc + kc + rot].to(F64), pos[r:r + 1], rot, 50.0)[0]
    close(cache.view(192, -1), want, dtype)
    if dtype == torch.bfloat16:
        packed = torch.zeros(80 * qc, dtype=dtype, device="cuda")
        ops.latent_prep(a.cuda(), qr, qw.cuda(), 1e-4, pos.cuda(), table, cq_packed=packed)
        assert torch.equal(ops.unpack_rows(packed, rows, qc), cq)


def test_operand_checks():
    """Wrong types and CPU tensors are refused by the wrappers, wrong sizes by the library."""
    from nanovllm_hip import ops
    with pytest.raises(RuntimeError, match="no CPU path"):
        ops.clamped_glu(torch.zeros(2, 16), 1.0, 1.0)
    with pytest.raises(TypeError):
        ops.clamped_glu(torch.zeros(2, 16, device="cuda", dtype=torch.float16), 1.0, 1.0)
    with pytest.raises(RuntimeError, match="inter"):
        ops.clamped_glu(torch.zeros(2, 6, device="cuda"), 1.0, 1.0)
    assert ops.latent_splits(32, 16, 1536, True) == 8
