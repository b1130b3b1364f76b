"""What tests of attention over pages share: random sequences in scattered pages, and comparisons of rounded results with float64 ones."""
import torch

BF16, F32 = torch.bfloat16, torch.float32


def randn(*shape, seed=0, scale=1.0, dtype=BF16):
    return (torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale).to(dtype)


def f64(t):
    return t.double().cpu()


def close(got, want, dtype, what="", slack=1.0):
    err = (f64(got) - want).abs().max().item()
    tol = (2e-5 if dtype == F32 else 2.0 ** -7) * max(1.0, want.abs().max().item()) * slack
    assert err <= tol, f"{what}: {err:.3e} > {tol:.3e}"


class Pages:
    """Random keys and values of several sequences in scattered pages; unused rows hold large garbage."""

    def __init__(self, lengths, kvh, dim, vdim, dtype, bs=64, seed=0):
        from nanovllm_hip.layers.paged_attention import padded_widths
        self.kvh, self.dim, self.vdim, self.dtype, self.bs, self.lengths = kvh, dim, vdim, dtype, bs, lengths
        self.dk, self.dv = padded_widths(dim, vdim)
        counts = [-(-n // bs) for n in lengths]
        order = torch.randperm(sum(counts) + 1, generator=torch.Generator().manual_seed(seed)).tolist()
        self.tables, at = torch.zeros(len(lengths), max(counts), dtype=torch.int32), 0
        for i, c in enumerate(counts):
            self.tables[i, :c] = torch.tensor(order[at:at + c])
            at += c
        self.k = [randn(n, kvh, dim, seed=seed + 10 * i + 1, dtype=dtype) for i, n in enumerate(lengths)]
        self.v = [randn(n, kvh, vdim, seed=seed + 10 * i + 2, dtype=dtype) for i, n in enumerate(lengths)]
        self.pages = len(order)

    def cache(self):
        raw = torch.full((self.pages, self.kvh, self.bs * (self.dk + self.dv)), 300.0, dtype=self.dtype)
        keys = raw[:, :, :self.bs * self.dk].view(self.pages, self.kvh, self.bs, self.dk)
        vals = raw[:, :, self.bs * self.dk:].view(self.pages, self.kvh, self.bs, self.dv)
        for i, n in enumerate(self.lengths):
            for t in range(n):
                p, o = self.tables[i, t // self.bs], t % self.bs
                keys[p, :, o] = 0
                vals[p, :, o] = 0
                keys[p, :, o, :self.dim], vals[p, :, o, :self.vdim] = self.k[i][t], self.v[i][t]
        return raw.view(self.pages, self.bs, self.kvh * (self.dk + self.dv)).cuda()

    def pad_q(self, q):
        out = torch.zeros(q.shape[0], q.shape[1], self.dk, dtype=q.dtype)
        out[:, :, :self.dim] = q
        return out.reshape(q.shape[0], -1).cuda()

    def unpad(self, o, heads):
        return f64(o).view(o.shape[0], heads, self.dv)[:, :, :self.vdim]


def standout_places(pos, window, keep):
    at = {0, 1, keep - 1, keep, keep + 1, 63, 64, 65, 127, 128, pos - 64, pos - 1, pos}
    if window:
        at |= {pos - window - 1, pos - window, pos - window + 1, pos - window + 2}
    return sorted(a for a in at if 0 <= a <= pos)
