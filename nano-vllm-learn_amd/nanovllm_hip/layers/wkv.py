"""Time mixing (RWKV style): heads with a matrix state whose rows decay by a factor per token and channel, w = exp(-exp(w2 tanh(w1 x) + w0)),
o = (S + diag(u) k v^T)^T r, S = diag(w) S + k v^T; every head's output is RMS-normed, scaled, gated by silu and projected.  Its five inputs are mixes of every token
with the one before (layers/streams.py TokenShift, in the order of MIXES).  The state is fp32, one per sequence and head (`state` [slots, heads, dim, dim], bound by
the runner).

Padded widths (zeros): heads to 64 / 128; wider ones run on the plain kernel.
"""
import torch
from torch import nn

from .. import ops
from .linear import linear, padded, round_up

MIXES = ("r", "k", "v", "g", "w")


class TimeMixing(nn.Module):
    mixes = MIXES
    segment_units = property(lambda self: self.heads)        # workgroups that walk one segment

    def __init__(self, in_width, in_cols, heads, dim, eps, dtype):
        super().__init__()
        self.in_width, self.in_cols, self.heads, self.dim, self.eps, self.dtype = in_width, in_cols, heads, dim, eps, dtype
        self.dk = next((w for w in (64, 128) if w >= dim), round_up(dim, 8))
        self.head_cols = heads * self.dk
        self.cols = round_up(self.head_cols, 64)
        self.state = torch.tensor([])
        self.step_ok = dtype == torch.bfloat16 and ops.wkv_supported(self.dk)

    def state_spec(self):
        """Per slot: name -> (shape, dtype) of what a sequence keeps between steps."""
        return {"state": ((self.heads, self.dk, self.dk), torch.float32)}

    def load(self, get):
        def head_rows(t):                            # [heads * dim, ...] -> [cols, ...]
            t = padded(t.reshape(self.heads, self.dim, -1), self.heads, self.dk, t.numel() // (self.heads * self.dim)).reshape(self.head_cols, -1)
            return padded(t, self.cols, t.shape[1])

        def vec(t):
            return head_rows(t.float())[:self.head_cols].reshape(-1).contiguous()
        self.rank = get("w1").shape[0]
        self.rank_cols = round_up(self.rank, 64)
        assert get("k").shape == (self.heads * self.dim, self.in_width) and get("w2").shape == (self.heads * self.dim, self.rank)
        reg = self.register_buffer
        w = [padded(head_rows(get(n)), self.cols, self.in_cols) for n in "rkvg"] + [padded(get("w1"), self.rank_cols, self.in_cols)]
        reg("w_in", torch.cat(w).to(self.dtype).contiguous())
        reg("w2", padded(head_rows(get("w2")), self.cols, self.rank_cols).to(self.dtype).contiguous())
        reg("w0", vec(get("w0")))
        reg("u", vec(get("u")))
        reg("norm", vec(get("norm")))
        reg("w_o", padded(head_rows(get("o").t()).t(), self.in_cols, self.cols).to(self.dtype).contiguous())

    @property
    def params(self):
        return dict(w0=self.w0, u=self.u, norm=self.norm, w2=self.w2)

    def forward(self, x, positions, step):
        """x [5, rows, in_cols] in the activation type -> the mixer's output [rows, in_cols]."""
        c, rows = self.cols, x.shape[1]
        r, k, v, g = (linear(x[i], self.w_in[i * c:(i + 1) * c]) for i in range(4))
        low = linear(x[4], self.w_in[4 * c:])
        n = step.num_decode if self.step_ok else 0                   # these rows take the one-launch step, the rest the chunked walk
        out = (torch.empty if c == self.head_cols else torch.zeros)((rows, c), dtype=x.dtype, device=x.device)
        o = out[:, :self.head_cols]
        if n:
            ops.wkv_step(r[:n], k[:n], v[:n], g[:n], low[:n], self.params, self.eps, self.dim, positions[:n], step.state_slots, self.state, out=o[:n])
        if n < rows:
            z = linear(ops.softcap_(low, 1.0), self.w2)
            ops.wkv_chunks(r, k, v, g, z, self.params, self.eps, self.dim, positions, step.state_slots, step.chunks[n:], step.summaries, self.state, out=o)
        return linear(out, self.w_o)

    def decode(self, xp, rows, positions, step, bufs):
        """Fused decode: five fragment-packed buffers in, output rows out (three launches)."""
        c = self.cols
        a = ops.fused_linear(xp, self.w_in, x_packed_rows=rows, workspace=bufs.workspace, x_groups=(5, c))
        mid = bufs.packed(c)
        ops.wkv_step(*(a[:, i * c:(i + 1) * c] for i in range(4)), a[:, 4 * c:], self.params, self.eps, self.dim, positions, step.state_slots, self.state, out_packed=mid,
                     want_out=False)
        return ops.fused_linear(mid, self.w_o, x_packed_rows=rows, workspace=bufs.workspace)

    def linears(self):
        return [(self.w_in, "none"), (self.w_o, "none")]
