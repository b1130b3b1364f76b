"""Lightning attention: heads with a matrix state and a constant decay each, S = decay S + k v^T, o = S^T q on SiLU-activated projections; the heads' outputs
are RMS-normed together, gated by a sigmoid and projected.  The state is fp32, one per sequence, head and pass over the layer (`state`
[passes, slots, heads, dk, dv], bound by the runner).

Padded widths (zeros): keys to 64 / 128 / 256, values to 64; wider keys run on the plain kernel.
"""
import torch
from torch import nn

from .. import ops
from .linear import linear, padded, round_up


class LightningAttention(nn.Module):
    segment_units = property(lambda self: self.heads * max(1, self.dv // 64))     # workgroups that walk one segment

    def __init__(self, in_width, in_cols, heads, dim, vdim, decay, eps, dtype, passes=1):
        super().__init__()
        assert len(decay) == heads, f"{len(decay)} decays for {heads} heads"
        self.in_width, self.in_cols, self.dtype, self.eps, self.passes = in_width, in_cols, dtype, eps, passes
        self.heads, self.dim, self.vdim, self.decay_values = heads, dim, vdim, [float(d) for d in decay]
        self.dk = next((w for w in (64, 128, 256) if w >= dim), round_up(dim, 8))
        self.dv = round_up(vdim, 64)
        self.cols = heads * self.dv
        self.qkv_cols = heads * (2 * self.dk + self.dv)
        self.state = torch.tensor([])
        self.fast = self.step_ok = dtype == torch.bfloat16 and ops.lightning_supported(self.dk, self.dv)

    def state_spec(self):
        """Per slot: name -> (shape, dtype) of what a sequence keeps between steps."""
        return {"state": ((self.heads, self.dk, self.dv), torch.float32)}

    def load(self, get):
        def heads_to(t, width, to):
            t = t.reshape(self.heads, width, -1)
            return padded(t, self.heads, to, t.shape[2]).reshape(self.heads * to, -1)
        assert get("q").shape == (self.heads * self.dim, self.in_width) and get("v").shape == (self.heads * self.vdim, self.in_width)
        rows = [heads_to(get(n), w, to) for n, w, to in (("q", self.dim, self.dk), ("k", self.dim, self.dk), ("v", self.vdim, self.dv), ("g", self.vdim, self.dv))]
        reg = self.register_buffer
        reg("w_in", padded(torch.cat(rows), self.qkv_cols + self.cols, self.in_cols).to(self.dtype).contiguous())
        reg("norm", heads_to(get("norm").float(), self.vdim, self.dv).reshape(-1).contiguous())
        reg("w_o", padded(heads_to(get("o").t(), self.vdim, self.dv).t(), self.in_cols, self.cols).to(self.dtype).contiguous())
        reg("decay", torch.tensor(self.decay_values, dtype=torch.float32))

    def _gate(self, o, a, **kw):
        return ops.norm_gate(o, a[:, self.qkv_cols:], self.norm, self.eps, self.heads * self.vdim, **kw)

    def forward(self, x, positions, step, run=0):
        """x [rows, in_cols] in the activation type -> the mixer's output, same shape; run: which pass over the layer this is."""
        a = linear(x, self.w_in)
        n = step.num_decode if self.step_ok else 0                   # these rows take the one-launch step, the rest the chunked walk
        o = torch.empty((x.shape[0], self.cols), dtype=x.dtype, device=x.device)
        if n:
            ops.lightning_step(a[:n], self.decay, positions[:n], step.state_slots, self.state[run], out=o[:n])
        if n < x.shape[0]:
            ops.lightning_chunks(a, self.decay, positions, step.state_slots, step.chunks[n:], step.summaries, self.state[run], out=o)
        return linear(self._gate(o, a), self.w_o)

    def decode(self, xp, rows, positions, step, bufs, run=0):
        """Fused decode: fragment-packed rows in, output rows out (four launches)."""
        a = ops.fused_linear(xp, self.w_in, x_packed_rows=rows, workspace=bufs.workspace)
        o = ops.lightning_step(a, self.decay, positions, step.state_slots, self.state[run])
        mid = bufs.packed(self.cols)
        self._gate(o, a, packed=mid)
        return ops.fused_linear(mid, self.w_o, x_packed_rows=rows, workspace=bufs.workspace)

    def linears(self):
        return [(self.w_in, "none"), (self.w_o, "none")]
