"""Selective scan (Mamba): a causal depthwise convolution and silu, step sizes and input and output vectors projected from its result, a diagonal state per channel,
output gate and projection.  State per sequence: the scan (`state` [slots, inner, states], fp32) and a ring of the convolution's last inputs (`conv_state`); both are
bound by the runner.

Padded widths (zeros): channels to a multiple of 64, states to a power of two: zero inputs keep a zero state.
"""
import torch
from torch import nn

from .. import ops
from .linear import linear, padded, round_up


class SelectiveScan(nn.Module):
    # what choose_segment takes for workgroups that walk one segment: it counts one per CU, the scan's small ones want company (three per CU)
    segment_units = property(lambda self: max(1, self.inner_cols // 192))

    def __init__(self, in_width, in_cols, inner, states, rank, taps, dtype):
        super().__init__()
        self.in_width, self.in_cols, self.inner, self.states, self.rank, self.taps, self.dtype = in_width, in_cols, inner, states, rank, taps, dtype
        self.inner_cols, self.rank_cols, self.n = round_up(inner, 64), round_up(rank, 64), ops.scan_states(states)
        if not self.n:
            raise ValueError(f"{states} states per channel are more than the scan kernels hold")
        self.x_cols = self.rank_cols + round_up(2 * self.n, 64)
        self.proj_cols = 2 * self.inner_cols
        self.state = self.conv_state = torch.tensor([])
        self.step_ok = dtype == torch.bfloat16

    def state_spec(self):
        """Per slot: name -> (shape, dtype) of what a sequence keeps between steps."""
        return {"state": ((self.inner_cols, self.n), torch.float32), "conv_state": ((self.taps, self.inner_cols), self.dtype)}

    def load(self, get):
        e, c, n, reg = self.inner, self.inner_cols, self.states, self.register_buffer

        def act(t):
            return t.to(self.dtype).contiguous()
        assert get("in").shape == (2 * e, self.in_width) and get("conv").shape == (e, self.taps) and get("x").shape == (self.rank + 2 * n, e) and get("A_log").shape == (e, n)
        reg("w_in", act(torch.cat([padded(t, c, self.in_cols) for t in get("in").split(e)])))
        reg("conv_w", padded(get("conv").float().t(), self.taps, c))
        reg("conv_b", padded(get("conv.b").float(), c))
        dt, b, cc = (padded(t, w, c) for t, w in zip(get("x").split([self.rank, n, n]), (self.rank_cols, self.n, self.n)))
        reg("w_x", act(padded(torch.cat([dt, b, cc]), self.x_cols, c)))
        reg("w_dt", act(padded(get("dt"), c, self.rank_cols)))
        reg("dt_bias", padded(get("dt.b").float(), c))
        reg("a_log2", padded(-torch.exp(get("A_log").double()) * 1.4426950408889634, c, self.n).float())
        reg("d", padded(get("D").float(), c))
        reg("w_o", act(padded(get("o"), self.in_cols, c)))

    @property
    def params(self):
        return dict(a_log2=self.a_log2, d=self.d, dt_bias=self.dt_bias, w_dt=self.w_dt)

    def _views(self, xz, dbc):
        """(input, step sizes' low-rank row, B | C, gate) of projected rows."""
        c, r = self.inner_cols, self.rank_cols
        return xz[:, :c], dbc[:, :r], dbc[:, r:r + 2 * self.n], xz[:, c:2 * c]

    def forward(self, x, positions, step):
        """x [rows, in_cols] in the activation type -> the mixer's output, same shape."""
        return linear(self.scan(linear(x, self.w_in), positions, step), self.w_o)

    def scan(self, xz, positions, step):
        """Everything between the projections; xz may be a slice of wider rows."""
        rows, n = xz.shape[0], step.num_decode if self.step_ok else 0      # the first n rows take the one-launch step, the rest the chunked walk
        x = ops.causal_conv(xz[:, :self.inner_cols], positions, step, self.conv_w, self.conv_b, self.conv_state)
        dbc = linear(x, self.w_x)
        _, low, bc, z = self._views(xz, dbc)
        out = torch.empty((rows, self.inner_cols), dtype=x.dtype, device=x.device)
        if n:
            ops.scan_step(x[:n], low[:n], bc[:n], z[:n], self.params, positions[:n], step.state_slots, self.state, out=out[:n])
        if n < rows:
            ops.scan_chunks(x, linear(low, self.w_dt), bc, z, self.params, positions, step.state_slots, step.chunks[n:], step.summaries, self.state, out=out)
        return out

    def decode_scan(self, xz, rows, positions, step, bufs):
        """scan() of single tokens, fragment-packed (three launches)."""
        mid = bufs.packed(self.inner_cols)
        x = ops.causal_conv(xz[:, :self.inner_cols], positions, step, self.conv_w, self.conv_b, self.conv_state, packed=mid)
        dbc = ops.fused_linear(mid, self.w_x, x_packed_rows=rows, workspace=bufs.workspace)
        _, low, bc, z = self._views(xz, dbc)
        ops.scan_step(x, low, bc, z, self.params, positions, step.state_slots, self.state, out_packed=mid, want_out=False)
        return mid

    def linears(self):
        return [(self.w_in, "none"), (self.w_x, "none"), (self.w_o, "none")]
