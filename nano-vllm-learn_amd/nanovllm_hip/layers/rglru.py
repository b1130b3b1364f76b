"""Recurrent block: gate branch and recurrent branch off one projection, a causal depthwise convolution, a real-gated linear recurrent unit,
output projection.  State per sequence: the recurrence (fp32) and a ring of the convolution's last inputs; both live in pools indexed by
state slot, bound by the runner (`state`, `conv_state`).

Widths are padded with zero channels (each diagonal block to a multiple of 32, of 64 where the sum needs it): zero inputs keep a zero state.
"""
import torch
import torch.nn.functional as F
from torch import nn

from .. import ops
from .linear import linear, padded, round_up


CUS = 256                     # compute units of an MI355X: one walking workgroup keeps one busy


SEGMENT_OVERHEAD = 0.8        # start of a walk (gate weights into registers, first rows) in units of one 64-token step
SUMMARY_SHARE = 0.7           # a summary walk's step against a full one's


def choose_segment(portions, blocks, chunk=64):
    """Tokens per segment for portions of these lengths: one workgroup walks one (segment, diagonal block), and cutting a portion into more than one
    costs a summary walk over all its segments but the last.  Returns the cheapest multiple of `chunk` among about ten per octave of lengths."""
    longest = max(portions, default=1)
    last = -(-longest // chunk)

    def cost(k):
        pieces = [-(-n // (k * chunk)) for n in portions]
        walk, summary = -(-sum(pieces) * blocks // CUS), -(-sum(p - 1 for p in pieces) * blocks // CUS)
        return (walk + SUMMARY_SHARE * summary) * (min(k, last) + SEGMENT_OVERHEAD)
    steps, k = [last], 1
    while k < last:
        steps.append(k)
        k += max(1, k // 8)
    return chunk * min(steps, key=cost)


class RGLRU(nn.Module):
    """decay_scale: log a = -decay_scale * r * softplus(lam)."""

    def __init__(self, in_width, in_cols, width, blocks, taps, dtype, decay_scale=8.0):
        super().__init__()
        assert width % blocks == 0, f"width {width} must split into {blocks} equal blocks"
        self.in_width, self.in_cols, self.dtype, self.decay_scale = in_width, in_cols, dtype, decay_scale
        self.width, self.blocks, self.size, self.taps = width, blocks, width // blocks, taps
        self.block = round_up(self.size, 32)
        if (self.block * blocks) % 64:
            self.block = round_up(self.size, 64)
        self.cols = self.block * blocks
        self.state = self.conv_state = torch.tensor([])
        self.step_ok = dtype == torch.bfloat16 and ops.rglru_step_supported(self.block)

    def state_spec(self):
        """Per slot: name -> (shape, dtype) of what a sequence keeps between steps."""
        return {"state": ((self.cols,), torch.float32), "conv_state": ((self.taps, self.cols), self.dtype)}

    def _channels(self, t):
        """Leading dimension `width` -> padded blocks."""
        t = t.reshape(self.blocks, self.size, -1)
        return padded(t, self.blocks, self.block, t.shape[2]).reshape(self.cols, -1)

    def load(self, get):
        """get(name) -> tensor of the checkpoint (names below the mixer's prefix)."""
        def act(t):
            return t.to(self.dtype).contiguous()

        def channel_vec(t):
            return self._channels(t.float()).reshape(-1).contiguous()
        assert get("x").shape == (self.width, self.in_width) and get("conv").shape == (self.width, self.taps)
        rows = [padded(self._channels(get(n)), self.cols, self.in_cols) for n in ("y", "x")]
        reg = self.register_buffer
        reg("w_yx", act(torch.cat(rows)))
        reg("b_yx", act(torch.cat([self._channels(get(n + ".b")).reshape(-1) for n in ("y", "x")])))
        reg("conv_w", self._channels(get("conv").float()).t().contiguous())
        reg("conv_b", channel_vec(get("conv.b")))
        for n in ("ra", "ri"):
            reg(n, act(padded(get(n), self.blocks, self.block, self.block)))
            reg(n + "_b", channel_vec(get(n + ".b")))
        reg("rate", self.decay_scale * F.softplus(channel_vec(get("lam")).double()).float())
        reg("w_o", act(padded(self._channels(get("o").t()).t(), self.in_cols, self.cols)))

    @property
    def params(self):
        return dict(conv_w=self.conv_w, conv_b=self.conv_b, ra=self.ra, ri=self.ri, ra_b=self.ra_b, ri_b=self.ri_b, rate=self.rate)

    def forward(self, x, positions, step):
        """x [rows, in_cols] in the activation type -> the block's output, same shape."""
        yx = linear(x, self.w_yx, self.b_yx)
        n = step.num_decode if self.step_ok else 0                   # these rows take the one-launch step, the rest the chunked scan
        out = torch.empty((x.shape[0], self.cols), dtype=x.dtype, device=x.device)
        if n:
            ops.rglru_step(yx[:n], self.params, positions[:n], step.state_slots, self.state, self.conv_state, out=out[:n])
        if n < x.shape[0]:
            ops.rglru_chunks(yx, self.params, positions, step.state_slots, step.chunks[n:], step.segment, step.summaries, self.state,
                             self.conv_state, out=out)
        return linear(out, self.w_o)

    def decode(self, xp, rows, positions, step, bufs):
        """Fused decode: fragment-packed rows in, output rows out (three launches)."""
        yx = ops.fused_linear(xp, self.w_yx, bias=self.b_yx, x_packed_rows=rows, workspace=bufs.workspace)
        mid = bufs.packed(self.cols)
        ops.rglru_step(yx, self.params, positions, step.state_slots, self.state, self.conv_state, out_packed=mid, want_out=False)
        return ops.fused_linear(mid, self.w_o, x_packed_rows=rows, workspace=bufs.workspace)

    def linears(self):
        return [(self.w_yx, "none"), (self.w_o, "none")]
