"""Several copies of the residual stream (hyper-connections), and what reads the token before.

HyperConnection: the weights of one sublayer, which reads sum_s read[s] x_s and whose output y goes into x_t <- sum_s mix[s, t] x_s + out[t] y.
TokenShift: h + (h' - h) shift with h' the previous token's h; a mixer that itself mixes every token with the previous one gets all of its mixes from the same
launch.  A sequence's last rows live in a ring (`ring` [slots, depth, cols], bound by the runner).
BigramEmbedding: embed[token] + bigram[hash of previous and current token]; the previous token lives in `last_token` [slots]."""
import torch
from torch import nn

from .. import ops
from .linear import padded


class HyperConnection(nn.Module):
    def __init__(self, streams):
        super().__init__()
        self.streams = streams

    def load(self, get):
        for name, n, shape in (("read", "in", (self.streams,)), ("out", "out", (self.streams,)), ("mix", "mix", (self.streams, self.streams))):
            assert get(n).shape == shape
            self.register_buffer(name, get(n).float().contiguous())


class TokenShift(nn.Module):
    def __init__(self, cols, dtype, mixes=0):
        super().__init__()
        self.cols, self.dtype, self.mixes = cols, dtype, mixes
        self.ring = torch.tensor([])

    def state_spec(self):
        """Per slot: name -> (shape, dtype) of what a sequence keeps between steps."""
        return {"ring": ((3 if self.mixes else 2, self.cols), self.dtype)}

    def load(self, shift, mu=()):
        """mu: the mixer's own mixes, in the order in which it takes them."""
        assert len(mu) == self.mixes
        self.register_buffer("shift", padded(shift.float(), self.cols))
        self.register_buffer("mu", torch.stack([padded(m.float(), self.cols) for m in mu]) if self.mixes else None)

    def forward(self, h, positions, step):
        """[rows, cols] -> the shifted rows, or [mixes, rows, cols]."""
        s = ops.token_shift(h, positions, step, self.shift, self.ring, self.mu)
        return s if self.mixes else s[0]

    def fused(self, positions, step, packed):
        """What ops.stream_mix needs to do this to single tokens in the launch that norms them; packed: where the rows go in fragment order."""
        return dict(positions=positions, step=step, shift=self.shift, ring=self.ring, mu=self.mu, packed=packed)


class BigramEmbedding(nn.Module):
    def __init__(self, vocab, width, cols, buckets, mul_prev, mul_cur, dtype):
        super().__init__()
        self.vocab, self.width, self.cols, self.dtype = vocab, width, cols, dtype
        self.buckets, self.mul_prev, self.mul_cur = buckets, mul_prev, mul_cur
        self.last_token = torch.tensor([])

    def state_spec(self):
        return {"last_token": ((), torch.int64)}

    def load(self, embed, bigram):
        assert embed.shape == (self.vocab, self.width) and bigram.shape == (self.buckets + 1, self.width)
        self.register_buffer("embed", padded(embed, self.vocab, self.cols).to(self.dtype).contiguous())
        self.register_buffer("bigram", padded(bigram, self.buckets + 1, self.cols).to(self.dtype).contiguous())

    def forward(self, tokens, positions, step):
        return ops.bigram_embed(tokens, positions, step, self.embed, self.bigram, self.mul_prev, self.mul_cur, self.last_token)
