"""Small configurations the Zaposun tests share."""
import torch

from oracle import zaposun_ref as Z


def wkv(heads, dim, ff=None):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def parallel(heads, kv_heads, dim, vdim, rot, chunk, scale, inner, state, rank, conv, ff=None, base=10000.0):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": rot}, "mask": {"size": chunk}}
    return {"type": "parallel", "mixer": {"left": left, "right": {"inner": inner, "state": state, "dt_rank": rank, "conv": conv}}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(width, vocab, layers, streams=3, groups=1, eps=1e-5, buckets=97, mul_prev=5, mul_cur=3, logit_scale=0.7, decay_rank=12):
    """(_decay_rank: only for the random weights; the framework reads it from the tensors)"""
    return {"architecture": "Zaposun", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps, "groups": groups}, "logit_scale": logit_scale,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}, "layers": layers, "_decay_rank": decay_rank}


CONFIGS = {
    # nothing a power of two, every layer unlike the others, layers without a feed-forward, a convolution of one tap, a chunk of one position
    "odd": config(72, 101, [parallel(6, 2, 20, 14, 12, 37, 0.31, 50, 5, 3, 3, ff=50), wkv(3, 20, ff=36), parallel(3, 3, 36, 22, 36, 1, 0.2, 130, 24, 70, 1), wkv(2, 44),
                            parallel(4, 1, 28, 40, 4, 100, 0.25, 70, 9, 20, 6, ff=70, base=300.0)], streams=3, groups=3),
    # heads and states of the fast kernels, chunks at and past page borders, shared keys, one norm group
    "wide": config(192, 160, [wkv(4, 64, ff=192), parallel(8, 2, 64, 64, 64, 64, 0.15, 256, 16, 64, 4, ff=320), wkv(2, 128), parallel(4, 4, 128, 32, 32, 129, 0.1, 192, 40, 12, 5, ff=64),
                              parallel(12, 1, 100, 128, 100, 65, 0.12, 64, 8, 8, 2)], streams=4, eps=1e-6, logit_scale=1.0, buckets=1, decay_rank=64),
    # beyond the fast kernels, in bf16 too: wide heads, wide keys, a negative scale, norm parts of 17 columns, more streams than any fixed form
    "plain": config(136, 90, [wkv(1, 150, ff=40), parallel(2, 1, 270, 40, 270, 30, 0.1, 40, 70, 5, 7), wkv(5, 8, ff=100), parallel(4, 2, 24, 16, 8, 50, -0.3, 136, 130, 9, 4, ff=24)], streams=5, groups=8,
                    buckets=1000, mul_prev=1, mul_cur=0, logit_scale=-1.5),
    # contractions longer than 1024 in every projection: the decode path's split-K workspace
    "long": config(1280, 300, [wkv(20, 64, ff=1100), parallel(12, 3, 128, 128, 64, 50, 0.12, 1500, 16, 80, 4, ff=1400)], streams=2, groups=5),
    # decays that leave the range of the matrix form of time mixing in some chunks
    "strong": config(128, 64, [wkv(2, 64, ff=64), wkv(1, 128), wkv(4, 32)], streams=2, groups=2),
}
_WEIGHTS = {}


def weights(name):
    if name not in _WEIGHTS:
        w = _WEIGHTS[name] = Z.random_weights(CONFIGS[name], seed=len(name))
        if name == "strong":
            for i in range(3):
                w[f"l{i}.mix.w0"] = (w[f"l{i}.mix.w0"].float() * 0.5 + 2.5).bfloat16()        # between -0.5 and 2.5: factors from 0.54 down to 5e-6 a token
    return _WEIGHTS[name]


class Portions:
    """Rows of a batch: portions = [(first position, tokens, state slot)].  meta(segment) is what the engine tells the kernels about them."""

    def __init__(self, portions, device="cuda"):
        self.portions, self.rows = portions, sum(n for _, n, _ in portions)
        self.single = all(n == 1 for _, n, _ in portions)
        self.device = device

    def i32(self, v):
        return torch.tensor(v, dtype=torch.int32, device=self.device)

    @property
    def positions(self):
        return torch.cat([torch.arange(p, p + n) for p, n, _ in self.portions]).to(self.device)

    @property
    def slots(self):
        return self.i32([s for *_, s in self.portions])

    def chunks(self, segment):
        out, at = [], 0
        for i, (_, n, _) in enumerate(self.portions):
            out += [(at + k, min(segment, n - k), i, k // segment) for k in range(0, n, segment)]
            at += n
        return self.i32(out), any(k for *_, k in out)

    def meta(self, single=None):
        from nanovllm_hip.utils.step import StepMeta
        single = self.single if single is None else single
        if single:
            return StepMeta(self.rows, None, None, self.slots, None, 64, False, 1)
        counts = torch.tensor([n for _, n, _ in self.portions])
        return StepMeta(0, None, None, self.slots, None, 64, False, 1, torch.arange(len(counts)).repeat_interleave(counts).int().to(self.device),
                        torch.cat([torch.zeros(1, dtype=torch.int64), counts.cumsum(0)]).int().to(self.device))


def feed_plan(lengths, cuts, slots):
    """Batches that feed sequences of these lengths in portions: cuts[i] cycles over the portion sizes of sequence i; yields [(sequence, first, count, slot)]."""
    at, turn = [0] * len(lengths), 0
    while any(a < n for a, n in zip(at, lengths)):
        batch = []
        for i, n in enumerate(lengths):
            if at[i] < n and (turn + i) % 4 != 3 or (at[i] < n and len(lengths) == 1):
                k = min(cuts[i][turn % len(cuts[i])], n - at[i])
                batch.append((i, at[i], k, slots[i]))
                at[i] += k
        turn += 1
        if batch:
            yield batch
