"""Zaposun: decoder of time-mixing layers (RWKV style) and layers that run chunked softmax attention with rotated values beside a selective scan, in any order, each
optionally followed by a gelu-gated feed-forward.  The residual stream exists in several copies (hyper-connections): a sublayer reads a weighted sum of them, RMS-normed
in equal groups of columns, and its output is spread over all copies while they are mixed.  A mixer reads every token shifted towards the one before; the
embedding adds a row per hashed pair of tokens.  Streams and norms are fp32.

bfloat16: matrix operands and activations in bf16, everything else in fp32.  float32: all of it in true 32-bit.
Batches of single tokens up to 64 rows take the fused decode path (activations in MFMA-fragment order between the launches); every other batch
runs row-major, decode rows and prompt portions side by side."""
from __future__ import annotations

from dataclasses import dataclass

import torch
from torch import nn

from .. import ops
from ..layers.linear import DecodeBuffers, linear, padded, round_up
from ..layers.mamba import SelectiveScan
from ..layers.mlp import GeluGLU
from ..layers.paged_attention import PagedAttention
from ..layers.parallel import ParallelMixer
from ..layers.rglru import choose_segment
from ..layers.rotary import rotation_table
from ..layers.streams import BigramEmbedding, HyperConnection, TokenShift
from ..layers.wkv import TimeMixing

FUSED_DECODE = True          # tests flip this to compare the fused decode path with the plain one
MAX_STREAMS = 16


@dataclass
class ZaposunConfig:
    hidden_size: int
    vocab_size: int
    layers: list                                    # entries of config.json: type, mixer, mlp
    norm_eps: float
    norm_groups: int
    streams: int
    bigram: dict                                    # buckets, mul_prev, mul_cur
    logit_scale: float
    name: str = "Zaposun"
    dtype: torch.dtype = torch.bfloat16
    kvcache_block_size: int = 64
    max_position_embeddings: int = 32768

    @classmethod
    def from_json(cls, d, **overrides):
        cfg = cls(**{**dict(hidden_size=d["width"], vocab_size=d["vocab"], layers=d["layers"], norm_eps=d["norm"]["eps"], norm_groups=d["norm"]["groups"], streams=d["streams"],
                            bigram=d["embedding"]["bigram"], logit_scale=d["logit_scale"]), **overrides})
        if cfg.hidden_size % cfg.norm_groups:
            raise ValueError(f"width {cfg.hidden_size} in {cfg.norm_groups} norm groups")
        if not 0 < cfg.streams <= MAX_STREAMS:
            raise ValueError(f"{cfg.streams} residual streams; 1 to {MAX_STREAMS} are supported")
        if cfg.bigram["buckets"] < 1:
            raise ValueError(f"{cfg.bigram['buckets']} bigram buckets")
        for i, layer in enumerate(cfg.layers):
            m = layer["mixer"]
            if layer["type"] not in ("wkv", "parallel"):
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer["type"] == "parallel":
                a = m["left"]
                if a["heads"] % a["kv_heads"]:
                    raise ValueError(f"layer {i}: {a['heads']} query heads over {a['kv_heads']} kv_heads")
                if a["rot"]["dims"] % 2 or a["rot"]["dims"] > a["dim"] or a["vdim"] % 2:
                    raise ValueError(f"layer {i}: rot.dims {a['rot']['dims']} of a head of {a['dim']}, values of {a['vdim']}")
                if a["mask"]["size"] < 1:
                    raise ValueError(f"layer {i}: mask.size {a['mask']['size']}")
            if layer["mlp"] is not None and layer["mlp"]["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {layer['mlp']['kind']!r}")
        return cfg

    @property
    def num_hidden_layers(self):
        return len(self.layers)


def _mixer(cfg, spec, d, cols):
    m = spec["mixer"]
    if spec["type"] == "wkv":
        return TimeMixing(d, cols, m["heads"], m["dim"], cfg.norm_eps, cfg.dtype)
    a, s = m["left"], m["right"]

    def table(dims):
        return (lambda device: rotation_table(dims, a["rot"]["base"], cfg.max_position_embeddings, device)) if dims else None
    left = PagedAttention(d, cols, a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["scale"], table(a["rot"]["dims"]), cfg.dtype, cfg.norm_eps, qk_norm="heads",
                          block_size=cfg.kvcache_block_size, chunk=a["mask"]["size"], v_rope=table(a["vdim"]), halves=a["rot"]["dims"])
    return ParallelMixer(d, cols, left, SelectiveScan(d, cols, s["inner"], s["state"], s["dt_rank"], s["conv"], cfg.dtype))


class ZaposunLayer(nn.Module):
    def __init__(self, cfg, index, cols):
        super().__init__()
        spec, d = cfg.layers[index], cfg.hidden_size
        self.mixer = _mixer(cfg, spec, d, cols)
        self.shift = TokenShift(cols, cfg.dtype, len(self.mixer.mixes))
        self.hc1 = HyperConnection(cfg.streams)
        self.mlp = self.hc2 = None
        if spec["mlp"] is not None:
            self.mlp, self.hc2 = GeluGLU(d, cols, spec["mlp"]["ff"], cfg.dtype), HyperConnection(cfg.streams)

    def load(self, get, cols):
        self.mixer.load(lambda n: get("mix." + n))
        self.shift.load(get("shift"), [get("mix.mu." + m) for m in self.mixer.mixes])
        self.hc1.load(lambda n: get("hc1." + n))
        self.register_buffer("norm1", padded(get("norm1").float(), cols))
        if self.mlp is not None:
            self.mlp.load(lambda n: get("mlp." + n))
            self.hc2.load(lambda n: get("hc2." + n))
            self.register_buffer("norm2", padded(get("norm2").float(), cols))


class ZaposunForCausalLM(nn.Module):
    uses_step_meta = True                           # forward takes a StepMeta; batches may mix decode rows and prompt portions

    def __init__(self, cfg: ZaposunConfig):
        super().__init__()
        self.cfg = cfg
        self.cols = round_up(cfg.hidden_size, 64)
        self.embed = BigramEmbedding(cfg.vocab_size, cfg.hidden_size, self.cols, cfg.bigram["buckets"], cfg.bigram["mul_prev"], cfg.bigram["mul_cur"], cfg.dtype)
        self.layers = nn.ModuleList([ZaposunLayer(cfg, i, self.cols) for i in range(cfg.num_hidden_layers)])
        self._bufs = {}

    # ------------------------------------------------------------------ weights
    def load_weights(self, get):
        """get(name) -> tensor under the checkpoint's names."""
        cfg, dtype = self.cfg, self.cfg.dtype
        self.embed.load(get("embed"), get("bigram"))
        for i, layer in enumerate(self.layers):
            layer.load(lambda n, i=i: get(f"l{i}.{n}"), self.cols)
        self.register_buffer("norm", padded(get("final.norm").float() * cfg.logit_scale, self.cols))     # (the logits' scale rides on the last norm)
        self.register_buffer("head", padded(get("head"), round_up(cfg.vocab_size, 64), self.cols).to(dtype).contiguous())
        return self

    def init_random(self, seed=0):
        """Deterministic random weights: N(0, 0.02) matrices, norms around one, decays and step sizes spread over short and long memories, streams that mix a little."""
        gen = torch.Generator().manual_seed(seed)
        return self.load_weights(_RandomTensors(self.cfg, gen))

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids, positions, step):
        """Returns the un-normalised sum of the residual streams of every row (fp32); compute_logits applies the final norm."""
        cfg, rows = self.cfg, input_ids.numel()
        fused = self._fused_ok(rows, step)
        bufs = self._decode_buffers(rows) if fused else None
        x = self.embed(input_ids, positions, step)                   # until the first update all streams are alike
        update = None

        def to_next(hc, norm, **kw):
            """Spread what the sublayer before left, norm what the one behind reads."""
            nonlocal x
            out = torch.empty((rows, cfg.streams, self.cols), dtype=torch.float32, device=x.device) if update is not None and x.dim() == 2 else None
            h = ops.stream_mix(x, cfg.streams, cfg.dtype, cfg.hidden_size, update=update, read=hc.read if hc is not None else None,
                               norm=(norm, cfg.norm_groups, cfg.norm_eps) if hc is not None else None, out=out, **kw)
            x = out if out is not None else x
            return h

        def result(y, hc):
            return dict(y if isinstance(y, dict) else dict(y=y), mix=hc.mix, out=hc.out, eps=cfg.norm_eps)
        for layer in self.layers:
            if fused:
                packed = bufs.packed(self.cols * len(layer.mixer.mixes)) if layer.mixer.mixes else bufs.stream
                to_next(layer.hc1, layer.norm1, want_rows=False, shift=layer.shift.fused(positions, step, packed))
                y = layer.mixer.decode(packed, rows, positions, step, bufs)
            else:
                y = layer.mixer(layer.shift(to_next(layer.hc1, layer.norm1), positions, step), positions, step)
            update = result(y, layer.hc1)
            if layer.mlp is not None:
                h = to_next(layer.hc2, layer.norm2, packed=bufs.stream if fused else None, want_rows=not fused)
                update = result(layer.mlp.decode(bufs.stream, rows, bufs) if fused else layer.mlp(h), layer.hc2)
        return to_next(None, None)

    def _fused_ok(self, rows, step):
        return (FUSED_DECODE and self.cfg.dtype == torch.bfloat16 and step.num_decode == rows and rows <= ops.LINEAR_SMALL_M_MAX
                and all(layer.mixer.step_ok for layer in self.layers))

    def _decode_buffers(self, rows):
        rows = round_up(rows, 16)
        if rows not in self._bufs:
            linears = [l for layer in self.layers for l in layer.mixer.linears() + (layer.mlp.linears() if layer.mlp is not None else [])]
            bufs = self._bufs[rows] = DecodeBuffers(rows, self.head.device, linears + [(self.head, "none")], self.cols)
            for layer in self.layers:
                if layer.mixer.mixes:
                    bufs.packed(self.cols * len(layer.mixer.mixes))
        return self._bufs[rows]

    def recurrence_segment(self, portions):
        """Tokens per recurrence segment for portions of these lengths (the layer with the fewest workgroups fills the GPU last)."""
        units = [layer.mixer.segment_units for layer in self.layers]
        return choose_segment(portions, min(units)) if units and portions else 64

    def compute_logits(self, x):
        """Logits [rows, vocab] (a view of padded rows) of residual-stream sums."""
        cfg, rows = self.cfg, x.shape[0]
        fused = FUSED_DECODE and cfg.dtype == torch.bfloat16 and rows <= ops.LINEAR_SMALL_M_MAX
        bufs = self._decode_buffers(rows) if fused else None
        h = ops.stream_mix(x, 1, cfg.dtype, cfg.hidden_size, norm=(self.norm, cfg.norm_groups, cfg.norm_eps), packed=bufs.stream if fused else None, want_rows=not fused)
        logits = ops.fused_linear(bufs.stream, self.head, x_packed_rows=rows, workspace=bufs.workspace) if fused else linear(h, self.head)
        return logits[:, :cfg.vocab_size]

    def greedy_candidates(self, hidden):
        return None

    def reserve_decode_workspace(self, batch, max_blocks, block_size, device):
        """Allocate what a captured decode step must find in place."""
        if FUSED_DECODE and self.cfg.dtype == torch.bfloat16 and batch <= ops.LINEAR_SMALL_M_MAX:
            self._decode_buffers(batch)


class _RandomTensors:
    """Checkpoint stand-in: every tensor of a configuration drawn when it is asked for."""
    DECAY_RANK = 64

    def __init__(self, cfg, gen):
        d, n = cfg.hidden_size, cfg.streams
        self._gen, self._streams, self._cache = gen, n, {}
        self._shapes = s = {"embed": (cfg.vocab_size, d), "bigram": (cfg.bigram["buckets"] + 1, d), "head": (cfg.vocab_size, d), "final.norm": (d,)}
        for i, layer in enumerate(cfg.layers):
            m, l, p = layer["mixer"], f"l{i}.", f"l{i}.mix."
            s.update({l + t: (d,) for t in ("norm1", "norm2", "shift")})
            for q in ("hc1.", "hc2."):
                s.update({l + q + "in": (n,), l + q + "out": (n,), l + q + "mix": (n, n)})
            if layer["type"] == "wkv":
                a = m["heads"] * m["dim"]
                s.update({p + "mu." + c: (d,) for c in "rkvgw"})
                s.update({p + c: (a, d) for c in "rkvg"})
                s.update({p + "w1": (self.DECAY_RANK, d), p + "w2": (a, self.DECAY_RANK), p + "w0": (a,), p + "u": (m["heads"], m["dim"]), p + "norm": (a,), p + "o": (d, a)})
            else:
                q, f = m["left"], p + "left."
                s.update({f + "q": (q["heads"] * q["dim"], d), f + "k": (q["kv_heads"] * q["dim"], d), f + "v": (q["kv_heads"] * q["vdim"], d), f + "q.norm": (q["dim"],),
                          f + "k.norm": (q["dim"],), f + "o": (d, q["heads"] * q["vdim"]), f + "out": (d,)})
                q, f = m["right"], p + "right."
                e, k, r = q["inner"], q["state"], q["dt_rank"]
                s.update({f + "in": (2 * e, d), f + "conv": (e, q["conv"]), f + "conv.b": (e,), f + "x": (r + 2 * k, e), f + "dt": (e, r), f + "dt.b": (e,), f + "A_log": (e, k),
                          f + "D": (e,), f + "o": (d, e), f + "out": (d,)})
            if layer["mlp"] is not None:
                f = layer["mlp"]["ff"]
                s.update({l + "mlp.gate": (f, d), l + "mlp.up": (f, d), l + "mlp.down": (d, f)})

    def _draw(self, name):
        shape, tail = self._shapes[name], name.rsplit(".", 1)[-1]
        t = torch.randn(shape, generator=self._gen) * 0.02
        if tail in ("norm", "norm1", "norm2", "D") or name.endswith(("left.out", "right.out")):
            t = 1.0 + t
        elif ".hc" in name:
            t = t + (torch.eye(self._streams) if tail == "mix" else 1.0 / self._streams if tail == "in" else 1.0)
        elif tail == "shift" or ".mu." in name:
            t = torch.rand(shape, generator=self._gen)
        elif tail in ("w0", "A_log") or name.endswith("dt.b"):
            t = torch.rand(shape, generator=self._gen) * (5.0 if tail == "w0" else 4.0) - (6.0 if tail == "w0" else 2.0 if tail == "A_log" else 5.0)
        return t.bfloat16()

    def __call__(self, name):
        if name not in self._cache:                          # (a loader may ask for a tensor twice)
            t = self._draw(name)
            if t.numel() > 1 << 22:
                return t
            self._cache[name] = t
        return self._cache[name]
