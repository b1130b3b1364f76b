"""Galirax: decoder whose layers run a mixer (softmax attention in two forms, or lightning attention) and a mixture of experts side by side on one layer
norm of the stream, x += mixer(h) + experts(h).  A run of layers may be looped: several passes with the same weights, each with its own cache and state.
The stream stays in fp32.

bfloat16: matrix operands and activations in bf16, everything else in fp32.  float32: all of it in true 32-bit.
Batches of single tokens up to 64 rows take the fused decode path (activations in MFMA-fragment order between the launches); every other batch
runs row-major, decode rows and prompt portions side by side."""
from __future__ import annotations

from dataclasses import dataclass, field

import torch
from torch import nn

from .. import ops
from ..layers.lightning import LightningAttention
from ..layers.linear import DecodeBuffers, linear, padded, round_up
from ..layers.moe import MixtureOfExperts
from ..layers.paged_attention import PagedAttention
from ..layers.rglru import choose_segment
from ..layers.rotary import rotation_table
from .looped import LoopedLayers

FUSED_DECODE = True          # tests flip this to compare the fused decode path with the plain one


@dataclass
class GaliraxConfig(LoopedLayers):
    hidden_size: int
    vocab_size: int
    layers: list                                    # entries of config.json: type, mixer, mlp
    norm_eps: float
    logit_softcap: float | None = None
    loop: dict | None = None                        # start, stop, times
    name: str = "Galirax"
    dtype: torch.dtype = torch.bfloat16
    kvcache_block_size: int = 64
    max_position_embeddings: int = 32768
    mixers: tuple = field(default=("attention", "attention_2", "lightning"), repr=False)

    @classmethod
    def from_json(cls, d, **overrides):
        cfg = cls(**{**dict(hidden_size=d["width"], vocab_size=d["vocab"], layers=d["layers"], norm_eps=d["norm"]["eps"], logit_softcap=d.get("logit_softcap"),
                            loop=d.get("loop")), **overrides})
        for i, layer in enumerate(cfg.layers):
            m = layer["mixer"]
            if layer["type"] not in cfg.mixers:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer["type"] == "lightning":
                if len(m["decay"]) != m["heads"]:
                    raise ValueError(f"layer {i}: {len(m['decay'])} decays for {m['heads']} heads")
            else:
                if m["heads"] % m["kv_heads"]:
                    raise ValueError(f"layer {i}: {m['heads']} query heads over {m['kv_heads']} kv_heads")
                if m["rot"]["dims"] % 2 or m["rot"]["dims"] > m["dim"]:
                    raise ValueError(f"layer {i}: rot.dims {m['rot']['dims']} of a head of {m['dim']}")
                if layer["type"] == "attention_2" and m["mask"]["size"] < 1:
                    raise ValueError(f"layer {i}: mask.size {m['mask']['size']}")
            if layer["mlp"] is not None:
                if layer["mlp"]["kind"] != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward {layer['mlp']['kind']!r}")
                r = layer["mlp"]["router"]
                g = r["groups"]
                if r["experts"] % g["count"] or not 0 < g["keep"] <= g["count"] or not 0 < r["top"] <= g["keep"] * (r["experts"] // g["count"]):
                    raise ValueError(f"layer {i}: top {r['top']} of {r['experts']} experts in {g['count']} groups, {g['keep']} kept")
        cfg.check_loop()
        return cfg


class GaliraxLayer(nn.Module):
    def __init__(self, cfg, index, cols):
        super().__init__()
        spec, d, passes = cfg.layers[index], cfg.hidden_size, cfg.passes(index)
        m = spec["mixer"]
        if spec["type"] == "lightning":
            self.mixer = LightningAttention(d, cols, m["heads"], m["dim"], m["vdim"], m["decay"], cfg.norm_eps, cfg.dtype, passes=passes)
        else:
            # the second form adds projection biases, the norm over whole projections and the window
            second = spec["type"] == "attention_2"
            mask = m["mask"] if second else {"size": 0}
            rot = m["rot"]
            self.mixer = PagedAttention(
                d, cols, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"],
                lambda device: rotation_table(rot["dims"], rot["base"], cfg.max_position_embeddings, device, rot.get("scaling")), cfg.dtype, cfg.norm_eps,
                bias=second, qk_norm=second, sink=True, window=mask["size"], keep_first=mask.get("keep_first", 0), passes=passes, block_size=cfg.kvcache_block_size)
        self.mlp = None
        if spec["mlp"] is not None:
            r = spec["mlp"]["router"]
            self.mlp = MixtureOfExperts(d, cols, spec["mlp"]["expert"]["ff"], r["experts"], r["top"], cfg.dtype, r["groups"]["count"], r["groups"]["keep"], r["scale"])

    def load(self, get, cols):
        self.mixer.load(lambda n: get("mix." + n))
        self.register_buffer("norm", padded(get("norm1").float(), cols))
        self.register_buffer("norm_b", padded(get("norm1.b").float(), cols))
        if self.mlp is not None:
            self.mlp.load(lambda n: get("mlp." + n))


class GaliraxForCausalLM(nn.Module):
    uses_step_meta = True                           # forward takes a StepMeta; batches may mix decode rows and prompt portions

    def __init__(self, cfg: GaliraxConfig):
        super().__init__()
        self.cfg = cfg
        self.cols = round_up(cfg.hidden_size, 64)
        self.layers = nn.ModuleList([GaliraxLayer(cfg, i, self.cols) for i in range(cfg.num_hidden_layers)])
        self.runs = cfg.runs()
        self._bufs = {}

    # ------------------------------------------------------------------ weights
    def load_weights(self, get):
        """get(name) -> tensor under the checkpoint's names."""
        cfg, dtype = self.cfg, self.cfg.dtype
        self.register_buffer("embed", padded(get("embed"), cfg.vocab_size, self.cols).to(dtype).contiguous())
        for i, layer in enumerate(self.layers):
            layer.load(lambda n, i=i: get(f"l{i}.{n}"), self.cols)
        self.register_buffer("norm", padded(get("final.norm").float(), self.cols))
        self.register_buffer("norm_b", padded(get("final.norm.b").float(), self.cols))
        self.register_buffer("head", padded(get("head"), round_up(cfg.vocab_size, 64), self.cols).to(dtype).contiguous())
        return self

    def init_random(self, seed=0):
        """Deterministic random weights (per device kind: experts are many, so they are drawn on the GPU where there is one): N(0, 0.02) matrices, norm
        weights around one."""
        device = "cuda" if torch.cuda.is_available() else "cpu"
        gen = torch.Generator(device).manual_seed(seed)
        return self.load_weights(_RandomTensors(self.cfg, lambda shape, std=0.02: (torch.randn(shape, generator=gen, device=device) * std).bfloat16()))

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids, positions, step):
        """Returns the un-normalised residual stream of every row (fp32); compute_logits applies the final norm."""
        cfg, rows = self.cfg, input_ids.numel()
        fused = self._fused_ok(rows, step)
        bufs = self._decode_buffers(rows) if fused else None
        x, _ = ops.embed_rows(input_ids, self.embed, 1.0)
        add = {}
        for i, run in self.runs:
            layer = self.layers[i]
            packed = bufs.stream if fused else None
            # what the previous layer adds, and the norm both sublayers of this one read
            h = ops.residual_norm(x, cfg.dtype, weight=layer.norm, bias=layer.norm_b, eps=cfg.norm_eps, n=cfg.hidden_size, packed=packed,
                                  want_rows=not fused or layer.mlp is not None, **add)
            y = layer.mixer.decode(packed, rows, positions, step, bufs, run) if fused else layer.mixer(h, positions, step, run)
            add = dict(y=y, experts=layer.mlp(h) if layer.mlp is not None else None)
        if add:
            ops.residual_norm(x, cfg.dtype, **add)
        return x

    def _fused_ok(self, rows, step):
        return (FUSED_DECODE and self.cfg.dtype == torch.bfloat16 and step.num_decode == rows and rows <= ops.LINEAR_SMALL_M_MAX
                and all(layer.mixer.step_ok for layer in self.layers))

    def _decode_buffers(self, rows):
        rows = round_up(rows, 16)
        if rows not in self._bufs:
            linears = [l for layer in self.layers for l in layer.mixer.linears()]
            self._bufs[rows] = DecodeBuffers(rows, self.embed.device, linears + [(self.head, "none")], self.cols)
        return self._bufs[rows]

    def recurrence_segment(self, portions):
        """Tokens per recurrence segment for portions of these lengths (the layer with the fewest workgroups fills the GPU last)."""
        units = [layer.mixer.segment_units for layer in self.layers if isinstance(layer.mixer, LightningAttention)]
        return choose_segment(portions, min(units)) if units and portions else 64

    def compute_logits(self, x):
        """Logits [rows, vocab] (a view of padded rows) of residual-stream rows."""
        cfg, rows = self.cfg, x.shape[0]
        fused = FUSED_DECODE and cfg.dtype == torch.bfloat16 and rows <= ops.LINEAR_SMALL_M_MAX
        bufs = self._decode_buffers(rows) if fused else None
        h = ops.residual_norm(x, cfg.dtype, weight=self.norm, bias=self.norm_b, eps=cfg.norm_eps, n=cfg.hidden_size, packed=bufs.stream if fused else None, want_rows=not fused)
        logits = ops.fused_linear(bufs.stream, self.head, x_packed_rows=rows, workspace=bufs.workspace) if fused else linear(h, self.head)
        logits = logits[:, :cfg.vocab_size]
        return ops.softcap_(logits, cfg.logit_softcap) if cfg.logit_softcap else logits

    def greedy_candidates(self, hidden):
        return None

    def reserve_decode_workspace(self, batch, max_blocks, block_size, device):
        """Allocate what a captured decode step must find in place."""
        if FUSED_DECODE and self.cfg.dtype == torch.bfloat16 and batch <= ops.LINEAR_SMALL_M_MAX:
            self._decode_buffers(batch)


class _RandomTensors:
    """Checkpoint stand-in: every tensor of a configuration drawn in the order it is asked for."""

    def __init__(self, cfg, draw):
        d, s = cfg.hidden_size, {"embed": (cfg.vocab_size, cfg.hidden_size), "head": (cfg.vocab_size, cfg.hidden_size), "final.norm": (cfg.hidden_size,),
                                 "final.norm.b": (cfg.hidden_size,)}
        self._draw, self._shapes = draw, s
        for i, layer in enumerate(cfg.layers):
            m, p = layer["mixer"], f"l{i}.mix."
            s[f"l{i}.norm1"] = s[f"l{i}.norm1.b"] = (d,)
            h = m["heads"]
            g = h if layer["type"] == "lightning" else m["kv_heads"]
            s.update({p + "q": (h * m["dim"], d), p + "k": (g * m["dim"], d), p + "v": (g * m["vdim"], d), p + "g": (h * m["vdim"], d), p + "o": (d, h * m["vdim"]),
                      p + "norm": (h * m["vdim"],), p + "sink": (h,), p + "q.b": (h * m["dim"],), p + "k.b": (g * m["dim"],), p + "v.b": (g * m["vdim"],),
                      p + "q.norm": (h * m["dim"],), p + "k.norm": (g * m["dim"],)})
            if layer["mlp"] is not None:
                f, e, q = layer["mlp"]["expert"]["ff"], layer["mlp"]["router"]["experts"], f"l{i}.mlp."
                s.update({q + "router": (e, d), q + "correction": (e,)})
                s.update({f"{q}e{k}.{n}": ((f, d) if n != "down" else (d, f)) for k in range(e) for n in ("gate", "up", "down")})
        self._cache = {}

    def __call__(self, name):
        if name not in self._cache:                          # (a loader may ask for a tensor twice)
            t = self._draw(self._shapes[name])
            self._cache[name] = 1.0 + t if name.endswith(("norm", "norm1")) else t
            if t.dim() > 1 and t.numel() > 1 << 16:
                return self._cache.pop(name)
        return self._cache[name]
