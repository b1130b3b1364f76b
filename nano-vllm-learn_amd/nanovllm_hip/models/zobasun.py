"""Zobasun: decoder of recurrent blocks and latent-attention layers in any order, each optionally followed by a clamped gated feed-forward.
A sublayer reads the residual stream itself and its OUTPUT is normalised (RMS, weight stored around zero) before it is added; the stream stays in
fp32.  Latent-attention layers may use the cache rows of an earlier one.

bfloat16: matrix operands and activations in bf16, everything else in fp32.  float32: all of it in true 32-bit.
Batches of single tokens up to 64 rows take the fused decode path (activations in MFMA-fragment order between the launches); every other batch
runs row-major, decode rows and prompt portions side by side."""
from __future__ import annotations

from dataclasses import dataclass, field

import torch
import torch.nn.functional as F
from torch import nn

from .. import ops
from ..layers.latent_attention import LatentAttention
from ..layers.linear import DecodeBuffers, linear, padded, round_up
from ..layers.mlp import ClampedGLU
from ..layers.rglru import RGLRU, choose_segment
from ..layers.rotary import rotation_table

FUSED_DECODE = True          # tests flip this to compare the fused decode path with the plain one


@dataclass
class ZobasunConfig:
    hidden_size: int
    vocab_size: int
    layers: list                                    # entries of config.json: type, mixer, mlp
    rms_norm_eps: float
    embedding_scale: float
    name: str = "Zobasun"
    dtype: torch.dtype = torch.bfloat16
    kvcache_block_size: int = 64
    max_position_embeddings: int = 32768
    mixers: tuple = field(default=("rglru", "latent_attention"), repr=False)

    @classmethod
    def from_json(cls, d, **overrides):
        cfg = cls(**{**dict(hidden_size=d["width"], vocab_size=d["vocab"], layers=d["layers"], rms_norm_eps=d["norm"]["eps"],
                            embedding_scale=d["embedding"]["scale"]), **overrides})
        for i, layer in enumerate(cfg.layers):
            m = layer["mixer"]
            if layer["type"] not in cfg.mixers:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer["mlp"] is not None and layer["mlp"]["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {layer['mlp']['kind']!r}")
            if layer["type"] == "latent_attention":
                if m["rot"]["dims"] != m["rot_dim"]:
                    raise ValueError(f"layer {i}: rot.dims {m['rot']['dims']} != rot_dim {m['rot_dim']}")
                if "kv_from" in m:
                    src = cfg.layers[m["kv_from"]] if 0 <= m["kv_from"] < i else None
                    if src is None or src["type"] != "latent_attention" or "kv_from" in src["mixer"] or src["mixer"]["rot"] != m["rot"]:
                        raise ValueError(f"layer {i}: kv_from {m['kv_from']} is no earlier latent-attention layer with a cache and rotation to share")
        return cfg

    @property
    def num_hidden_layers(self):
        return len(self.layers)


class ZobasunLayer(nn.Module):
    def __init__(self, cfg, index, earlier, cols):
        super().__init__()
        spec, d = cfg.layers[index], cfg.hidden_size
        m = spec["mixer"]
        if spec["type"] == "rglru":
            self.mixer = RGLRU(d, cols, m["width"], m["blocks"], m["conv"], cfg.dtype)
        else:
            self.mixer = LatentAttention(
                d, cols, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"], m["scale"], cfg.rms_norm_eps,
                lambda device, m=m: rotation_table(m["rot"]["dims"], m["rot"]["base"], cfg.max_position_embeddings, device), cfg.dtype,
                source=earlier[m["kv_from"]].mixer if "kv_from" in m else None)
        self.mlp = ClampedGLU(d, cols, spec["mlp"]["ff"], spec["mlp"]["limit"], cfg.dtype) if spec["mlp"] is not None else None

    def load(self, get, cols):
        self.mixer.load(lambda n: get("mix." + n))
        self.register_buffer("norm1", padded(1.0 + get("norm1").float(), cols))
        if self.mlp is not None:
            self.mlp.load(lambda n: get("mlp." + n))
            self.register_buffer("norm2", padded(1.0 + get("norm2").float(), cols))


class ZobasunForCausalLM(nn.Module):
    uses_step_meta = True                           # forward takes a StepMeta; batches may mix decode rows and prompt portions

    def __init__(self, cfg: ZobasunConfig):
        super().__init__()
        self.cfg = cfg
        self.cols = round_up(cfg.hidden_size, 64)
        layers = []
        for i in range(cfg.num_hidden_layers):
            layers.append(ZobasunLayer(cfg, i, layers, self.cols))
        self.layers = nn.ModuleList(layers)
        self._bufs = {}

    # ------------------------------------------------------------------ weights
    def load_weights(self, get):
        """get(name) -> tensor under the checkpoint's names."""
        cfg, dtype = self.cfg, self.cfg.dtype
        self.register_buffer("embed", padded(get("embed"), cfg.vocab_size, self.cols).to(dtype).contiguous())
        for i, layer in enumerate(self.layers):
            layer.load(lambda n, i=i: get(f"l{i}.{n}"), self.cols)
        self.register_buffer("final_norm", padded(1.0 + get("final.norm").float(), self.cols))
        self.register_buffer("head", padded(get("head"), round_up(cfg.vocab_size, 64), self.cols).to(dtype).contiguous())
        return self

    def init_random(self, seed=0):
        """Deterministic random weights: N(0, 0.02) matrices, decay parameters spread over short and long memories."""
        gen = torch.Generator().manual_seed(seed)

        def get(shape, std=0.02):
            return (torch.randn(shape, generator=gen) * std).bfloat16()
        return self.load_weights(_RandomTensors(self.cfg, get, gen))

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids, positions, step):
        """Returns the un-normalised residual stream of every row (fp32); compute_logits applies the final norm."""
        cfg = self.cfg
        if self._fused_ok(input_ids.numel(), step):
            return self._forward_decode(input_ids, positions, step)
        x, xb = ops.embed_rows(input_ids, self.embed, cfg.embedding_scale)
        n, eps = cfg.hidden_size, cfg.rms_norm_eps
        for layer in self.layers:
            xb = ops.norm_residual(x, layer.norm1, eps, n, cfg.dtype, y=layer.mixer(xb, positions, step))
            if layer.mlp is not None:
                xb = ops.norm_residual(x, layer.norm2, eps, n, cfg.dtype, y=layer.mlp(xb))
        return x

    def _fused_ok(self, rows, step):
        return (FUSED_DECODE and self.cfg.dtype == torch.bfloat16 and step.num_decode == rows and rows <= ops.LINEAR_SMALL_M_MAX
                and all(getattr(layer.mixer, "step_ok", True) for layer in self.layers))

    def _decode_buffers(self, rows):
        rows = round_up(rows, 16)
        if rows not in self._bufs:
            lin = [l for layer in self.layers for l in layer.mixer.linears() + (layer.mlp.linears() if layer.mlp is not None else [])]
            self._bufs[rows] = DecodeBuffers(rows, self.embed.device, lin + [(self.head, "none")], self.cols)
        return self._bufs[rows]

    def _forward_decode(self, input_ids, positions, step):
        cfg, rows = self.cfg, input_ids.numel()
        n, eps, bufs = cfg.hidden_size, cfg.rms_norm_eps, self._decode_buffers(rows)
        xp = bufs.stream
        x, _ = ops.embed_rows(input_ids, self.embed, cfg.embedding_scale, packed=xp)
        for layer in self.layers:
            y = layer.mixer.decode(xp, rows, positions, step, bufs)
            ops.norm_residual(x, layer.norm1, eps, n, cfg.dtype, y=y, packed=xp, want_rows=False)
            if layer.mlp is not None:
                ops.norm_residual(x, layer.norm2, eps, n, cfg.dtype, y=layer.mlp.decode(xp, rows, bufs), packed=xp, want_rows=False)
        return x

    def recurrence_segment(self, portions):
        """Tokens per recurrence segment for portions of these lengths (the layer with the fewest blocks fills the GPU last)."""
        blocks = [layer.mixer.blocks for layer in self.layers if isinstance(layer.mixer, RGLRU)]
        return choose_segment(portions, min(blocks), ops.rglru_chunk_tokens()) if blocks and portions else ops.rglru_chunk_tokens()

    def compute_logits(self, x):
        """Logits [rows, vocab] (a view of padded rows) of residual-stream rows."""
        cfg, rows = self.cfg, x.shape[0]
        if FUSED_DECODE and cfg.dtype == torch.bfloat16 and rows <= ops.LINEAR_SMALL_M_MAX:
            bufs = self._decode_buffers(rows)
            ops.norm_residual(x, self.final_norm, cfg.rms_norm_eps, cfg.hidden_size, cfg.dtype, packed=bufs.stream, want_rows=False)
            return ops.fused_linear(bufs.stream, self.head, x_packed_rows=rows, workspace=bufs.workspace)[:, :cfg.vocab_size]
        h = ops.norm_residual(x, self.final_norm, cfg.rms_norm_eps, cfg.hidden_size, cfg.dtype)
        return linear(h, self.head)[:, :self.cfg.vocab_size]

    def greedy_candidates(self, hidden):
        return None

    def reserve_decode_workspace(self, batch, max_blocks, block_size, device):
        """Allocate what a captured decode step must find in place."""
        if FUSED_DECODE and self.cfg.dtype == torch.bfloat16 and batch <= ops.LINEAR_SMALL_M_MAX:
            self._decode_buffers(batch)


class _RandomTensors:
    """Checkpoint stand-in: every tensor of a configuration drawn in the order it is asked for."""

    def __init__(self, cfg, get, gen):
        self._get, self._gen, self._shapes = get, gen, {"embed": (cfg.vocab_size, cfg.hidden_size), "head": (cfg.vocab_size, cfg.hidden_size),
                                                        "final.norm": (cfg.hidden_size,)}
        d, s = cfg.hidden_size, self._shapes
        for i, layer in enumerate(cfg.layers):
            m, p = layer["mixer"], f"l{i}.mix."
            s[f"l{i}.norm1"] = s[f"l{i}.norm2"] = (d,)
            if layer["type"] == "rglru":
                w, b = m["width"], m["blocks"]
                s.update({p + "y": (w, d), p + "x": (w, d), p + "y.b": (w,), p + "x.b": (w,), p + "conv": (w, m["conv"]), p + "conv.b": (w,),
                          p + "ra": (b, w // b, w // b), p + "ri": (b, w // b, w // b), p + "ra.b": (b, w // b), p + "ri.b": (b, w // b), p + "lam": (w,),
                          p + "o": (d, w)})
            else:
                h, qr, kr = m["heads"], m["q_rank"], m["kv_rank"]
                s.update({p + "dq": (qr, d), p + "dq.norm": (qr,), p + "uq": (h * (m["dim"] + m["rot_dim"]), qr), p + "dkv": (kr + m["rot_dim"], d),
                          p + "dkv.norm": (kr,), p + "uk": (h * m["dim"], kr), p + "uv": (h * m["vdim"], kr), p + "o": (d, h * m["vdim"])})
            if layer["mlp"] is not None:
                f, q = layer["mlp"]["ff"], f"l{i}.mlp."
                s.update({q + "gate": (f, d), q + "up": (f, d), q + "down": (d, f)})

    def __call__(self, name):
        shape = self._shapes[name]
        if name.endswith(".lam"):
            return (torch.rand(shape, generator=self._gen) * 8.0 - 7.0).bfloat16()
        if name.endswith("q.norm") or name.endswith("kv.norm"):
            return 1.0 + self._get(shape)
        return self._get(shape)
