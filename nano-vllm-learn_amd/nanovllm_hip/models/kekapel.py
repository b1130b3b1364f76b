"""Kekapel: decoder of windowed softmax attention whose capped scores are mixed across the heads, each layer with a PolyNorm feed-forward, a mixture of clamped
gated experts or none.  Layer norms (weight and bias) stand before and after every sublayer, x += mult norm_b(f(norm(x))); positions enter as learned rows
added to the embedding.  A run of layers may be looped: every pass has its own cache, begins by adding a step vector, and from the second on the embedding.
The stream stays in fp32.

bfloat16: matrix operands and activations in bf16, everything else in fp32.  float32: all of it in true 32-bit.
Batches of single tokens up to 64 rows take the fused decode path (activations in MFMA-fragment order between the launches); every other batch
runs row-major, decode rows and prompt portions side by side."""
from __future__ import annotations

from dataclasses import dataclass, field

import torch
from torch import nn

from .. import ops
from ..layers.linear import DecodeBuffers, linear, padded, round_up
from ..layers.mlp import PolyNormMLP
from ..layers.moe import MixtureOfExperts
from ..layers.paged_attention import PagedAttention
from .looped import LoopedLayers

FUSED_DECODE = True          # tests flip this to compare the fused decode path with the plain one
GATE_ALPHA = 1.702           # of the experts' gated unit


@dataclass
class KekapelConfig(LoopedLayers):
    hidden_size: int
    vocab_size: int
    layers: list                                    # entries of config.json: type, mixer, mlp
    norm_eps: float
    embedding_scale: float
    residual_mult: float
    max_position_embeddings: int                    # rows of the position table; an override can only lower it
    loop: dict | None = None                        # start, stop, times
    name: str = "Kekapel"
    dtype: torch.dtype = torch.bfloat16
    kvcache_block_size: int = 64
    position_rows: int = field(default=0, repr=False)

    @classmethod
    def from_json(cls, d, **overrides):
        cfg = cls(**{**dict(hidden_size=d["width"], vocab_size=d["vocab"], layers=d["layers"], norm_eps=d["norm"]["eps"], embedding_scale=d["embedding"]["scale"],
                            residual_mult=d["residual_mult"], max_position_embeddings=d["max_positions"], loop=d.get("loop"), position_rows=d["max_positions"]), **overrides})
        cfg.max_position_embeddings = min(cfg.max_position_embeddings, cfg.position_rows)
        for i, layer in enumerate(cfg.layers):
            m, mlp = layer["mixer"], layer["mlp"]
            if layer["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: {m['heads']} query heads over {m['kv_heads']} kv_heads")
            if m["mask"]["size"] < 1:
                raise ValueError(f"layer {i}: mask.size {m['mask']['size']}")
            if not m["softcap"] > 0:
                raise ValueError(f"layer {i}: softcap {m['softcap']}")
            if mlp is not None:
                if mlp["kind"] not in ("dense", "moe"):
                    raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
                if mlp["kind"] == "moe" and not 0 < mlp["router"]["top"] <= mlp["router"]["experts"]:
                    raise ValueError(f"layer {i}: top {mlp['router']['top']} of {mlp['router']['experts']} experts")
        cfg.check_loop()
        return cfg


class KekapelLayer(nn.Module):
    def __init__(self, cfg, index, cols):
        super().__init__()
        spec, d = cfg.layers[index], cfg.hidden_size
        m, mlp = spec["mixer"], spec["mlp"]
        self.mixer = PagedAttention(d, cols, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], None, cfg.dtype, cfg.norm_eps, qk_norm="heads",
                                    window=m["mask"]["size"], passes=cfg.passes(index), block_size=cfg.kvcache_block_size, talk=True, softcap=m["softcap"])
        self.mlp = None
        if mlp is not None and mlp["kind"] == "dense":
            self.mlp = PolyNormMLP(d, cols, mlp["ff"], cfg.norm_eps, cfg.dtype)
        elif mlp is not None:
            self.mlp = MixtureOfExperts(d, cols, mlp["expert"]["ff"], mlp["router"]["experts"], mlp["router"]["top"], cfg.dtype, softmax=True,
                                        unit=(mlp["expert"]["limit"], GATE_ALPHA))
        self.experts = isinstance(self.mlp, MixtureOfExperts)

    def load(self, get, cols):
        self.mixer.load(lambda n: get("mix." + n))
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if self.mlp is not None else ()):
            self.register_buffer(n, padded(get(n).float(), cols))
            self.register_buffer(n + "_b", padded(get(n + ".b").float(), cols))
        if self.mlp is not None:
            self.mlp.load(lambda n: get("mlp." + n))

    def norm(self, n):
        return getattr(self, n), getattr(self, n + "_b")


class KekapelForCausalLM(nn.Module):
    uses_step_meta = True                           # forward takes a StepMeta; batches may mix decode rows and prompt portions

    def __init__(self, cfg: KekapelConfig):
        super().__init__()
        self.cfg = cfg
        self.cols = round_up(cfg.hidden_size, 64)
        self.layers = nn.ModuleList([KekapelLayer(cfg, i, self.cols) for i in range(cfg.num_hidden_layers)])
        self.runs = cfg.runs()
        self._bufs = {}

    # ------------------------------------------------------------------ weights
    def load_weights(self, get):
        """get(name) -> tensor under the checkpoint's names."""
        cfg, dtype, cols = self.cfg, self.cfg.dtype, self.cols
        self.register_buffer("embed", padded(get("embed"), cfg.vocab_size, cols).to(dtype).contiguous())
        assert get("pos").shape == (cfg.position_rows, cfg.hidden_size)
        self.register_buffer("pos", padded(get("pos").float(), cfg.position_rows, cols))
        self.register_buffer("step", padded(get("loop.step").float(), cfg.loop["times"], cols) if cfg.loop is not None else None)
        for i, layer in enumerate(self.layers):
            layer.load(lambda n, i=i: get(f"l{i}.{n}"), cols)
        self.register_buffer("norm", padded(get("final.norm").float(), cols))
        self.register_buffer("norm_b", padded(get("final.norm.b").float(), cols))
        self.register_buffer("head", padded(get("head"), round_up(cfg.vocab_size, 64), cols).to(dtype).contiguous())
        return self

    def init_random(self, seed=0):
        """Deterministic random weights (per device kind: experts are many, so they are drawn on the GPU where there is one): N(0, 0.02) matrices, norm weights
        around one, heads mixed a little."""
        device = "cuda" if torch.cuda.is_available() else "cpu"
        gen = torch.Generator(device).manual_seed(seed)
        return self.load_weights(_RandomTensors(self.cfg, lambda shape, std=0.02: (torch.randn(shape, generator=gen, device=device) * std).bfloat16()))

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids, positions, step):
        """Returns the un-normalised residual stream of every row (fp32); compute_logits applies the final norm."""
        cfg, rows = self.cfg, input_ids.numel()
        fused = self._fused_ok(rows, step)
        bufs = self._decode_buffers(rows) if fused else None
        packed = bufs.stream if fused else None
        loop = cfg.loop if cfg.loop is not None and cfg.loop["start"] < cfg.loop["stop"] else None
        first = torch.empty((rows, self.cols), dtype=torch.float32, device=self.embed.device) if loop is not None and loop["times"] > 1 else None
        x, _ = ops.embed_rows(input_ids, self.embed, cfg.embedding_scale, positions=positions, table=self.pos, copy=first, want_rows=False)

        def to_next(norm, want_rows, **add):
            """Add what the sublayer before left, norm for the one behind."""
            return ops.residual_norm(x, cfg.dtype, weight=norm[0], bias=norm[1], eps=cfg.norm_eps, n=cfg.hidden_size, packed=packed, want_rows=want_rows,
                                     mult=cfg.residual_mult, **add)
        add = {}
        for i, run in self.runs:
            layer = self.layers[i]
            if loop is not None and i == loop["start"]:
                add = dict(add, shift=self.step[run], base=first if run else None)
            h = to_next(layer.norm("norm1"), not fused, **add)
            y = layer.mixer.decode(packed, rows, positions, step, bufs, run) if fused else layer.mixer(h, positions, step, run)
            add = dict(y=y, post=layer.norm("norm1b"))
            if layer.mlp is not None:
                h = to_next(layer.norm("norm2"), not fused or layer.experts, **add)
                if layer.experts:
                    add = dict(experts=layer.mlp(h))
                else:
                    add = dict(y=layer.mlp.decode(packed, rows, bufs) if fused else layer.mlp(h))
                add["post"] = layer.norm("norm2b")
        if add:
            ops.residual_norm(x, cfg.dtype, eps=cfg.norm_eps, n=cfg.hidden_size, mult=cfg.residual_mult, **add)
        return x

    def _fused_ok(self, rows, step):
        return (FUSED_DECODE and self.cfg.dtype == torch.bfloat16 and step.num_decode == rows and rows <= ops.LINEAR_SMALL_M_MAX
                and all(layer.mixer.step_ok for layer in self.layers))

    def _decode_buffers(self, rows):
        rows = round_up(rows, 16)
        if rows not in self._bufs:
            linears = [l for layer in self.layers for l in layer.mixer.linears() + (layer.mlp.linears() if isinstance(layer.mlp, PolyNormMLP) else [])]
            self._bufs[rows] = DecodeBuffers(rows, self.embed.device, linears + [(self.head, "none")], self.cols)
        return self._bufs[rows]

    def recurrence_segment(self, portions):
        return 64                                   # (no layer is recurrent)

    def compute_logits(self, x):
        """Logits [rows, vocab] (a view of padded rows) of residual-stream rows."""
        cfg, rows = self.cfg, x.shape[0]
        fused = FUSED_DECODE and cfg.dtype == torch.bfloat16 and rows <= ops.LINEAR_SMALL_M_MAX
        bufs = self._decode_buffers(rows) if fused else None
        h = ops.residual_norm(x, cfg.dtype, weight=self.norm, bias=self.norm_b, eps=cfg.norm_eps, n=cfg.hidden_size, packed=bufs.stream if fused else None, want_rows=not fused)
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

    def __init__(self, cfg, draw):
        d = cfg.hidden_size
        self._draw, self._cache = draw, {}
        self._shapes = s = {"embed": (cfg.vocab_size, d), "pos": (cfg.position_rows, d), "head": (cfg.vocab_size, d), "final.norm": (d,), "final.norm.b": (d,)}
        if cfg.loop is not None:
            s["loop.step"] = (cfg.loop["times"], d)
        for i, layer in enumerate(cfg.layers):
            m, p, q, mlp = layer["mixer"], f"l{i}.mix.", f"l{i}.mlp.", layer["mlp"]
            s.update({f"l{i}.{n}{b}": (d,) for n in ("norm1", "norm1b", "norm2", "norm2b") for b in ("", ".b")})
            h, g = m["heads"], m["kv_heads"]
            s.update({p + "q": (h * m["dim"], d), p + "k": (g * m["dim"], d), p + "v": (g * m["vdim"], d), p + "o": (d, h * m["vdim"]), p + "q.norm": (m["dim"],),
                      p + "k.norm": (m["dim"],), p + "talk": (h, h)})
            if mlp is not None and mlp["kind"] == "dense":
                s.update({q + "up": (mlp["ff"], d), q + "down": (d, mlp["ff"]), q + "act": (4,)})
            elif mlp is not None:
                f, e = mlp["expert"]["ff"], mlp["router"]["experts"]
                s.update({q + "router": (e, d), q + "router.b": (e,)})
                s.update({f"{q}e{k}.{n}": ((f, d) if n != "down" else (d, f)) for k in range(e) for n in ("gate", "up", "down")})

    def __call__(self, name):
        if name not in self._cache:                          # (a loader may ask for a tensor twice)
            t = self._draw(self._shapes[name])
            if name.endswith(("norm", "norm1", "norm2", "norm1b", "norm2b", ".act")):
                t = 1.0 + t
            elif name.endswith(".talk"):
                t = t + torch.eye(t.shape[0], device=t.device, dtype=t.dtype)
            if t.dim() > 1 and t.numel() > 1 << 16:
                return t
            self._cache[name] = t
        return self._cache[name]
