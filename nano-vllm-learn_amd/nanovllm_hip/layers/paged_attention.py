"""Softmax attention with grouped heads over its own pages: optional projection biases, RMS norm over the whole query and key projections or over every head,
rotation of the leading dimensions, values that turn with their position (the output is turned back), a sliding window with kept first tokens, chunks of positions that
do not see each other, a learned sink per head, scores capped and mixed across the heads.  Every pass
over the layer (a looped layer has several) has its own cache, bound by the runner (`page_cache` [passes, pages, block_size, kv_heads * (dk + dv)], inside a page [kv head][keys | values]).

Single rows (decode) stream the visible keys; prompt portions run the MFMA kernel over the pages.  Widths those kernels do not take, and fp32 models, use
the plain kernel for both.  Padded widths (zeros): keys to 64 / 128 / 192 / 256, values to 64 / 128 / 256.
"""
import torch
from torch import nn

from .. import ops
from .linear import linear, padded, round_up
from .rotary import halves_to_pairs


def padded_widths(dim, vdim):
    """Key and value widths of the MFMA kernels that hold `dim` and `vdim`, or the next multiples of 8."""
    if dim > 256 or vdim > 256:
        return round_up(dim, 8), round_up(vdim, 8)
    dk, dv = round_up(dim, 64), (64 if vdim <= 64 else 128 if vdim <= 128 else 256)
    return (256, 256) if dv == 256 else (dk, dv)


class PagedAttention(nn.Module):
    cache_name = "page_cache"

    def __init__(self, in_width, in_cols, heads, kv_heads, dim, vdim, scale, rope, dtype, eps, bias=False, qk_norm=False, sink=False, window=0, keep_first=0, passes=1,
                 block_size=64, talk=False, softcap=0.0, chunk=0, v_rope=None, halves=None):
        """rope: device -> rotation table, or None.  qk_norm: True (whole projections) or "heads" (one weight for all heads).  talk: scores, capped by softcap
        tanh(score / softcap) if that is not 0, are mixed across the heads before the softmax.  chunk: positions of a chunk (0: one).  v_rope: device -> table of the
        values, all of their dimensions.  halves (not None): the checkpoint pairs dimension i of queries and keys with i + halves / 2 (values: with i + vdim / 2) where
        the kernels take neighbours: weights are reordered while they are read."""
        super().__init__()
        assert talk or not softcap, "capped scores come with mixed heads"
        assert not (talk and (chunk or v_rope)), "mixed heads know windows only"
        assert not (chunk and window)
        assert heads % kv_heads == 0, f"{heads} query heads must share {kv_heads} key/value heads evenly"
        self.in_width, self.in_cols, self.dtype, self.eps, self.rope = in_width, in_cols, dtype, eps, rope
        self.heads, self.kv_heads, self.dim, self.vdim, self.scale = heads, kv_heads, dim, vdim, float(scale)
        self.bias, self.qk_norm, self.has_sink, self.window, self.keep_first, self.passes = bias, qk_norm, sink, int(window), int(keep_first), passes
        self.dk, self.dv = padded_widths(dim, vdim)
        self.q_cols, self.k_cols, self.v_cols = heads * self.dk, kv_heads * self.dk, kv_heads * self.dv
        self.out_cols = round_up(heads * self.dv, 64)
        self.proj_cols = round_up(self.q_cols + self.k_cols + self.v_cols, 64)
        self.page_cache = torch.tensor([])
        self.talking, self.softcap, self.chunk, self.v_rope, self.halves = talk, float(softcap), int(chunk), v_rope, halves
        self.fast = self.fast_prompt = dtype == torch.bfloat16 and heads * self.dv == self.out_cols
        if talk:
            self.fast = self.fast and ops.talk_rows_supported(heads, self.dk, self.dv, block_size)
            self.fast_prompt = self.fast_prompt and ops.talk_prompt_supported(heads, kv_heads, self.dk, self.dv, block_size, self.softcap)
        else:                                                # (the MFMA prompt kernel takes the maximum before the scale)
            self.fast = self.fast_prompt = self.fast and self.scale > 0 and ops.paged_attend_supported(self.dk, self.dv, block_size)

    def cache_row(self):
        """Elements and type of one token's cache row."""
        return self.k_cols + self.v_cols, self.dtype

    def load(self, get):
        """get(name) -> tensor of the checkpoint (names below the mixer's prefix)."""
        h, g, c, reg = self.heads, self.kv_heads, self.in_cols, self.register_buffer
        assert get("q").shape == (h * self.dim, self.in_width) and get("v").shape == (g * self.vdim, self.in_width)

        qk_order = halves_to_pairs(self.dim, self.halves) if self.halves is not None else None
        v_order = halves_to_pairs(self.vdim, self.vdim) if self.halves is not None and self.v_rope is not None else None

        def head_rows(t, n, width, to, order=None):          # [n * width, ...] -> [n * to, ...]
            t = t.reshape(n, width, -1)
            if order is not None:
                t = t[:, order]
            return padded(t, n, to, t.shape[2]).reshape(n * to, -1)
        parts = [("q", h, self.dim, self.dk, qk_order), ("k", g, self.dim, self.dk, qk_order), ("v", g, self.vdim, self.dv, v_order)]
        w = torch.cat([padded(head_rows(get(n), *s), s[0] * s[2], c) for n, *s in parts])
        reg("w_qkv", padded(w, self.proj_cols, c).to(self.dtype).contiguous())
        reg("b_qkv", padded(torch.cat([head_rows(get(n + ".b"), *s).reshape(-1) for n, *s in parts]), self.proj_cols).to(self.dtype).contiguous() if self.bias else None)
        for n, heads in (("q", h), ("k", g)):
            shared = self.qk_norm == "heads"
            reg(n + "_norm", head_rows(get(n + ".norm").float(), 1 if shared else heads, self.dim, self.dk, qk_order).reshape(-1).contiguous() if self.qk_norm else None)
        reg("sink", get("sink").float().contiguous() if self.has_sink else None)
        reg("talk", get("talk").float().contiguous() if self.talking else None)
        if self.talking:
            self.fast_prompt = self.fast_prompt and self.talk.abs().max().item() <= ops.TALK_PROMPT_MAX
        o = get("o").reshape(self.in_width, h, self.vdim)
        o = padded(o if v_order is None else o[:, :, v_order], self.in_width, h, self.dv).reshape(self.in_width, h * self.dv)
        reg("w_o", padded(o, c, self.out_cols).to(self.dtype).contiguous())

    def _prep(self, qkv, positions, step, cache):
        each = self.qk_norm == "heads"
        norm = dict(q_weight=self.q_norm, k_weight=self.k_norm, q_n=self.dim if each else self.heads * self.dim, k_n=self.dim if each else self.kv_heads * self.dim,
                    eps=self.eps, head_norm=each) if self.qk_norm else {}
        table = self.rope(qkv.device) if self.rope is not None else None
        ops.attn_prep(qkv, self.heads, self.kv_heads, self.dk, self.dv, positions, table, cache, step.slot_mapping,
                      v_cos_sin=self.v_rope(qkv.device) if self.v_rope is not None else None, **norm)

    def _mask(self):
        mask = dict(window=self.window, keep_first=self.keep_first, sink=self.sink)
        if self.talking:
            return dict(mask, talk=self.talk, softcap=self.softcap)
        return dict(mask, chunk=self.chunk, turn=self.v_rope(self.w_o.device) if self.v_rope is not None else None)

    def _rows(self, q, positions, step, cache, row_seq=None, **kw):
        attend = ops.talk_rows if self.talking else ops.paged_attend_rows
        return attend(q, cache, step.block_tables, positions, self.heads, self.kv_heads, self.dk, self.dv, self.scale, step.max_context,
                      row_seq=row_seq, **self._mask(), **kw)

    def forward(self, x, positions, step, run=0):
        """x [rows, in_cols] in the activation type -> the mixer's output, same shape; run: which pass over the layer this is."""
        return linear(self.attend(linear(x, self.w_qkv, self.b_qkv), positions, step, run), self.w_o)

    def attend(self, qkv, positions, step, run=0):
        """Everything between the projections; qkv may be a slice of wider rows (queries are rewritten)."""
        rows, n, cache = qkv.shape[0], step.num_decode, self.page_cache[run]
        self._prep(qkv, positions, step, cache)
        alloc = torch.empty if self.heads * self.dv == self.out_cols else torch.zeros
        out = alloc((rows, self.out_cols), dtype=qkv.dtype, device=qkv.device)
        o = out[:, :self.heads * self.dv]
        if n:
            self._rows(qkv[:n], positions[:n], step, cache, out=o[:n])
        if n < rows and self.fast_prompt:
            attend = ops.talk_prompt if self.talking else ops.paged_attend_prompt
            attend(qkv[n:], cache, step.block_tables[n:], step.cu_q, step.cu_k, step.max_q, self.heads, self.kv_heads, self.dk, self.dv, self.scale, out=o[n:], **self._mask())
        elif n < rows:
            self._rows(qkv[n:], positions[n:], step, cache, row_seq=step.row_seq[n:], out=o[n:])
        return out

    @property
    def step_ok(self):
        return self.fast

    def decode(self, xp, rows, positions, step, bufs, run=0):
        """Fused decode: fragment-packed rows in, output rows out (four launches)."""
        qkv = ops.fused_linear(xp, self.w_qkv, bias=self.b_qkv, x_packed_rows=rows, workspace=bufs.workspace)
        return ops.fused_linear(self.decode_attend(qkv, positions, step, bufs, run), self.w_o, x_packed_rows=rows, workspace=bufs.workspace)

    def decode_attend(self, qkv, positions, step, bufs, run=0):
        """attend() of single tokens, fragment-packed."""
        self._prep(qkv, positions, step, self.page_cache[run])
        mid = bufs.packed(self.out_cols)
        self._rows(qkv, positions, step, self.page_cache[run], out_packed=mid, want_out=False)
        return mid

    def linears(self):
        return [(self.w_qkv, "none"), (self.w_o, "none")]
