"""Latent attention: queries through a low-rank latent, keys and values expanded per head from one normed latent per token plus one rotated key
part shared by all heads.  Only [latent | rotated part] is cached, one row per token in pages (`latent_cache`, bound by the runner); a layer
built with `source` reads another layer's cache instead of keeping its own.

Single rows (decode) attend in the latent space, one stream over the cache for all heads; prompt portions expand keys and values of what they
can see and run the MFMA prefill kernel.  Shapes the MFMA kernels do not take, and fp32 models, use the plain latent kernel for both.

Padded widths (zeros): query latent to 64, latent to a width the decode kernel has, rotated part to 64, per-head key width to 64, value to 64.
"""
import torch
from torch import nn

from .. import ops
from .linear import linear, padded, round_up

_LATENT_COLS = (64, 128, 192, 256, 384, 512)             # latent widths of the MFMA decode kernel


class LatentAttention(nn.Module):
    def __init__(self, in_width, in_cols, heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, eps, rope, dtype, source=None):
        super().__init__()
        self.in_width, self.in_cols, self.dtype = in_width, in_cols, dtype
        self.heads, self.dim, self.rot_dim, self.vdim, self.q_rank, self.kv_rank = heads, dim, rot_dim, vdim, q_rank, kv_rank
        self.scale, self.eps, self.rope = float(scale), eps, rope
        self.q_cols = round_up(q_rank, 64)
        self.kv_cols = next((c for c in _LATENT_COLS if c >= kv_rank), round_up(kv_rank, 64))
        self.rot_cols = round_up(rot_dim, 64)
        self.dk = round_up(round_up(dim, 32) + round_up(rot_dim, 8), 64)
        self.dim_cols = max(round_up(dim, 32), self.dk - self.rot_cols)
        self.v_cols = round_up(vdim, 64)
        # the owner of the cache: a list keeps it out of this module's children
        self._source = [source] if source is not None else []
        if source is None:
            self.latent_cache = torch.tensor([])
        else:
            assert not source._source, "the source layer of a shared cache keeps a cache of its own"
            assert (source.kv_rank, source.rot_dim, source.kv_cols, source.rot_cols) == (kv_rank, rot_dim, self.kv_cols, self.rot_cols), "shared cache rows differ"
        self.expand_ok = dtype == torch.bfloat16 and self.scale > 0 and ops.latent_prefill_supported(self.dk, self.v_cols)

    def cache_row(self):
        """Elements and type of one token's cache row; None when another layer's cache is used."""
        return None if self._source else (self.kv_cols + self.rot_cols, self.dtype)

    @property
    def cache(self):
        return self._source[0].latent_cache if self._source else self.latent_cache

    def load(self, get):
        def act(t):
            return t.to(self.dtype).contiguous()
        h, c = self.heads, self.in_cols
        reg = self.register_buffer
        down = [padded(get("dq"), self.q_cols, c)]
        if not self._source:
            dkv = get("dkv")
            assert dkv.shape == (self.kv_rank + self.rot_dim, self.in_width)
            down += [padded(dkv[:self.kv_rank], self.kv_cols, c), padded(dkv[self.kv_rank:], self.rot_cols, c)]
            reg("kv_norm", padded(get("dkv.norm").float(), self.kv_cols))
        reg("w_down", act(torch.cat(down)))
        reg("q_norm", padded(get("dq.norm").float(), self.q_cols))
        uq = get("uq").view(h, self.dim + self.rot_dim, self.q_rank)
        full = uq.new_zeros(h, self.dk, self.q_cols)
        full[:, :self.dim, :self.q_rank] = uq[:, :self.dim]
        full[:, self.dim_cols:self.dim_cols + self.rot_dim, :self.q_rank] = uq[:, self.dim:]
        reg("w_uq", act(full.view(h * self.dk, self.q_cols)))
        uk = padded(get("uk").view(h, self.dim, self.kv_rank), h, self.dim_cols, self.kv_cols)
        uv = padded(get("uv").view(h, self.vdim, self.kv_rank), h, self.v_cols, self.kv_cols)
        reg("w_uk", act(uk.transpose(1, 2)))                                     # [heads, kv_cols, dim_cols]: absorbed form
        reg("w_uv", act(uv))                                                     # [heads, v_cols, kv_cols]
        if self.expand_ok:                                                       # one projection expands keys and values
            reg("w_ukv", act(torch.cat([uk.reshape(-1, self.kv_cols), uv.reshape(-1, self.kv_cols)])))
        o = get("o").view(self.in_width, h, self.vdim)
        reg("w_o", act(padded(padded(o, self.in_width, h, self.v_cols).reshape(self.in_width, h * self.v_cols), c, h * self.v_cols)))

    def _prep(self, a, positions, step, cq_packed=None):
        kv = {} if self._source else dict(kv_rank=self.kv_rank, kv_weight=self.kv_norm, cache=self.cache, slots=step.slot_mapping)
        return ops.latent_prep(a, self.q_rank, self.q_norm, self.eps, positions, self.rope(a.device), cq_packed=cq_packed, **kv)

    def _rows(self, q, positions, step, tables, row_seq=None, **kw):
        return ops.latent_attention(q, self.cache, tables, positions, self.rope(q.device), self.w_uk, self.w_uv, self.scale, self.rot_dim,
                                    step.max_context, row_seq=row_seq, **kw)

    def forward(self, x, positions, step):
        cq = self._prep(linear(x, self.w_down), positions, step)
        q = linear(cq, self.w_uq)
        rows, n = x.shape[0], step.num_decode
        out = torch.empty((rows, self.heads * self.v_cols), dtype=x.dtype, device=x.device)
        if n:
            self._rows(q[:n], positions[:n], step, step.block_tables, out=out[:n])
        if n < rows and not self.expand_ok:
            self._rows(q[n:], positions[n:], step, step.block_tables, row_seq=step.row_seq[n:], out=out[n:])
        elif n < rows:
            seen = ops.latent_gather(self.cache, step.cu_k, step.total_k, step.block_tables[n:])
            kv = linear(seen[:, :self.kv_cols], self.w_ukv)
            k, v = kv.split([self.heads * self.dim_cols, self.heads * self.v_cols], dim=1)
            ops.latent_prefill(q[n:].view(-1, self.heads, self.dk), k.unflatten(1, (self.heads, self.dim_cols)), seen[:, self.kv_cols:],
                               v.unflatten(1, (self.heads, self.v_cols)), step.cu_q, step.cu_k, step.max_q, positions[n:], self.rope(x.device),
                               self.scale, out=out[n:])
        return linear(out, self.w_o)

    def decode(self, xp, rows, positions, step, bufs):
        """Fused decode: fragment-packed rows in, output rows out."""
        a = ops.fused_linear(xp, self.w_down, x_packed_rows=rows, workspace=bufs.workspace)
        cq = bufs.packed(self.q_cols)
        self._prep(a, positions, step, cq_packed=cq)
        q = ops.fused_linear(cq, self.w_uq, x_packed_rows=rows, workspace=bufs.workspace)
        mid = bufs.packed(self.heads * self.v_cols)
        self._rows(q, positions, step, step.block_tables, out_packed=mid, want_out=False)
        return ops.fused_linear(mid, self.w_o, x_packed_rows=rows, workspace=bufs.workspace)

    def linears(self):
        return [(self.w_down, "none"), (self.w_uq, "none"), (self.w_o, "none")]
