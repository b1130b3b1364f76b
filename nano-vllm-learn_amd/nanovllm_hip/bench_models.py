"""Zobasun beside the closest other model (a Qwen2-shaped stack) at equal size, on random weights: prefill and decode throughput through the engine,
and each hot kernel against its roofline.  bench.py --beside SIZE prints the result as one JSON line."""
from __future__ import annotations

import time

import torch

from . import ops
from .engine.llm_engine import LLMEngine
from .engine.model_runner import recurrence_chunks
from .layers.rglru import choose_segment
from .layers.rotary import rotation_table
from .models.qwen import ModelConfig
from .models.zobasun import ZobasunConfig

HBM_GBPS, MFMA_TFLOPS = 8000.0, 2500.0          # MI355X peaks (dense bf16)

# width, feed-forward, layers; attention heads (128 wide); latent ranks and widths; recurrence width, blocks
SIZES = {
    "1k": dict(width=1024, ff=3072, layers=12, heads=8, kv_heads=2, q_rank=384, kv_rank=256, dim=64, rot=64, vdim=64, rec=1024, blocks=4),
    "2k": dict(width=2048, ff=6144, layers=12, heads=16, kv_heads=4, q_rank=768, kv_rank=512, dim=128, rot=64, vdim=128, rec=2560, blocks=10),
    "4k": dict(width=4096, ff=12288, layers=6, heads=32, kv_heads=8, q_rank=1536, kv_rank=512, dim=128, rot=64, vdim=128, rec=4096, blocks=16),
}
VOCAB = 32000


def configs(size):
    """(Zobasun configuration: two recurrent layers for every latent-attention one; Qwen2-shaped configuration of the same width, depth and feed-forward)."""
    s = SIZES[size]
    mlp = {"kind": "dense", "ff": s["ff"], "limit": 7.0}
    rec = {"type": "rglru", "mixer": {"width": s["rec"], "blocks": s["blocks"], "conv": 4}, "mlp": mlp}
    att = {"type": "latent_attention", "mlp": mlp, "mixer": dict(
        heads=s["heads"], dim=s["dim"], rot_dim=s["rot"], vdim=s["vdim"], q_rank=s["q_rank"], kv_rank=s["kv_rank"], scale=(s["dim"] + s["rot"]) ** -0.5,
        rot={"base": 10000.0, "dims": s["rot"]})}
    new = ZobasunConfig.from_json({"width": s["width"], "vocab": VOCAB, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
                                   "layers": [(rec, rec, att)[i % 3] for i in range(s["layers"])]})
    old = ModelConfig(name=f"Qwen2-shaped {size}", num_hidden_layers=s["layers"], hidden_size=s["width"], num_attention_heads=s["heads"],
                      num_key_value_heads=s["kv_heads"], head_dim=128, intermediate_size=s["ff"], vocab_size=VOCAB, tie_word_embeddings=False, qkv_bias=True,
                      qk_norm=False)
    return new, old


def _engine_throughput(cfg, batch, prompt, decode_steps, repeats=3):
    """Prefill tokens/s (batch x prompt tokens in one step) and decode tokens/s (graph session) of one engine."""
    bs = cfg.kvcache_block_size
    blocks = batch * -(-(prompt + decode_steps + 8) // bs) + 8
    eng = LLMEngine(cfg, blocks, max_num_seqs=max(batch, 4), max_num_batched_tokens=batch * prompt, max_model_len=max(4096, prompt + decode_steps + 8))
    gen = torch.Generator().manual_seed(0)

    def prefill():
        seqs = [eng.sequence(torch.randint(0, VOCAB, (prompt,), generator=gen).tolist(), decode_steps + 1) for _ in range(batch)]
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        eng.prefill(seqs, reserve_tokens=decode_steps + 8)
        torch.cuda.synchronize()
        return seqs, time.perf_counter() - t0

    best = None
    for i in range(repeats + 1):                          # the first one loads kernels and lets the GEMM library choose
        seqs, t = prefill()
        best = t if i == 1 or (i > 1 and t < best) else best
        if i < repeats:
            for s in seqs:
                eng.release(s)
    sess = eng.runner.decode_session(seqs, decode_steps + 4)
    sess.step(4)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    sess.step(decode_steps)
    torch.cuda.synchronize()
    dec = time.perf_counter() - t0
    weights = sum(t.numel() * t.element_size() for t in list(eng.runner.model.buffers()) + list(eng.runner.model.parameters()))
    del sess, eng
    torch.cuda.empty_cache()
    return {"prefill_tok_s": round(batch * prompt / best), "prefill_ms": round(best * 1e3, 3), "decode_tok_s": round(batch * decode_steps / dec),
            "decode_ms_per_step": round(dec / decode_steps * 1e3, 4), "weight_bytes": weights}


def _time(calls, iters=10):
    """us per call: the calls of one pass over distinct operands captured in a graph and replayed."""
    for c in calls[:2]:
        c()
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        for c in calls:
            c()
    graph.replay()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(iters):
        graph.replay()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) * 1e3 / (iters * len(calls))


def _line(us, nbytes=0, flops=0):
    floor = max(nbytes / (HBM_GBPS * 1e3), flops / (MFMA_TFLOPS * 1e6))
    return {"us": round(us, 2), "bound": "hbm" if nbytes / HBM_GBPS * 1e3 >= flops / MFMA_TFLOPS else "mfma", "GBps": round(nbytes / us / 1e3, 1),
            "TFLOPs": round(flops / us / 1e6, 1), "roofline": round(floor / us, 4)}


def _randn(*shape, dtype=torch.bfloat16):
    return torch.randn(*shape, device="cuda", dtype=dtype)


@torch.inference_mode()
def kernels(size, batch=32, ctx=1536, seqs=16, prompt=1024):
    """Each hot kernel of the two models alone; operands cycle through more than the memory-side cache holds where that matters."""
    s, out = SIZES[size], {}
    rows, h, dim, rot, vdim, kv = seqs * prompt, s["heads"], s["dim"], s["rot"], s["vdim"], s["kv_rank"]
    width, ff, rec, blocks = s["width"], s["ff"], s["rec"], s["blocks"]
    dk, cols, scale = dim + rot, kv + 64, (dim + rot) ** -0.5
    table = rotation_table(rot, 10000.0, 4096, "cuda")
    pairs = seqs * prompt * (prompt + 1) / 2
    cu = torch.arange(0, rows + 1, prompt, dtype=torch.int32, device="cuda")
    pos = torch.arange(prompt, device="cuda").repeat(seqs)
    # ---- attention over prompts
    q, k, v, kr = _randn(rows, h, dk), _randn(rows, h, dim), _randn(rows, h, vdim), _randn(rows, 64)
    o = torch.empty(rows, h * vdim, device="cuda", dtype=torch.bfloat16)
    us = _time([lambda: ops.latent_prefill(q, k, kr, v, cu, cu, prompt, pos, table, scale, out=o)] * 4)
    out["latent_prefill"] = _line(us, 2 * rows * (h * (dk + dim + 2 * vdim) + 64), 2 * h * (dk + vdim) * pairs)
    qkv = [_randn(rows, (h + 2 * s["kv_heads"]) * 128) for _ in range(2)]

    def old_prefill(x, pv_fp16):
        p = x.view(rows, -1, 128)
        ops.flash_attn_varlen_func(p[:, :h], p[:, h:h + s["kv_heads"]], p[:, h + s["kv_heads"]:], prompt, cu, prompt, cu, pv_fp16=pv_fp16)
    for name, form in (("qwen_prefill_attention", None), ("qwen_prefill_attention_exact", False)):
        us = _time([lambda x=x: old_prefill(x, form) for x in qkv] * 2)
        out[name] = _line(us, 4 * rows * (h + s["kv_heads"]) * 128, 4 * 128 * h * pairs)
    del q, k, v, qkv
    # ---- decode attention
    pages = -(-ctx // 64)
    n = max(2, int(3e8 // (batch * pages * 64 * cols * 2)) + 1)
    caches = [_randn(batch * pages, 64, cols) for _ in range(n)]
    bt = torch.randperm(batch * pages).view(batch, pages).int().cuda()
    dpos = torch.full((batch,), ctx - 1, device="cuda")
    q, uk, uv = _randn(batch, h * dk), _randn(h, kv, dim), _randn(h, vdim, kv)
    o = torch.empty(batch, h * vdim, device="cuda", dtype=torch.bfloat16)
    us = _time([lambda c=c: ops.latent_attention(q, c, bt, dpos, table, uk, uv, scale, rot, ctx, out=o) for c in caches] * 3)
    out["latent_decode (absorb + attend + value)"] = _line(us, batch * ctx * cols * 2 + 2 * (uk.numel() + uv.numel() + q.numel() + o.numel()))
    del caches
    hk = s["kv_heads"]
    opages = -(-ctx // 256)
    n = max(2, int(3e8 // (4 * batch * opages * 256 * hk * 128)) + 1)
    caches = [_randn(2, batch * opages, 256, hk, 128) for _ in range(n)]
    obt = torch.randperm(batch * opages).view(batch, opages).int().cuda()
    cl = torch.full((batch,), ctx, dtype=torch.int32, device="cuda")
    oq = _randn(batch, h, 128)
    us = _time([lambda c=c: ops.flash_attn_with_kvcache(oq, c[0], c[1], cl, obt) for c in caches] * 3)
    out["qwen_decode_attention"] = _line(us, batch * (4 * ctx * hk * 128 + 4 * h * 128))
    del caches
    # ---- recurrence
    p = dict(conv_w=_randn(4, rec, dtype=torch.float32), conv_b=_randn(rec, dtype=torch.float32), ra=_randn(blocks, rec // blocks, rec // blocks) * 0.05,
             ri=_randn(blocks, rec // blocks, rec // blocks) * 0.05, ra_b=_randn(rec, dtype=torch.float32), ri_b=_randn(rec, dtype=torch.float32),
             rate=torch.rand(rec, device="cuda"))
    slots = torch.arange(max(seqs, batch), dtype=torch.int32, device="cuda")
    state, ring = torch.zeros(max(seqs, batch), rec, device="cuda"), torch.zeros(max(seqs, batch), 4, rec, dtype=torch.bfloat16, device="cuda")
    yx = [_randn(rows, 2 * rec) for _ in range(2)]
    o = torch.empty(rows, rec, device="cuda", dtype=torch.bfloat16)
    seg = choose_segment([prompt] * seqs, blocks)
    chunks = torch.tensor([c for i in range(seqs) for c in recurrence_chunks(i * prompt, prompt, i, seg)], dtype=torch.int32, device="cuda")
    us = _time([lambda x=x: ops.rglru_chunks(x, p, pos, slots, chunks, seg, seg < prompt, state, ring, out=o) for x in yx] * 2)
    out["rglru_chunks"] = _line(us, rows * rec * 6, 4 * rows * rec * (rec // blocks))
    x1 = _randn(batch, 2 * rec)
    us = _time([lambda: ops.rglru_step(x1, p, dpos, slots, state, ring)] * 20)
    out["rglru_step"] = _line(us, 2 * (p["ra"].numel() + p["ri"].numel()) + batch * rec * (6 + 8 + 8))
    # ---- row ops
    xs, ys, w = _randn(rows, width, dtype=torch.float32), [_randn(rows, width) for _ in range(4)], _randn(width, dtype=torch.float32)
    us = _time([lambda y=y: ops.norm_residual(xs, w, 1e-6, width, torch.bfloat16, y=y) for y in ys])
    out["norm_residual"] = _line(us, rows * width * 12)
    rs, wb = _randn(rows, width), _randn(width)
    us = _time([lambda y=y: ops.add_rmsnorm(y, wb, 1e-6, rs) for y in ys])
    out["qwen_add_rmsnorm"] = _line(us, rows * width * 8)
    gu = [_randn(rows, 2 * ff) for _ in range(2)]
    out["clamped_glu"] = _line(_time([lambda g=g: ops.clamped_glu(g, 7.0, 1.702) for g in gu]), rows * ff * 6)
    out["qwen_silu_mul"] = _line(_time([lambda g=g: ops.silu_mul(g) for g in gu]), rows * ff * 6)
    del gu, yx
    # ---- row ops around latent attention
    a = [_randn(rows, s["q_rank"] + cols) for _ in range(4)]
    cache = torch.zeros(rows // 64, 64, cols, dtype=torch.bfloat16, device="cuda")
    slot = torch.arange(rows, dtype=torch.int32, device="cuda")
    qw, kw = torch.ones(s["q_rank"], device="cuda"), torch.ones(kv, device="cuda")
    us = _time([lambda t=t: ops.latent_prep(t, s["q_rank"], qw, 1e-6, pos, table, kv_rank=kv, kv_weight=kw, cache=cache, slots=slot) for t in a])
    out["latent_prep"] = _line(us, rows * 4 * (s["q_rank"] + cols))
    gt = torch.arange(rows // 64, dtype=torch.int32, device="cuda").view(seqs, -1)
    out["latent_gather"] = _line(_time([lambda: ops.latent_gather(cache, cu, rows, gt)] * 4), rows * 4 * cols)
    torch.cuda.empty_cache()
    return out


def run(size, only=None):
    torch.manual_seed(0)
    new, old = configs(size)
    res = {"metric": "Zobasun beside a Qwen2-shaped stack of equal width, depth and feed-forward (random weights)", "size": size, "shape": SIZES[size], "dtype": "bf16"}
    if only in (None, "kernels"):
        res["kernels"] = kernels(size)
    if only in (None, "engine"):
        for batch, prompt in ((16, 1024), (2, 8192)):
            for name, cfg in (("zobasun", new), ("qwen", old)):
                res[f"{name}_{batch}x{prompt}"] = _engine_throughput(cfg, batch, prompt, 64)
        for name, cfg in (("zobasun", new), ("qwen", old)):
            res[f"{name}_32x1024"] = _engine_throughput(cfg, 32, 1024, 256, repeats=1)
    return res
