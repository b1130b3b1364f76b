"""Zobasun, Galirax, Kekapel or Zaposun beside the closest other model (a Qwen2-shaped stack; for Kekapel also Galirax with windows in every layer, for Zaposun also
Zobasun) at equal size, on random weights: prefill and decode throughput through the engine, and each hot kernel against its roofline.
bench.py --beside SIZE [--beside-model NAME] prints the result as one JSON line."""
from __future__ import annotations

import time

import torch

import torch.nn.functional as F

from . import ops
from .engine.llm_engine import LLMEngine
from .engine.model_runner import recurrence_chunks
from .layers.rglru import choose_segment
from .layers.rotary import rotation_table
from .models.galirax import GaliraxConfig
from .models.kekapel import KekapelConfig
from .models.qwen import ModelConfig
from .models.zaposun import ZaposunConfig
from .models.zobasun import ZobasunConfig
from .utils.step import StepMeta

HBM_GBPS, MFMA_TFLOPS = 8000.0, 2500.0          # MI355X peaks (dense bf16)

# width, feed-forward, layers; attention heads (128 wide); latent ranks and widths; recurrence width, blocks; experts (each ff / top wide)
SIZES = {
    "1k": dict(width=1024, ff=3072, layers=12, heads=8, kv_heads=2, q_rank=384, kv_rank=256, dim=64, rot=64, vdim=64, rec=1024, blocks=4, experts=32, top=4),
    "2k": dict(width=2048, ff=6144, layers=12, heads=16, kv_heads=4, q_rank=768, kv_rank=512, dim=128, rot=64, vdim=128, rec=2560, blocks=10, experts=32, top=4),
    "4k": dict(width=4096, ff=12288, layers=6, heads=32, kv_heads=8, q_rank=1536, kv_rank=512, dim=128, rot=64, vdim=128, rec=4096, blocks=16, experts=32, top=4),
}
VOCAB = 32000
WINDOW, KEEP = 512, 4                           # Galirax's windowed layers; Kekapel's window; Zaposun's chunks
STREAMS, STATES, TAPS = 4, 16, 4                # Zaposun


def qwen_config(size):
    s = SIZES[size]
    return ModelConfig(name=f"Qwen2-shaped {size}", num_hidden_layers=s["layers"], hidden_size=s["width"], num_attention_heads=s["heads"],
                       num_key_value_heads=s["kv_heads"], head_dim=128, intermediate_size=s["ff"], vocab_size=VOCAB, tie_word_embeddings=False, qkv_bias=True,
                       qk_norm=False)


def galirax_config(size, windows_only=False):
    """Windowed attention, lightning attention, full attention in turn (windows_only: windowed attention in every layer); the experts a token uses are together
    as wide as the Qwen stack's feed-forward."""
    s = SIZES[size]
    mlp = {"kind": "moe", "expert": {"ff": s["ff"] // s["top"]}, "router": {"experts": s["experts"], "top": s["top"], "groups": {"count": 8, "keep": 4}, "scale": 2.5}}
    att = dict(heads=s["heads"], kv_heads=s["kv_heads"], dim=128, vdim=128, scale=128 ** -0.5, rot={"base": 10000.0, "dims": 128})
    kinds = [("attention_2", {**att, "mask": {"size": WINDOW, "keep_first": KEEP}}),
             ("lightning", dict(heads=s["heads"], dim=128, vdim=128, decay=[1 - 2.0 ** -(3 + 6 * i / s["heads"]) for i in range(s["heads"])])), ("attention", att)]
    if windows_only:
        kinds = kinds[:1] * 3
    return GaliraxConfig.from_json({"width": s["width"], "vocab": VOCAB, "norm": {"eps": 1e-6}, "logit_softcap": 15.0,
                                    "layers": [dict(type=kinds[i % 3][0], mixer=kinds[i % 3][1], mlp=mlp) for i in range(s["layers"])]})


def kekapel_config(size):
    """Windowed attention with mixed heads in every layer, dense feed-forwards and experts in turn."""
    s = SIZES[size]
    att = dict(heads=s["heads"], kv_heads=s["kv_heads"], dim=128, vdim=128, scale=128 ** -0.5, softcap=20.0, mask={"size": WINDOW})
    mlps = ({"kind": "dense", "ff": s["ff"]}, {"kind": "moe", "expert": {"ff": s["ff"] // s["top"], "limit": 7.0}, "router": {"experts": s["experts"], "top": s["top"]}})
    return KekapelConfig.from_json({"width": s["width"], "vocab": VOCAB, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0}, "residual_mult": 0.7, "max_positions": 16384,
                                    "layers": [dict(type="attention", mixer=att, mlp=mlps[i % 2]) for i in range(s["layers"])]})


def zaposun_config(size):
    """Time mixing (heads of 64) and attention beside a scan of twice the width in turn."""
    s = SIZES[size]
    mlp = {"kind": "dense", "ff": s["ff"]}
    wkv = {"type": "wkv", "mixer": {"heads": s["width"] // 64, "dim": 64}, "mlp": mlp}
    par = {"type": "parallel", "mlp": mlp, "mixer": {
        "left": dict(heads=s["heads"], kv_heads=s["kv_heads"], dim=128, vdim=128, scale=128 ** -0.5, rot={"base": 10000.0, "dims": 128}, mask={"size": WINDOW}),
        "right": dict(inner=2 * s["width"], state=STATES, dt_rank=s["width"] // 16, conv=TAPS)}}
    return ZaposunConfig.from_json({"width": s["width"], "vocab": VOCAB, "norm": {"eps": 1e-6, "groups": 2}, "streams": STREAMS, "logit_scale": 1.0,
                                    "embedding": {"bigram": {"buckets": 4093, "mul_prev": 29, "mul_cur": 13}}, "layers": [(wkv, par)[i % 2] for i in range(s["layers"])]})


def zobasun_config(size):
    """Two recurrent layers for every latent-attention one."""
    s = SIZES[size]
    mlp = {"kind": "dense", "ff": s["ff"], "limit": 7.0}
    rec = {"type": "rglru", "mixer": {"width": s["rec"], "blocks": s["blocks"], "conv": 4}, "mlp": mlp}
    att = {"type": "latent_attention", "mlp": mlp, "mixer": dict(
        heads=s["heads"], dim=s["dim"], rot_dim=s["rot"], vdim=s["vdim"], q_rank=s["q_rank"], kv_rank=s["kv_rank"], scale=(s["dim"] + s["rot"]) ** -0.5,
        rot={"base": 10000.0, "dims": s["rot"]})}
    return ZobasunConfig.from_json({"width": s["width"], "vocab": VOCAB, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
                                    "layers": [(rec, rec, att)[i % 3] for i in range(s["layers"])]})


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


def qwen_attention(size, batch, ctx, seqs, prompt):
    """The Qwen stack's prompt and decode attention."""
    s, out, rows = SIZES[size], {}, seqs * prompt
    h, hk = s["heads"], s["kv_heads"]
    cu = torch.arange(0, rows + 1, prompt, dtype=torch.int32, device="cuda")
    pairs = seqs * prompt * (prompt + 1) / 2
    qkv = [_randn(rows, (h + 2 * hk) * 128) for _ in range(2)]

    def old_prefill(x, pv_fp16):
        p = x.view(rows, -1, 128)
        ops.flash_attn_varlen_func(p[:, :h], p[:, h:h + hk], p[:, h + hk:], prompt, cu, prompt, cu, pv_fp16=pv_fp16)
    for name, form in (("qwen_prefill_attention", None), ("qwen_prefill_attention_exact", False)):
        us = _time([lambda x=x: old_prefill(x, form) for x in qkv] * 2)
        out[name] = _line(us, 4 * rows * (h + hk) * 128, 4 * 128 * h * pairs)
    oq = _randn(batch, h, 128)
    for name, c in (("qwen_decode_attention", ctx), (f"qwen_decode_attention, context {WINDOW + KEEP}", WINDOW + KEEP)):
        opages = -(-c // 256)
        n = max(2, int(3e8 // (4 * batch * opages * 256 * hk * 128)) + 1)
        caches = [_randn(2, batch * opages, 256, hk, 128) for _ in range(n)]
        obt = torch.randperm(batch * opages).view(batch, opages).int().cuda()
        cl = torch.full((batch,), c, dtype=torch.int32, device="cuda")
        us = _time([lambda kv=kv: ops.flash_attn_with_kvcache(oq, kv[0], kv[1], cl, obt) for kv in caches] * 3)
        out[name] = _line(us, batch * (4 * c * hk * 128 + 4 * h * 128))
        del caches
    return out


@torch.inference_mode()
def galirax_kernels(size, batch=32, ctx=1536, seqs=16, prompt=1024):
    """Each hot kernel of Galirax alone, and the Qwen stack's like ones; operands cycle through more than the memory-side cache holds where that matters."""
    s, out, rows = SIZES[size], qwen_attention(size, batch, ctx, seqs, prompt), seqs * prompt
    h, g, d, width, experts, top = s["heads"], s["kv_heads"], 128, s["width"], s["experts"], s["top"]
    ff = s["ff"] // top
    cu = torch.arange(0, rows + 1, prompt, dtype=torch.int32, device="cuda")
    pos = torch.arange(prompt, device="cuda").repeat(seqs)
    table = rotation_table(d, 10000.0, 4096, "cuda")
    sink = torch.ones(h, device="cuda")
    # ---- attention over prompts, row ops in front
    cols = (h + 2 * g) * d
    qkv = [_randn(rows, cols) for _ in range(3)]
    cache = torch.zeros(rows // 64, 64, 2 * g * d, dtype=torch.bfloat16, device="cuda")
    slot = torch.arange(rows, dtype=torch.int32, device="cuda")
    qw, kw = torch.ones(h * d, device="cuda"), torch.ones(g * d, device="cuda")
    us = _time([lambda x=x: ops.attn_prep(x, h, g, d, d, pos, table, cache, slot, qw, kw, h * d, g * d, 1e-6) for x in qkv])
    out["attn_prep"] = _line(us, rows * 4 * cols)
    bt = torch.arange(rows // 64, dtype=torch.int32, device="cuda").view(seqs, -1)
    o = torch.empty(rows, h * d, device="cuda", dtype=torch.bfloat16)
    nbytes = 4 * rows * (h + g) * d
    for name, mask in (("paged_prompt", {}), ("paged_prompt_window", dict(window=WINDOW, keep_first=KEEP))):
        us = _time([lambda x=x: ops.paged_attend_prompt(x, cache, bt, cu, cu, prompt, h, g, d, d, d ** -0.5, sink=sink, out=o, **mask) for x in qkv] * 2)
        seen = sum(min(t + 1, WINDOW) + min(KEEP, max(0, t + 1 - WINDOW)) for t in range(prompt)) if mask else prompt * (prompt + 1) / 2
        out[name] = _line(us, nbytes, 4 * d * h * seqs * seen)
    del qkv, o, cache
    # ---- decode attention
    pages = -(-ctx // 64)
    n = max(2, int(3e8 // (batch * pages * 64 * 4 * g * d)) + 1)
    caches = [_randn(batch * pages, 64, 2 * g * d) for _ in range(n)]
    bt = torch.randperm(batch * pages).view(batch, pages).int().cuda()
    dpos = torch.full((batch,), ctx - 1, device="cuda")
    q, o = _randn(batch, h * d), torch.empty(batch, h * d, device="cuda", dtype=torch.bfloat16)
    for name, mask, seen in (("paged_rows", {}, ctx), ("paged_rows_window", dict(window=WINDOW, keep_first=KEEP), WINDOW + KEEP)):
        us = _time([lambda c=c: ops.paged_attend_rows(q, c, bt, dpos, h, g, d, d, d ** -0.5, ctx, sink=sink, out=o, **mask) for c in caches] * 3)
        out[name] = _line(us, batch * (4 * seen * g * d + 4 * h * d))
    del caches
    # ---- lightning attention
    x = [_randn(rows, 4 * h * d) for _ in range(2)]
    decay = torch.linspace(0.8, 0.999, h, device="cuda")
    slots = torch.arange(max(seqs, batch), dtype=torch.int32, device="cuda")
    state = torch.zeros(max(seqs, batch), h, d, d, device="cuda")
    o = torch.empty(rows, h * d, device="cuda", dtype=torch.bfloat16)
    seg = choose_segment([prompt] * seqs, h * 2)
    chunks = torch.tensor([c for i in range(seqs) for c in recurrence_chunks(i * prompt, prompt, i, seg)], dtype=torch.int32, device="cuda")
    us = _time([lambda a=a: ops.lightning_chunks(a, decay, pos, slots, chunks, seg < prompt, state, out=o) for a in x] * 2)
    out["lightning_chunks"] = _line(us, rows * 8 * h * d, 4 * rows * h * d * d)
    us = _time([lambda a=a: ops.norm_gate(o, a[:, 3 * h * d:], qw, 1e-6, h * d) for a in x])
    out["norm_gate"] = _line(us, rows * 6 * h * d)
    x1 = _randn(batch, 4 * h * d)
    states = [torch.zeros(batch, h, d, d, device="cuda") for _ in range(max(2, int(3e8 // (4 * batch * h * d * d)) + 1))]
    us = _time([lambda t=t: ops.lightning_step(x1, decay, dpos, slots, t) for t in states] * 3)
    out["lightning_step"] = _line(us, 8 * batch * h * d * d)
    del x, o, states, state
    # ---- experts, large batch
    xs, router, corr = [_randn(rows, width) for _ in range(2)], _randn(experts, width) * width ** -0.5, torch.zeros(experts, device="cuda")
    us = _time([lambda a=a: ops.moe_route(a, router, corr, top, 8, 4, 2.5) for a in xs] * 2)
    out["moe_route"] = _line(us, 2 * rows * width, 2 * rows * width * experts)
    ids, ew = ops.moe_route(xs[0], router, corr, top, 8, 4, 2.5)
    us = _time([lambda: ops.moe_dispatch(ids, experts, torch.bfloat16)] * 4)
    out["moe_dispatch"] = _line(us, 8 * rows * top)
    dispatch = ops.moe_dispatch(ids, experts, torch.bfloat16)
    wgu = [_randn(experts, 2 * ff, width) * 0.02 for _ in range(max(1, int(3e8 // (4 * experts * ff * width)) + 1))]
    wdn = [_randn(experts, width, ff) * 0.02 for _ in range(max(1, int(3e8 // (2 * experts * ff * width)) + 1))]
    us = _time([lambda w=w: ops.moe_gemm(xs[0], w, ids, True, dispatch) for w in wgu[:2]])
    out["moe_gate_up"] = _line(us, 0, 4 * rows * top * ff * width)
    act = ops.moe_gemm(xs[0], wgu[0], ids, True, dispatch)
    us = _time([lambda w=w: ops.moe_gemm(act, w, ids, False, dispatch) for w in wdn[:2]])
    out["moe_down"] = _line(us, 0, 2 * rows * top * ff * width)
    e = ops.moe_gemm(act, wdn[0], ids, False, dispatch)
    del act
    qgu, qdn = _randn(2 * s["ff"], width), _randn(width, s["ff"])
    us = _time([lambda a=a: ops.silu_mul(F.linear(a, qgu)) for a in xs])
    out["qwen_gate_up (product + silu_mul)"] = _line(us, 0, 4 * rows * s["ff"] * width)
    t = _randn(rows, s["ff"])
    out["qwen_down"] = _line(_time([lambda: F.linear(t, qdn)] * 2), 0, 2 * rows * s["ff"] * width)
    del t
    # ---- residual and norm
    st, w32 = _randn(rows, width, dtype=torch.float32), torch.ones(width, device="cuda")
    us = _time([lambda a=a: ops.residual_norm(st, torch.bfloat16, y=a, experts=(e, ew), weight=w32, bias=w32, eps=1e-6) for a in xs])
    out["residual_norm"] = _line(us, rows * width * (8 + 2 + 2 * top + 2))
    rs, wb = _randn(rows, width), _randn(width)
    out["qwen_add_rmsnorm"] = _line(_time([lambda a=a: ops.add_rmsnorm(a, wb, 1e-6, rs) for a in xs]), rows * width * 8)
    del xs, st, rs, e
    # ---- experts, decode batch
    x1 = _randn(batch, width)
    ids, _ = ops.moe_route(x1, router, corr, top, 8, 4, 2.5)
    used = ids.unique().numel()
    us = _time([lambda w=w: ops.moe_gemm(x1, w, ids, True) for w in wgu] * 3)
    out["moe_gate_up_decode"] = _line(us, used * 4 * ff * width)
    a1 = ops.moe_gemm(x1, wgu[0], ids, True)
    us = _time([lambda w=w: ops.moe_gemm(a1, w, ids, False) for w in wdn] * 3)
    out["moe_down_decode"] = _line(us, used * 2 * ff * width)
    del wgu, wdn
    ws = torch.zeros(max(ops.linear_workspace_bytes(batch, 2 * s["ff"], width, "silu_mul"), ops.linear_workspace_bytes(batch, width, s["ff"]), 16), dtype=torch.uint8, device="cuda")
    xp, mid = ops.pack_rows(x1), torch.zeros((batch + 15) // 16 * 16 * s["ff"], dtype=torch.bfloat16, device="cuda")
    qgus = [_randn(2 * s["ff"], width) for _ in range(int(3e8 // (4 * s["ff"] * width)) + 2)]
    us = _time([lambda w=w: ops.fused_linear(xp, w, x_packed_rows=batch, epilogue="silu_mul", out_packed=mid, want_out=False, workspace=ws) for w in qgus] * 2)
    out["qwen_gate_up_decode"] = _line(us, 4 * s["ff"] * width)
    del qgus
    qdns = [_randn(width, s["ff"]) for _ in range(int(3e8 // (2 * s["ff"] * width)) + 2)]
    us = _time([lambda w=w: ops.fused_linear(mid, w, x_packed_rows=batch, workspace=ws) for w in qdns] * 2)
    out["qwen_down_decode"] = _line(us, 2 * s["ff"] * width)
    us = _time([lambda: ops.moe_route(x1, router, corr, top, 8, 4, 2.5)] * 20)
    out["moe_route_decode"] = _line(us, 2 * (batch + experts) * width)
    torch.cuda.empty_cache()
    return out


@torch.inference_mode()
def zobasun_kernels(size, batch=32, ctx=1536, seqs=16, prompt=1024):
    """Each hot kernel of the two models alone; operands cycle through more than the memory-side cache holds where that matters."""
    s, out = SIZES[size], qwen_attention(size, batch, ctx, seqs, prompt)
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
    del q, k, v
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


@torch.inference_mode()
def kekapel_kernels(size, batch=32, ctx=1536, seqs=16, prompt=1024):
    """Each hot kernel of Kekapel alone, and on the same operands the like kernels of Galirax (paged attention, prep, residual, experts) and of the Qwen stack."""
    s, out, rows = SIZES[size], {}, seqs * prompt
    h, g, d, width, experts, top = s["heads"], s["kv_heads"], 128, s["width"], s["experts"], s["top"]
    ff, cap, scale = s["ff"] // top, 20.0, d ** -0.5
    cu = torch.arange(0, rows + 1, prompt, dtype=torch.int32, device="cuda")
    pos = torch.arange(prompt, device="cuda").repeat(seqs)
    talk = torch.eye(h, device="cuda") + 0.1 * _randn(h, h, dtype=torch.float32)
    # ---- attention over prompts, row ops in front
    cols = (h + 2 * g) * d
    qkv = [_randn(rows, cols) for _ in range(3)]
    cache = torch.zeros(rows // 64, 64, 2 * g * d, dtype=torch.bfloat16, device="cuda")
    slot = torch.arange(rows, dtype=torch.int32, device="cuda")
    one, qw, kw = torch.ones(d, device="cuda"), torch.ones(h * d, device="cuda"), torch.ones(g * d, device="cuda")
    us = _time([lambda x=x: ops.attn_prep(x, h, g, d, d, pos, None, cache, slot, one, one, d, d, 1e-6, head_norm=True) for x in qkv])
    out["attn_prep, norm per head"] = _line(us, rows * 4 * cols)
    us = _time([lambda x=x: ops.attn_prep(x, h, g, d, d, pos, None, cache, slot, qw, kw, h * d, g * d, 1e-6) for x in qkv])
    out["galirax attn_prep"] = _line(us, rows * 4 * cols)
    bt = torch.arange(rows // 64, dtype=torch.int32, device="cuda").view(seqs, -1)
    o = torch.empty(rows, h * d, device="cuda", dtype=torch.bfloat16)
    nbytes = 4 * rows * (h + g) * d
    for name, window in (("prompt", 0), (f"prompt, window {WINDOW}", WINDOW)):
        seen = seqs * (sum(min(t + 1, window) for t in range(prompt)) if window else prompt * (prompt + 1) / 2)
        us = _time([lambda x=x: ops.talk_prompt(x, cache, bt, cu, cu, prompt, h, g, d, d, scale, talk, cap, window=window, out=o) for x in qkv] * 2)
        out[f"talk_{name}"] = _line(us, nbytes, (4 * d + 2 * h) * h * seen)
        us = _time([lambda x=x: ops.paged_attend_prompt(x, cache, bt, cu, cu, prompt, h, g, d, d, scale, window=window, out=o) for x in qkv] * 2)
        out[f"galirax paged_{name}"] = _line(us, nbytes, 4 * d * h * seen)
    del qkv, o, cache
    # ---- decode attention
    pages = -(-ctx // 64)
    n = max(2, int(3e8 // (batch * pages * 64 * 4 * g * d)) + 1)
    caches = [_randn(batch * pages, 64, 2 * g * d) for _ in range(n)]
    bt = torch.randperm(batch * pages).view(batch, pages).int().cuda()
    dpos = torch.full((batch,), ctx - 1, device="cuda")
    q, o = _randn(batch, h * d), torch.empty(batch, h * d, device="cuda", dtype=torch.bfloat16)
    for name, window in (("rows", 0), (f"rows, window {WINDOW}", WINDOW)):
        nbytes = batch * (4 * (window or ctx) * g * d + 4 * h * d)
        us = _time([lambda c=c: ops.talk_rows(q, c, bt, dpos, h, g, d, d, scale, ctx, talk, cap, window=window, out=o) for c in caches] * 3)
        out[f"talk_{name} (scores + rows)"] = _line(us, nbytes)
        us = _time([lambda c=c: ops.paged_attend_rows(q, c, bt, dpos, h, g, d, d, scale, ctx, window=window, out=o) for c in caches] * 3)
        out[f"galirax paged_{name}"] = _line(us, nbytes)
    del caches
    # ---- feed-forwards
    xs, router, bias = [_randn(rows, width) for _ in range(2)], _randn(experts, width) * width ** -0.5, torch.zeros(experts, device="cuda")
    z, coef = [_randn(rows, s["ff"]) for _ in range(2)], torch.ones(4, device="cuda")
    out["poly_norm"] = _line(_time([lambda t=t: ops.poly_norm(t, coef, 1e-6, s["ff"]) for t in z] * 2), rows * s["ff"] * 4)
    gu = [_randn(rows, 2 * s["ff"]) for _ in range(2)]
    out["qwen_silu_mul"] = _line(_time([lambda t=t: ops.silu_mul(t) for t in gu]), rows * s["ff"] * 6)
    del z, gu
    us = _time([lambda a=a: ops.moe_route(a, router, bias, top, softmax=True) for a in xs] * 2)
    out["moe_route, softmax"] = _line(us, 2 * rows * width, 2 * rows * width * experts)
    us = _time([lambda a=a: ops.moe_route(a, router, bias, top, 8, 4, 2.5) for a in xs] * 2)
    out["galirax moe_route"] = _line(us, 2 * rows * width, 2 * rows * width * experts)
    ids, ew = ops.moe_route(xs[0], router, bias, top, softmax=True)
    dispatch, unit = ops.moe_dispatch(ids, experts, torch.bfloat16), (7.0, 1.702)
    wgu = [_randn(experts, 2 * ff, width) * 0.02 for _ in range(2)]
    for name, u in (("moe_gate_up, clamped unit", unit), ("galirax moe_gate_up", None)):
        out[name] = _line(_time([lambda w=w: ops.moe_gemm(xs[0], w, ids, True, dispatch, u) for w in wgu]), 0, 4 * rows * top * ff * width)
    e, st, w32 = _randn(rows * top, width), _randn(rows, width, dtype=torch.float32), torch.ones(width, device="cuda")
    norm = dict(weight=w32, bias=w32, eps=1e-6)
    for name, kw in (("residual_norm, both sides", dict(post=(w32, w32), mult=0.7)), ("galirax residual_norm", {})):
        us = _time([lambda a=a: ops.residual_norm(st, torch.bfloat16, y=a, **norm, **kw) for a in xs])
        out[f"{name}, attention"] = _line(us, rows * width * (8 + 2 + 2))
        us = _time([lambda: ops.residual_norm(st, torch.bfloat16, experts=(e, ew), **norm, **kw)] * 2)
        out[f"{name}, experts"] = _line(us, rows * width * (8 + 2 * top + 2))
    del e, st, xs
    # ---- decode batch
    x1 = _randn(batch, width)
    ids, _ = ops.moe_route(x1, router, bias, top, softmax=True)
    used = ids.unique().numel()
    wgu += [_randn(experts, 2 * ff, width) * 0.02 for _ in range(max(0, int(3e8 // (4 * experts * ff * width)) - 1))]
    for name, u in (("moe_gate_up_decode, clamped unit", unit), ("galirax moe_gate_up_decode", None)):
        out[name] = _line(_time([lambda w=w: ops.moe_gemm(x1, w, ids, True, None, u) for w in wgu] * 3), used * 4 * ff * width)
    del wgu
    for name, kw in (("moe_route_decode, softmax", dict(softmax=True)), ("galirax moe_route_decode", dict(groups=8, keep=4, scale=2.5))):
        out[name] = _line(_time([lambda: ops.moe_route(x1, router, bias, top, **kw)] * 20), 2 * (batch + experts) * width)
    z = _randn(batch, s["ff"])
    packed = torch.zeros((batch + 15) // 16 * 16 * s["ff"], dtype=torch.bfloat16, device="cuda")
    out["poly_norm_decode"] = _line(_time([lambda: ops.poly_norm(z, coef, 1e-6, s["ff"], packed=packed)] * 20), batch * s["ff"] * 4)
    torch.cuda.empty_cache()
    return out


@torch.inference_mode()
def zaposun_kernels(size, batch=32, ctx=1536, seqs=16, prompt=1024):
    """Each hot kernel of Zaposun alone, and on operands of the same size the like kernels of Galirax (lightning attention, windowed attention, prep, residual), of
    Zobasun (recurrence) and of the Qwen stack."""
    s, out, rows = SIZES[size], {}, seqs * prompt
    h, g, d, width, ff = s["heads"], s["kv_heads"], 128, s["width"], s["ff"]
    cu = torch.arange(0, rows + 1, prompt, dtype=torch.int32, device="cuda")
    pos = torch.arange(prompt, device="cuda").repeat(seqs)
    slots = torch.arange(max(seqs, batch), dtype=torch.int32, device="cuda")
    row_seq = torch.arange(seqs, dtype=torch.int32, device="cuda").repeat_interleave(prompt)
    dpos = torch.full((batch,), ctx - 1, device="cuda")
    many = StepMeta(0, None, None, slots[:seqs], None, 64, False, prompt, row_seq, cu)
    single = StepMeta(batch, None, None, slots[:batch], None, 64, False, ctx)
    f32, one = torch.float32, torch.ones(width, device="cuda")

    def segments(units):
        seg = choose_segment([prompt] * seqs, units)
        return torch.tensor([c for i in range(seqs) for c in recurrence_chunks(i * prompt, prompt, i, seg)], dtype=torch.int32, device="cuda"), seg < prompt
    # ---- residual streams, shifts
    ys = [_randn(rows, width) for _ in range(3)]
    mix, vec, w32 = torch.eye(STREAMS, device="cuda"), torch.full((STREAMS,), 0.3, device="cuda"), (one, 2, 1e-6)
    xs = [_randn(rows, STREAMS, width, dtype=f32)]
    us = _time([lambda y=y: ops.stream_mix(xs[0], STREAMS, torch.bfloat16, width, dict(y=y, mix=mix, out=vec), vec, w32) for y in ys])
    out["stream_mix"] = _line(us, rows * width * (8 * STREAMS + 4))
    us = _time([lambda y=y: ops.stream_mix(xs[0], STREAMS, torch.bfloat16, width, dict(y=y, mix=mix, out=vec, eps=1e-6, post=(ys[0], one, one, 0.5)), vec, w32) for y in ys[1:]])
    out["stream_mix, two mixers"] = _line(us, rows * width * (8 * STREAMS + 6))
    st = xs.pop()[:, 0].contiguous()
    us = _time([lambda y=y: ops.residual_norm(st, torch.bfloat16, y=y, weight=one, bias=one, eps=1e-6) for y in ys])
    out["galirax residual_norm"] = _line(us, rows * width * 12)
    ring, mu = torch.zeros(max(seqs, batch), 3, width, device="cuda", dtype=torch.bfloat16), torch.rand(5, width, device="cuda")
    us = _time([lambda y=y: ops.token_shift(y, pos, many, one, ring, mu) for y in ys])
    out["token_shift, five mixes"] = _line(us, rows * width * 12)
    ring2 = torch.zeros(max(seqs, batch), 2, width, device="cuda", dtype=torch.bfloat16)
    us = _time([lambda y=y: ops.token_shift(y, pos, many, one, ring2) for y in ys])
    out["token_shift"] = _line(us, rows * width * 4)
    x1 = [_randn(batch, STREAMS, width, dtype=f32) for _ in range(4)]
    y1, pk = _randn(batch, width), torch.zeros((batch + 15) // 16 * 16 * width * 5, dtype=torch.bfloat16, device="cuda")
    us = _time([lambda x=x: ops.stream_mix(x, STREAMS, torch.bfloat16, width, dict(y=y1, mix=mix, out=vec), vec, w32) for x in x1] * 5)
    out["stream_mix_decode"] = _line(us, batch * width * (8 * STREAMS + 4))
    sh = dict(positions=dpos, step=single, shift=one, ring=ring, mu=mu, packed=pk)
    us = _time([lambda x=x: ops.stream_mix(x, STREAMS, torch.bfloat16, width, dict(y=y1, mix=mix, out=vec), vec, w32, want_rows=False, shift=sh) for x in x1] * 5)
    out["stream_mix_decode with five shifted mixes"] = _line(us, batch * width * (8 * STREAMS + 2 + 16))
    x1 = _randn(batch, width, dtype=f32)
    us = _time([lambda: ops.residual_norm(x1, torch.bfloat16, y=y1, weight=one, bias=one, eps=1e-6)] * 20)
    out["galirax residual_norm_decode"] = _line(us, batch * width * 12)
    del ys, st
    # ---- time mixing
    hw = width // 64
    x = [[_randn(rows, width) for _ in range(5)] for _ in range(2)]
    p = dict(w0=torch.rand(width, device="cuda") * 5 - 6, u=_randn(width, dtype=f32), norm=one, w2=_randn(width, 64) * 0.05)
    o = torch.empty(rows, width, device="cuda", dtype=torch.bfloat16)
    state = torch.zeros(max(seqs, batch), hw, 64, 64, device="cuda")
    chunks, more = segments(hw)
    us = _time([lambda a=a: ops.wkv_chunks(*a, p, 1e-6, 64, pos, slots, chunks, more, state, out=o) for a in x] * 2)
    out["wkv_chunks"] = _line(us, rows * 12 * width, 4 * rows * width * 64)
    x1 = [_randn(batch, width) for _ in range(4)]
    z1 = _randn(batch, 64)
    states = [torch.zeros(batch, hw, 64, 64, device="cuda") for _ in range(max(2, int(3e8 // (4 * batch * width * 64)) + 1))]
    us = _time([lambda t=t: ops.wkv_step(*x1, z1, p, 1e-6, 64, dpos, slots, t) for t in states] * 3)
    out["wkv_step"] = _line(us, 8 * batch * width * 64)
    del x, states, state
    x = [_randn(rows, 4 * h * d) for _ in range(2)]
    decay, state = torch.linspace(0.8, 0.999, h, device="cuda"), torch.zeros(max(seqs, batch), h, d, d, device="cuda")
    o = torch.empty(rows, h * d, device="cuda", dtype=torch.bfloat16)
    chunks, more = segments(h * 2)
    us = _time([lambda a=a: ops.lightning_chunks(a, decay, pos, slots, chunks, more, state, out=o) for a in x] * 2)
    out["galirax lightning_chunks"] = _line(us, rows * 8 * h * d, 4 * rows * h * d * d)
    x1 = _randn(batch, 4 * h * d)
    states = [torch.zeros(batch, h, d, d, device="cuda") for _ in range(max(2, int(3e8 // (4 * batch * h * d * d)) + 1))]
    us = _time([lambda t=t: ops.lightning_step(x1, decay, dpos, slots, t) for t in states] * 3)
    out["galirax lightning_step"] = _line(us, 8 * batch * h * d * d)
    del x, states, state
    # ---- scan
    inner, rank = 2 * width, width // 16
    xz = [_randn(rows, 2 * inner) for _ in range(2)]
    conv, bias, cring = _randn(TAPS, inner, dtype=f32), _randn(inner, dtype=f32), torch.zeros(max(seqs, batch), TAPS, inner, device="cuda", dtype=torch.bfloat16)
    us = _time([lambda a=a: ops.causal_conv(a[:, :inner], pos, many, conv, bias, cring) for a in xz] * 2)
    out["causal_conv"] = _line(us, rows * inner * 4)
    dt, bc = _randn(rows, inner), _randn(rows, 64)
    p = dict(a_log2=-torch.rand(inner, STATES, device="cuda") * 4, d=torch.ones(inner, device="cuda"), dt_bias=torch.rand(inner, device="cuda") * 4 - 5, w_dt=_randn(inner, (rank + 63) // 64 * 64) * 0.1)
    o = torch.empty(rows, inner, device="cuda", dtype=torch.bfloat16)
    state = torch.zeros(max(seqs, batch), inner, STATES, device="cuda")
    chunks, more = segments(inner // 192)
    us = _time([lambda a=a: ops.scan_chunks(a[:, :inner], dt, bc, a[:, inner:], p, pos, slots, chunks, more, state, out=o) for a in xz] * 2)
    out["scan_chunks"] = _line(us, rows * inner * 8)
    x1, low, bc1 = _randn(batch, 2 * inner), _randn(batch, p["w_dt"].shape[1]), _randn(batch, 64)
    states = [torch.zeros(batch, inner, STATES, device="cuda") for _ in range(max(2, int(3e8 // (4 * batch * inner * STATES)) + 1))]
    us = _time([lambda t=t: ops.scan_step(x1[:, :inner], low, bc1, x1[:, inner:], p, dpos, slots, t) for t in states] * 3)
    out["scan_step"] = _line(us, batch * inner * (8 * STATES + 6) + 2 * p["w_dt"].numel())
    us = _time([lambda: ops.causal_conv(x1[:, :inner], dpos, single, conv, bias, cring)] * 20)
    out["causal_conv_decode"] = _line(us, batch * inner * 2 * (TAPS + 2))
    del xz, dt, o, states, state
    rec, blocks = s["rec"], s["blocks"]
    p = dict(conv_w=_randn(4, rec, dtype=f32), conv_b=_randn(rec, dtype=f32), ra=_randn(blocks, rec // blocks, rec // blocks) * 0.05, ri=_randn(blocks, rec // blocks, rec // blocks) * 0.05,
             ra_b=_randn(rec, dtype=f32), ri_b=_randn(rec, dtype=f32), rate=torch.rand(rec, device="cuda"))
    state, cring = torch.zeros(max(seqs, batch), rec, device="cuda"), torch.zeros(max(seqs, batch), 4, rec, dtype=torch.bfloat16, device="cuda")
    yx, o = [_randn(rows, 2 * rec) for _ in range(2)], torch.empty(rows, rec, device="cuda", dtype=torch.bfloat16)
    seg = choose_segment([prompt] * seqs, blocks)
    chunks, more = segments(blocks)
    us = _time([lambda a=a: ops.rglru_chunks(a, p, pos, slots, chunks, seg, more, state, cring, out=o) for a in yx] * 2)
    out["zobasun rglru_chunks"] = _line(us, rows * rec * 6, 4 * rows * rec * (rec // blocks))
    x1 = _randn(batch, 2 * rec)
    us = _time([lambda: ops.rglru_step(x1, p, dpos, slots, state, cring)] * 20)
    out["zobasun rglru_step"] = _line(us, 2 * (p["ra"].numel() + p["ri"].numel()) + batch * rec * 22)
    del yx, o, state, cring
    # ---- attention: values turned, chunks
    cols = (h + 2 * g) * d
    qkv = [_randn(rows, cols) for _ in range(3)]
    cache, slot = torch.zeros(rows // 64, 64, 2 * g * d, dtype=torch.bfloat16, device="cuda"), torch.arange(rows, dtype=torch.int32, device="cuda")
    head, qw, kw, table = torch.ones(d, device="cuda"), torch.ones(h * d, device="cuda"), torch.ones(g * d, device="cuda"), rotation_table(d, 10000.0, 4096, "cuda")
    us = _time([lambda a=a: ops.attn_prep(a, h, g, d, d, pos, table, cache, slot, head, head, d, d, 1e-6, head_norm=True, v_cos_sin=table) for a in qkv])
    out["attn_prep, values turned"] = _line(us, rows * 4 * cols)
    us = _time([lambda a=a: ops.attn_prep(a, h, g, d, d, pos, table, cache, slot, qw, kw, h * d, g * d, 1e-6) for a in qkv])
    out["galirax attn_prep"] = _line(us, rows * 4 * cols)
    bt, o = torch.arange(rows // 64, dtype=torch.int32, device="cuda").view(seqs, -1), torch.empty(rows, h * d, device="cuda", dtype=torch.bfloat16)
    for name, mask, seen in (("paged_prompt, chunks, values turned", dict(chunk=WINDOW, turn=table), sum(t % WINDOW + 1 for t in range(prompt))),
                             ("galirax paged_prompt, window", dict(window=WINDOW), sum(min(t + 1, WINDOW) for t in range(prompt)))):
        us = _time([lambda a=a: ops.paged_attend_prompt(a, cache, bt, cu, cu, prompt, h, g, d, d, d ** -0.5, out=o, **mask) for a in qkv] * 2)
        out[name] = _line(us, 4 * rows * (h + g) * d, 4 * d * h * seqs * seen)
    del qkv, cache, o
    pages = -(-ctx // 64)
    n = max(2, int(3e8 // (batch * pages * 64 * 4 * g * d)) + 1)
    caches, bt = [_randn(batch * pages, 64, 2 * g * d) for _ in range(n)], torch.randperm(batch * pages).view(batch, pages).int().cuda()
    q, o = _randn(batch, h * d), torch.empty(batch, h * d, device="cuda", dtype=torch.bfloat16)
    for name, mask in (("paged_rows, chunks, values turned", dict(chunk=WINDOW, turn=table)), ("galirax paged_rows, window", dict(window=WINDOW))):      # (a full chunk)
        us = _time([lambda c=c: ops.paged_attend_rows(q, c, bt, dpos, h, g, d, d, d ** -0.5, ctx, out=o, **mask) for c in caches] * 3)
        out[name] = _line(us, batch * (4 * WINDOW * g * d + 4 * h * d))
    del caches
    # ---- feed-forward, grouped projection
    gu = [_randn(rows, 2 * ff) for _ in range(2)]
    out["gelu_glu"] = _line(_time([lambda t=t: ops.gelu_glu(t) for t in gu]), rows * ff * 6)
    out["qwen silu_mul"] = _line(_time([lambda t=t: ops.silu_mul(t) for t in gu]), rows * ff * 6)
    del gu
    xp = ops.pack_rows(_randn(batch, width))
    for name, glu, n in (("gate_up_decode, gelu", "gelu", 2 * ff), ("qwen gate_up_decode", None, 2 * ff)):
        ws = torch.zeros(max(16, ops.linear_workspace_bytes(batch, n, width, "silu_mul")), dtype=torch.uint8, device="cuda")
        mid = torch.zeros((batch + 15) // 16 * 16 * ff, dtype=torch.bfloat16, device="cuda")
        ww = [_randn(n, width) for _ in range(int(3e8 // (2 * n * width)) + 2)]
        us = _time([lambda w=w: ops.fused_linear(xp, w, x_packed_rows=batch, epilogue="silu_mul", out_packed=mid, want_out=False, workspace=ws, glu=glu) for w in ww] * 2)
        out[name] = _line(us, 2 * n * width)
    n = 4 * width + 64
    ws = torch.zeros(max(16, ops.linear_workspace_bytes(batch, n, width)), dtype=torch.uint8, device="cuda")
    ww = [_randn(n, width) for _ in range(int(3e8 // (2 * n * width)) + 2)]
    us = _time([lambda w=w: ops.fused_linear(pk, w, x_packed_rows=batch, workspace=ws, x_groups=(5, width)) for w in ww] * 2)
    out["projection of five inputs, decode"] = _line(us, 2 * n * width)
    us = _time([lambda w=w: ops.fused_linear(xp, w, x_packed_rows=batch, workspace=ws) for w in ww] * 2)
    out["projection of one input, decode"] = _line(us, 2 * n * width)
    torch.cuda.empty_cache()
    return out


MODELS = {"zobasun": (zobasun_config, zobasun_kernels), "galirax": (galirax_config, galirax_kernels), "kekapel": (kekapel_config, kekapel_kernels),
          "zaposun": (zaposun_config, zaposun_kernels)}


def run(size, only=None, model="zobasun"):
    torch.manual_seed(0)
    config, kernels = MODELS[model]
    beside = [("qwen", qwen_config(size))]
    if model == "kekapel":
        beside.append(("galirax", galirax_config(size, windows_only=True)))
    if model == "zaposun":
        beside.append(("zobasun", zobasun_config(size)))
    stacks = [(model, config(size)), *beside]
    res = {"metric": f"{stacks[0][1].name} beside a Qwen2-shaped stack of equal width, depth and feed-forward (random weights)", "size": size, "shape": SIZES[size], "dtype": "bf16"}
    if only in (None, "kernels"):
        res["kernels"] = kernels(size)
    if only in (None, "engine"):
        for batch, prompt in ((16, 1024), (2, 8192)):
            for name, cfg in stacks:
                res[f"{name}_{batch}x{prompt}"] = _engine_throughput(cfg, batch, prompt, 64)
        for name, cfg in stacks:
            res[f"{name}_32x1024"] = _engine_throughput(cfg, 32, 1024, 256, repeats=1)
    return res
