"""Host side of the Zobasun model on the CPU: configuration, registry, checkpoint, step metadata, scheduler and state slots — and the plain
reference itself (oracle/zobasun_ref.py) against closed forms, with planted mistakes that must show."""
import copy
import json
import math
import os

import pytest
import torch

from oracle import zobasun_ref as Z
from zobasun_cases import CONFIGS, config, latent, recurrent, save_checkpoint, tokens, weights


# ------------------------------------------------------------------------------------------------ reference
def test_reference_recurrence_closed_form():
    """Constant gates: S_t = b (1 - a^t) / (1 - a)."""
    lam, r, i, u = torch.tensor([-2.0, 0.5], dtype=torch.float64), 0.3, 0.6, 1.7
    ones = torch.ones(40, 2, dtype=torch.float64)
    s, last = Z.rglru_recurrence(u * ones, r * ones, i * ones, lam)
    a = torch.exp(-8 * r * torch.log(1 + torch.exp(lam)))
    t = torch.arange(1, 41, dtype=torch.float64)[:, None]
    assert torch.allclose(s, torch.sqrt(1 - a * a) * i * u * (1 - a ** t) / (1 - a), rtol=1e-12)
    assert torch.equal(last, s[-1])


def test_reference_rotation_depends_on_distance_only():
    g = torch.Generator().manual_seed(0)
    q, k = torch.randn(1, 16, generator=g, dtype=torch.float64), torch.randn(1, 16, generator=g, dtype=torch.float64)

    def score(i, j):
        return (Z.rotate_pairs(q, torch.tensor([i]), 12, 900.0) * Z.rotate_pairs(k, torch.tensor([j]), 12, 900.0)).sum().item()
    assert math.isclose(score(70, 3), score(167, 100), rel_tol=1e-12)
    assert not math.isclose(score(70, 3), score(70, 4), rel_tol=1e-6)
    x = Z.rotate_pairs(q, torch.tensor([5]), 12, 900.0)
    assert torch.equal(x[:, 12:], q[:, 12:]) and torch.allclose(x.norm(), q.norm())


@pytest.mark.parametrize("plant", ["one_plus_w", "glu_shift", "rotation_halves", "first_token_gain", "conv_order", "scale", "kv_from"])
def test_planted_mistakes_show(monkeypatch, plant):
    """A reference with one equation wrong is far from the right one, so the comparisons of the GPU tests have teeth."""
    cfg, w = CONFIGS["odd"], weights("odd")
    toks = tokens(40, cfg["vocab"], 3)
    good = Z.forward(cfg, w, toks)
    if plant == "one_plus_w":
        monkeypatch.setattr(Z, "zero_centred_norm", lambda x, g, eps: Z.rms_norm(x, eps) * g)
    elif plant == "glu_shift":
        monkeypatch.setattr(Z, "clamped_glu", lambda g, u, lim: (lambda a: a * torch.sigmoid(1.702 * a) * u.clamp(-lim, lim))(g.clamp(max=lim)))
    elif plant == "rotation_halves":
        def halves(x, pos, dims, base):
            i = torch.arange(dims // 2)
            perm = torch.stack([i, i + dims // 2], 1).reshape(-1)
            y = x.clone()
            y[..., perm] = RP(x[..., perm], pos, dims, base)[..., :dims]
            return y
        RP = Z.rotate_pairs
        monkeypatch.setattr(Z, "rotate_pairs", halves)
    elif plant == "first_token_gain":
        rec = Z.rglru_recurrence

        def first(u, r, i, lam, state=None):
            s, last = rec(u, r, i, lam, i[0] * u[0])
            return s, last
        monkeypatch.setattr(Z, "rglru_recurrence", first)
    elif plant == "conv_order":
        conv = Z.causal_conv
        monkeypatch.setattr(Z, "causal_conv", lambda v, taps, bias: conv(v, taps.flip(1), bias))
    else:
        cfg = copy.deepcopy(cfg)
        if plant == "scale":
            cfg["layers"][2]["mixer"]["scale"] *= 1.5
        else:
            w = dict(w, **{"l2.mix.dkv": w["l0.mix.dkv"].flip(0), "l2.mix.dkv.norm": w["l0.mix.dkv.norm"]})
            del cfg["layers"][2]["mixer"]["kv_from"]
    bad = Z.forward(cfg, w, toks)
    assert (bad - good).pow(2).mean().sqrt() > 0.02 * good.pow(2).mean().sqrt()


# ------------------------------------------------------------------------------------------------ configuration, registry, checkpoint
def test_config_and_registry(tmp_path):
    from nanovllm_hip.models import REGISTRY, load_config, model_class
    from nanovllm_hip.models.zobasun import ZobasunConfig, ZobasunForCausalLM
    save_checkpoint(tmp_path, CONFIGS["odd"], {"x": torch.zeros(1)})
    cfg = load_config(str(tmp_path), dtype=torch.float32)
    assert isinstance(cfg, ZobasunConfig) and model_class(cfg) is ZobasunForCausalLM and cfg.dtype == torch.float32
    assert (cfg.hidden_size, cfg.vocab_size, cfg.num_hidden_layers, cfg.rms_norm_eps, cfg.embedding_scale) == (72, 101, 5, 1e-5, 3.0)
    assert {"Qwen2ForCausalLM", "Qwen3ForCausalLM"} <= set(REGISTRY)
    with open(os.path.join(tmp_path, "config.json"), "w") as f:
        json.dump({"architecture": "Nothing"}, f)
    with pytest.raises(ValueError, match="unknown architecture"):
        load_config(str(tmp_path))


@pytest.mark.parametrize("edit,match", [
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=4), "kv_from"),
    (lambda c: c["layers"][4]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][0].update(type="other"), "unknown mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="other"), "unknown feed-forward"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=8), "rot.dims"),
])
def test_config_refuses(edit, match):
    from nanovllm_hip.models.zobasun import ZobasunConfig
    cfg = copy.deepcopy(CONFIGS["odd"])
    edit(cfg)
    with pytest.raises(ValueError, match=match):
        ZobasunConfig.from_json(cfg)


def test_qwen_hf_config_and_weights(tmp_path):
    """The registry's other family: Hugging Face names land in the fused projections."""
    from nanovllm_hip.models import build_model, load_config
    from safetensors.torch import save_file
    hf = dict(architectures=["Qwen3ForCausalLM"], num_hidden_layers=1, hidden_size=128, num_attention_heads=4, num_key_value_heads=2, head_dim=64,
              intermediate_size=192, vocab_size=50, tie_word_embeddings=True, rope_theta=5e5)
    with open(os.path.join(tmp_path, "config.json"), "w") as f:
        json.dump(hf, f)
    g = torch.Generator().manual_seed(0)
    p = "model.layers.0."
    shapes = {"model.embed_tokens.weight": (50, 128), "model.norm.weight": (128,), p + "self_attn.q_proj.weight": (256, 128), p + "self_attn.k_proj.weight": (128, 128),
              p + "self_attn.v_proj.weight": (128, 128), p + "self_attn.o_proj.weight": (128, 256), p + "self_attn.q_norm.weight": (64,), p + "self_attn.k_norm.weight": (64,),
              p + "mlp.gate_proj.weight": (192, 128), p + "mlp.up_proj.weight": (192, 128), p + "mlp.down_proj.weight": (128, 192),
              p + "input_layernorm.weight": (128,), p + "post_attention_layernorm.weight": (128,)}
    w = {k: torch.randn(s, generator=g) for k, s in shapes.items()}
    save_file(w, os.path.join(tmp_path, "model.safetensors"))
    cfg = load_config(str(tmp_path))
    assert cfg.qk_norm and not cfg.qkv_bias and cfg.rope_theta == 5e5
    layer = build_model(cfg, str(tmp_path)).layers[0]
    assert torch.equal(layer.self_attn.qkv_proj.weight[256:384], w[p + "self_attn.k_proj.weight"])
    assert torch.equal(layer.mlp.gate_up_proj.weight[192:], w[p + "mlp.up_proj.weight"])
    assert torch.equal(layer.self_attn.k_norm.weight, w[p + "self_attn.k_norm.weight"])


def test_checkpoint_tensors_all_read_and_padding_is_zero(tmp_path, recwarn):
    from nanovllm_hip.models import build_model, load_config
    save_checkpoint(tmp_path, CONFIGS["odd"], weights("odd"))
    m = build_model(load_config(str(tmp_path), dtype=torch.float32), str(tmp_path))
    assert not [w for w in recwarn.list if "no layer" in str(w.message)]
    rec, att = m.layers[1].mixer, m.layers[0].mixer
    assert rec.cols % 64 == 0 and rec.block % 32 == 0 and rec.cols == rec.block * 3
    used = torch.zeros(3, rec.block, dtype=torch.bool)
    used[:, :44] = True
    unused = ~used.reshape(-1)
    assert rec.w_yx[:rec.cols][unused].abs().sum() == 0 and rec.w_o[:, unused].abs().sum() == 0
    assert torch.equal(rec.w_yx[rec.cols:, :72][used.reshape(-1)], weights("odd")["l1.mix.x"].float())
    assert torch.equal(att.w_uk[1, :36, :20], weights("odd")["l0.mix.uk"].float()[20:40].t())
    assert m.layers[2].mixer.cache_row() is None and m.layers[2].mixer._source[0] is att
    assert m.head.shape[0] % 64 == 0 and m.head[101:].abs().sum() == 0
    del m
    w = {k: v for k, v in weights("odd").items() if k != "l3.mix.lam"}
    save_checkpoint(tmp_path, CONFIGS["odd"], w)
    with pytest.raises(KeyError, match="l3.mix.lam"):
        build_model(load_config(str(tmp_path)), str(tmp_path))
    save_checkpoint(tmp_path, CONFIGS["odd"], dict(weights("odd"), stray=torch.zeros(2)))
    with pytest.warns(UserWarning, match="stray"):
        build_model(load_config(str(tmp_path)), str(tmp_path))


# ------------------------------------------------------------------------------------------------ step metadata
def _seq(n, cached, blocks, slot, bs=64):
    from nanovllm_hip.engine.sequence import Sequence
    s = Sequence(list(range(n)), block_size=bs)
    s.num_cached_tokens, s.block_table, s.state_slot = cached, blocks, slot
    return s


def test_step_meta_orders_single_tokens_first():
    from nanovllm_hip.engine.model_runner import build_step_meta
    a, b, c = _seq(130, 0, [4, 1, 7], 2), _seq(66, 65, [0, 3], 0), _seq(70, 63, [9, 5], 1)
    m = build_step_meta([(a, 130), (b, 1), (c, 7)], 64, 64)
    assert m["order"] == [1, 0, 2] and m["num_decode"] == 1
    assert m["positions"].tolist() == [65] + list(range(130)) + list(range(63, 70))
    assert m["input_ids"].tolist() == m["positions"].tolist()
    assert m["slot_mapping"][0] == 3 * 64 + 1 and m["slot_mapping"][1] == 4 * 64 and m["slot_mapping"][130] == 7 * 64 + 1
    assert m["slot_mapping"][131:].tolist() == [9 * 64 + 63] + [5 * 64 + k for k in range(6)]
    assert m["chunks"].tolist() == [[0, 1, 0, 0], [1, 64, 1, 0], [65, 64, 1, 1], [129, 2, 1, 2], [131, 7, 2, 0]]
    assert m["cu_q"].tolist() == [0, 130, 137] and m["cu_k"].tolist() == [0, 130, 200] and (m["max_q"], m["total_k"], m["max_context"]) == (130, 200, 130)
    assert m["state_slots"].tolist() == [0, 2, 1] and m["row_seq"].tolist() == [0] + [1] * 130 + [2] * 7
    assert m["block_tables"].tolist() == [[0, 3, 0], [4, 1, 7], [9, 5, 0]]


def test_step_meta_refuses_tokens_without_pages():
    from nanovllm_hip.engine.model_runner import build_step_meta
    with pytest.raises(AssertionError):
        build_step_meta([(_seq(70, 0, [1], 0), 70)], 64)


def test_segment_choice():
    from nanovllm_hip.layers.rglru import choose_segment
    assert choose_segment([1024] * 32, 16) == 1024                # enough workgroups: one walk each
    assert choose_segment([8192], 10) <= 512 and choose_segment([2], 4) == 64 and choose_segment([], 4) == 64
    assert all(choose_segment([n] * m, b) % 64 == 0 for n in (63, 65, 1000, 30000) for m in (1, 7) for b in (1, 10))


# ------------------------------------------------------------------------------------------------ scheduler
def _scheduler(blocks, slots=4, mixed=True, **kw):
    from nanovllm_hip.engine.block_manager import BlockManager, StateSlots
    from nanovllm_hip.engine.scheduler import Scheduler
    return Scheduler(BlockManager(blocks, 64), StateSlots(slots), mixed=mixed, **kw)


def _drive(sch, seqs, limit=400):
    """Run the schedule with made-up tokens; returns the batches as (sequence index, tokens) lists."""
    log = []
    while sch.unfinished():
        batch = sch.schedule()
        log.append([(seqs.index(s), n) for s, n in batch])
        for s, n in batch:
            assert len(s.block_table) * 64 >= s.num_cached_tokens + n and s.state_slot >= 0
            s.num_cached_tokens += n
        for s, _ in batch:
            if s.num_cached_tokens == len(s):
                s.append_token(1)
                if s.finished:
                    sch.finish(s)
        live = [s for s in seqs if s.state_slot >= 0]
        assert len({s.state_slot for s in live}) == len(live)
        used = [b for s in live for b in s.block_table]
        assert len(set(used)) == len(used) and set(used) == sch.block_manager.used_block_ids
        assert len(log) < limit
    return log


def _mk(n, out):
    from nanovllm_hip.engine.sequence import Sequence
    return Sequence([1] * n, max_tokens=out, block_size=64)


def test_scheduler_mixes_portions_with_decoding():
    sch = _scheduler(64, max_num_batched_tokens=100)
    seqs = [_mk(30, 5), _mk(210, 3), _mk(5, 2)]
    for s in seqs:
        sch.add(s)
    log = _drive(sch, seqs)
    assert log[0] == [(0, 30), (1, 70)] and log[1] == [(0, 1), (1, 99)] and log[2] == [(0, 1), (1, 41), (2, 5)]
    assert all(s.finished for s in seqs) and all(sum(n for _, n in b) <= 100 for b in log)
    assert len(sch.block_manager.free_block_ids) == 64 and len(sch.state_slots.free) == 4


def test_scheduler_respects_slots_and_reuses_them():
    sch = _scheduler(64, slots=2)
    seqs = [_mk(10 + i, 3) for i in range(7)]
    for s in seqs:
        sch.add(s)
    log = _drive(sch, seqs)
    assert all(len(b) <= 2 for b in log) and all(s.finished for s in seqs)


def test_scheduler_preempts_the_youngest_and_finishes_everything():
    sch = _scheduler(4)
    seqs = [_mk(100, 60), _mk(60, 60)]
    for s in seqs:
        sch.add(s)
    log = _drive(sch, seqs)
    assert all(s.finished for s in seqs)
    assert any(b == [(1, n)] or (1, n) in b for b in log[1:] for n in range(61, 121)), "the younger sequence started over from its own tokens"


def test_scheduler_prefill_first_keeps_phases_apart():
    sch = _scheduler(64, mixed=False, max_num_batched_tokens=100)
    seqs = [_mk(60, 4), _mk(50, 4), _mk(30, 4)]
    for s in seqs:
        sch.add(s)
    log = _drive(sch, seqs)
    assert log[0] == [(0, 60)] and log[1] == [(1, 50), (2, 30)] and all(n == 1 for b in log[2:] for _, n in b)


def test_scheduler_reports_a_pool_too_small():
    sch = _scheduler(1)
    sch.add(_mk(100, 2))
    with pytest.raises(RuntimeError, match="out of memory"):
        sch.schedule()


def test_decoding_only_when_nothing_can_be_admitted():
    sch = _scheduler(8, slots=2)
    a, b, c = _mk(10, 9), _mk(10, 9), _mk(10, 9)
    for s in (a, b):
        sch.add(s)
    for s, n in sch.schedule():
        s.num_cached_tokens += n
        s.append_token(1)
    assert sch.decoding() == [a, b]
    sch.add(c)
    assert sch.decoding() == [a, b]                       # no slot for c
    sch.finish(b)
    assert sch.decoding() == []                           # c can come in now


def test_entry_points_refuse_bad_arguments():
    """The C ABI's own checks (no GPU): null descriptors, types, shapes."""
    import ctypes
    from nanovllm_hip import _lib
    lib = _lib.load()
    assert lib.nvh_rglru_chunks(None, 0, 0, None) == -5 and lib.nvh_latent_attention(None, 0, 0, None) == -5
    d = _lib.RglruDesc()
    assert lib.nvh_rglru_chunks(ctypes.byref(d), 0, 0, None) == 0                     # no chunks: nothing to do
    d.n_chunks = 1
    assert lib.nvh_rglru_chunks(ctypes.byref(d), 0, 7, None) == -1
    assert lib.nvh_rglru_chunks(ctypes.byref(d), 0, 0, None) == -5
    p = _lib.LatentPrefillDesc()
    p.batch, p.max_q = 1, 1
    assert lib.nvh_latent_prefill(ctypes.byref(p), 1, None) == -1 and lib.nvh_latent_prefill(ctypes.byref(p), 0, None) == -5
    assert lib.nvh_latent_prefill_supported(192, 128) and not lib.nvh_latent_prefill_supported(320, 128)
    assert lib.nvh_latent_attend_mfma(512, 64, 64) and not lib.nvh_latent_attend_mfma(640, 64, 64) and not lib.nvh_latent_attend_mfma(512, 64, 32)
    assert config(8, 8, [recurrent(8, 1, 1), latent(1, 8, 8, 8, 8, 8, 1.0)])["layers"][1]["mixer"]["heads"] == 1
