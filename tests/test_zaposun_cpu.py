"""Host side of the Zaposun model on the CPU: configuration, registry, checkpoint, state pools, step metadata — and the plain reference itself
(oracle/zaposun_ref.py) against closed forms, with planted mistakes that must show."""
import copy
import math

import pytest
import torch

from oracle import zaposun_ref as Z
from zaposun_cases import CONFIGS, config, parallel, weights, wkv
from zobasun_cases import save_checkpoint, tokens

F64 = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


# ------------------------------------------------------------------------------------------------ reference
def test_reference_group_norm_by_hand():
    x = torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=F64)
    w = torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=F64)
    got = Z.group_norm(x, w, 2, 0.5)
    a, b = math.sqrt(12.5 + 0.5), math.sqrt(2.0 + 0.5)
    assert torch.allclose(got, torch.tensor([[3 / a, 8 / a, 0.0, 8 / b]], dtype=F64))
    assert torch.allclose(Z.group_norm(rnd(3, 12), torch.ones(12, dtype=F64), 1, 0.1), Z.rms(rnd(3, 12), 0.1))


def test_reference_streams_by_hand():
    xs = torch.tensor([[[1.0]], [[10.0]]], dtype=F64)
    assert Z.read_streams(xs, torch.tensor([0.5, 0.25], dtype=F64)).item() == 3.0
    new = Z.update_streams(xs, torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=F64), torch.tensor([1.0, -1.0], dtype=F64), torch.tensor([[100.0]], dtype=F64))
    assert new.flatten().tolist() == [1 + 30 + 100, 2 + 40 - 100]


def test_reference_shift_and_bigram_rows():
    h = torch.tensor([[1.0], [3.0], [7.0]], dtype=F64)
    assert Z.lerp_previous(h, torch.tensor([0.25], dtype=F64)).flatten().tolist() == [0.75, 2.5, 6.0]
    assert Z.bigram_rows([4, 9, 9], 7, 3, 2) == [7, (12 + 18) % 7, (27 + 18) % 7]


def test_reference_time_mixing_sums_up():
    """With a constant decay the state is a geometric sum; the bonus counts for the token itself only."""
    r, k, v, u = rnd(5, 3), rnd(5, 3, seed=1), rnd(5, 2, seed=2), rnd(3, seed=3)
    d = torch.tensor([0.5, 1.0, 0.0], dtype=F64)
    o, s = Z.wkv_scan(r, k, v, d.expand(5, 3), u)
    for t in range(5):
        want = (r[t] * u * k[t]).sum() * v[t] + sum((r[t] * d ** (t - 1 - j) * k[j]).sum() * v[j] for j in range(t))
        assert torch.allclose(o[t], want)
    assert torch.allclose(s, sum(torch.outer(d ** (4 - j) * k[j], v[j]) for j in range(5)))
    o2, s2 = Z.wkv_scan(r[2:], k[2:], v[2:], d.expand(3, 3), u, Z.wkv_scan(r[:2], k[:2], v[:2], d.expand(2, 3), u)[1])
    assert torch.allclose(o2, o[2:]) and torch.allclose(s2, s)


def test_reference_rotation_turns_by_distance():
    q, k = rnd(1, 1, 12), rnd(1, 1, 12, seed=1)

    def score(i, j):
        return (Z.rotate_half(q, torch.tensor([i]), 8, 100.0) * Z.rotate_half(k, torch.tensor([j]), 8, 100.0)).sum()
    assert torch.allclose(score(7, 3), score(104, 100)) and not torch.allclose(score(7, 3), score(7, 4))
    x = Z.rotate_half(q, torch.tensor([1]), 8, 100.0)[0, 0]
    a = 100.0 ** (-2.0 / 8)
    assert torch.allclose(x[1], q[0, 0, 1] * math.cos(a) - q[0, 0, 5] * math.sin(a)) and torch.equal(x[8:], q[0, 0, 8:])
    assert torch.allclose(Z.rotate_half(Z.rotate_half(q, torch.tensor([9]), 12, 50.0), torch.tensor([-9]), 12, 50.0), q)


def test_reference_chunks():
    ok = Z.visible(10, 4)
    assert ok[3].nonzero().flatten().tolist() == [0, 1, 2, 3] and ok[4].nonzero().flatten().tolist() == [4] and ok[9].nonzero().flatten().tolist() == [8, 9]
    assert torch.equal(Z.visible(5, 1), torch.eye(5, dtype=torch.bool)) and torch.equal(Z.visible(5, 9), torch.ones(5, 5, dtype=torch.bool).tril())


def test_reference_conv_and_scan_by_hand():
    x, w = torch.tensor([[1.0], [2.0], [4.0]], dtype=F64), torch.tensor([[10.0, 1.0]], dtype=F64)
    assert Z.causal_conv(x, w, torch.tensor([0.5], dtype=F64)).flatten().tolist() == [1.5, 12.5, 24.5]
    dt, a = torch.tensor([[1.0], [2.0]], dtype=F64), torch.tensor([[-0.5]], dtype=F64)
    y, s = Z.selective_scan(x[:2], dt, a, torch.tensor([[3.0], [5.0]], dtype=F64), torch.tensor([[1.0], [2.0]], dtype=F64), torch.tensor([10.0], dtype=F64))
    want = math.exp(-1.0) * 3.0 + 2.0 * 2.0 * 5.0
    assert torch.allclose(y.flatten(), torch.tensor([3.0 + 10.0, 2 * want + 20.0], dtype=F64)) and torch.allclose(s, torch.tensor([[want]], dtype=F64))


def test_reference_units_by_hand():
    z = torch.tensor([-30.0, 0.0, 1.0, 30.0], dtype=F64)
    assert torch.allclose(Z.softplus(z), torch.tensor([math.exp(-30.0), math.log(2.0), math.log(1 + math.e), 30.0], dtype=F64), rtol=1e-6)
    assert torch.allclose(Z.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh")) and torch.allclose(Z.silu(z), torch.nn.functional.silu(z))


def replaced(name, make):
    """Plants: the reference's function `name` gives way to what `make` builds from it."""
    def plant(monkeypatch):
        monkeypatch.setattr(Z, name, make(getattr(Z, name)))
    return plant


def _no_bonus(f):
    return lambda r, k, v, d, u, state=None: f(r, k, v, d, torch.zeros_like(u), state)


def _bonus_in_the_state(f):
    return lambda r, k, v, d, u, state=None: f(r, k, v, d, torch.ones_like(u), state)


PLANTS = {
    "chunk one longer": replaced("visible", lambda f: lambda n, size: f(n, size + 1)),
    "window instead of chunk": replaced("visible", lambda f: lambda n, size: torch.ones(n, n, dtype=torch.bool).tril() & ~torch.ones(n, n, dtype=torch.bool).tril(-size)),
    "output not turned back": replaced("rotate_half", lambda f: lambda x, pos, dims, base: x if pos[-1] < 0 else f(x, pos, dims, base)),
    "neighbours turned": replaced("rotate_half", lambda f: lambda x, pos, dims, base: torch.cat([f(x[..., :dims].unflatten(-1, (dims // 2, 2)).transpose(-1, -2).flatten(-2), pos, dims, base)
                                  .unflatten(-1, (2, dims // 2)).transpose(-1, -2).flatten(-2), x[..., dims:]], -1)),
    "no bonus": replaced("wkv_scan", _no_bonus),
    "bonus of one": replaced("wkv_scan", _bonus_in_the_state),
    "decay without its outer exponential": replaced("wkv_decay", lambda f: lambda w, p, x: torch.sigmoid(-torch.log(-torch.log(f(w, p, x))))),
    "decay of the next token": replaced("wkv_decay", lambda f: lambda w, p, x: Z.previous(f(w, p, x))),
    "shift not applied": replaced("lerp_previous", lambda f: lambda h, mu: h),
    "shift the other way": replaced("lerp_previous", lambda f: lambda h, mu: Z.previous(h) + (h - Z.previous(h)) * mu),
    "first row its own predecessor": replaced("previous", lambda f: lambda h: torch.cat([h[:1], h[:-1]])),
    "streams read alike": replaced("read_streams", lambda f: lambda xs, w: f(xs, torch.full_like(w, w.mean().item()))),
    "mix transposed": replaced("update_streams", lambda f: lambda xs, mix, out, y: f(xs, mix.T, out, y)),
    "streams updated one after the other": replaced("update_streams", lambda f: lambda xs, mix, out, y: f(torch.cat([f(xs, mix, out, y)[:1], xs[1:]]), mix, out, y)),
    "one norm group": replaced("group_norm", lambda f: lambda x, w, groups, eps: f(x, w, 1, eps)),
    "no bigram": replaced("bigram_rows", lambda f: lambda toks, buckets, a, b: [buckets] * len(toks)),
    "bigram the other way round": replaced("bigram_rows", lambda f: lambda toks, buckets, a, b: f(toks, buckets, b, a)),
    "first token hashed": replaced("bigram_rows", lambda f: lambda toks, buckets, a, b: [toks[0] * b % buckets] + f(toks, buckets, a, b)[1:]),
    "convolution reversed": replaced("causal_conv", lambda f: lambda x, w, b: f(x, w.flip(1), b)),
    "no skip": replaced("selective_scan", lambda f: lambda x, dt, a, b, c, d, state=None: f(x, dt, a, b, c, torch.zeros_like(d), state)),
    "input not scaled by dt": replaced("selective_scan", lambda f: lambda x, dt, a, b, c, d, state=None: f(x / dt, dt, a, b, c, d, state)),
    "exact gelu": replaced("gelu_tanh", lambda f: torch.nn.functional.gelu),
}


@pytest.mark.parametrize("name", sorted(PLANTS))
def test_planted_mistakes_show(monkeypatch, name):
    """A reference with one equation wrong is far from the right one, so the comparisons of the GPU tests have teeth."""
    cfg, w = CONFIGS["odd"], weights("odd")
    toks = tokens(130, cfg["vocab"], 3)
    good = Z.forward(cfg, w, toks)
    PLANTS[name](monkeypatch)
    bad = Z.forward(cfg, w, toks)
    err = (bad - good).pow(2).mean(1).sqrt() / good.std()
    assert err.max() > (3 if name == "exact gelu" else 20) * 5e-5 and err.mean() > (1e-4 if name == "exact gelu" else 5e-4)


def _other_half(cfg, w):
    w["l0.mix.left.out"], w["l0.mix.right.out"] = w["l0.mix.right.out"], w["l0.mix.left.out"]


def _no_key_norm_weight(cfg, w):
    w["l0.mix.left.k.norm"] = torch.ones_like(w["l0.mix.left.k.norm"])


def _scale(cfg, w):
    cfg["layers"][0]["mixer"]["left"]["scale"] *= 1.5


def _base(cfg, w):
    cfg["layers"][0]["mixer"]["left"]["rot"]["base"] *= 2.0


def _mixes_swapped(cfg, w):
    w["l1.mix.mu.r"], w["l1.mix.mu.k"] = w["l1.mix.mu.k"], w["l1.mix.mu.r"]


def _second_connection_for_the_first(cfg, w):
    w["l0.hc1.out"] = w["l0.hc2.out"]


def _logit_scale(cfg, w):
    cfg["logit_scale"] *= 1.1


@pytest.mark.parametrize("edit", [_other_half, _no_key_norm_weight, _scale, _base, _mixes_swapped, _second_connection_for_the_first, _logit_scale], ids=lambda f: f.__name__[1:])
def test_planted_structure_shows(edit):
    cfg, w = copy.deepcopy(CONFIGS["odd"]), dict(weights("odd"))
    toks = tokens(60, cfg["vocab"], 3)
    good = Z.forward(cfg, w, toks)
    edit(cfg, w)
    assert (Z.forward(cfg, w, toks) - good).pow(2).mean().sqrt() > 0.005 * good.std()


# ------------------------------------------------------------------------------------------------ configuration, registry, checkpoint
def test_config_and_registry(tmp_path):
    from nanovllm_hip.models import load_config, model_class
    from nanovllm_hip.models.zaposun import ZaposunConfig, ZaposunForCausalLM
    save_checkpoint(tmp_path, CONFIGS["odd"], {"x": torch.zeros(1)})
    cfg = load_config(str(tmp_path), dtype=torch.float32)
    assert isinstance(cfg, ZaposunConfig) and model_class(cfg) is ZaposunForCausalLM and cfg.dtype == torch.float32
    assert (cfg.hidden_size, cfg.vocab_size, cfg.num_hidden_layers, cfg.norm_eps, cfg.norm_groups, cfg.streams, cfg.logit_scale) == (72, 101, 5, 1e-5, 3, 3, 0.7)
    assert cfg.bigram == {"buckets": 97, "mul_prev": 5, "mul_cur": 3}


@pytest.mark.parametrize("edit,match", [
    (lambda c: c["layers"][0].update(type="other"), "unknown mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="other"), "unknown feed-forward"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=22), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(vdim=13), "values of 13"),
    (lambda c: c["norm"].update(groups=5), "norm groups"),
    (lambda c: c.update(streams=17), "streams"),
])
def test_config_refuses(edit, match):
    from nanovllm_hip.models.zaposun import ZaposunConfig
    cfg = copy.deepcopy(CONFIGS["odd"])
    edit(cfg)
    with pytest.raises(ValueError, match=match):
        ZaposunConfig.from_json(cfg)


def test_too_many_states_are_refused():
    from nanovllm_hip.models.zaposun import ZaposunConfig, ZaposunForCausalLM
    with pytest.raises(ValueError, match="states"):
        ZaposunForCausalLM(ZaposunConfig.from_json(config(64, 10, [parallel(1, 1, 8, 8, 8, 5, 1.0, 8, 257, 4, 2)])))


def test_pairs_of_halves():
    from nanovllm_hip.layers.rotary import halves_to_pairs
    assert halves_to_pairs(9, 6).tolist() == [0, 3, 1, 4, 2, 5, 6, 7, 8] and halves_to_pairs(3, 0).tolist() == [0, 1, 2] and halves_to_pairs(4, 4).tolist() == [0, 2, 1, 3]


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_checkpoint_is_read_whole(name, tmp_path):
    """Every tensor lands somewhere, padding stays zero, and what the layers hold gives the reference's numbers back."""
    from nanovllm_hip.models import build_model, load_config
    from nanovllm_hip.utils import loader
    cfg, w = CONFIGS[name], weights(name)
    save_checkpoint(tmp_path, cfg, w)
    ckpt = loader.Checkpoint(str(tmp_path))
    c = load_config(str(tmp_path), dtype=torch.float32)
    model = build_model(c, str(tmp_path))
    type(model)(c).load_weights(ckpt)
    assert ckpt.unread() == []
    d = cfg["width"]
    assert torch.equal(model.embed.bigram[-1, :d], w["bigram"][-1].float()) and not model.embed.embed[:, d:].any()
    h = torch.zeros(3, model.cols)
    h[:, :d] = torch.randn(3, d)
    for i, layer in enumerate(model.layers):
        m, spec, p = layer.mixer, cfg["layers"][i], f"l{i}.mix."
        s = spec["mixer"]
        assert torch.equal(layer.shift.shift[:d], w[f"l{i}.shift"].float()) and not layer.norm1[d:].any() and torch.equal(layer.hc1.mix, w[f"l{i}.hc1.mix"].float())
        if spec["type"] == "wkv":
            rows = (h @ m.w_in.T)[:, m.cols:2 * m.cols][:, :m.head_cols].view(3, m.heads, m.dk)
            want = h[:, :d] @ w[p + "k"].float().T
            assert torch.allclose(rows[:, :, :s["dim"]].reshape(3, -1), want, atol=1e-4) and not rows[:, :, s["dim"]:].any()
            assert torch.equal(layer.shift.mu[4, :d], w[p + "mu.w"].float())
            y = torch.randn(3, s["heads"], s["dim"])
            full = torch.zeros(3, m.cols)
            full[:, :m.head_cols].view(3, m.heads, m.dk)[:, :, :s["dim"]] = y
            assert torch.allclose((full @ m.w_o.T)[:, :d], y.reshape(3, -1) @ w[p + "o"].float().T, atol=1e-4)
        else:
            a, b, cut = m.left, m.right, m.left.proj_cols
            proj = h @ m.w_in.T
            assert torch.allclose(proj[:, cut + b.inner_cols:cut + b.inner_cols + b.inner], h[:, :d] @ w[p + "right.in"].float()[b.inner:].T, atol=1e-4)
            q = proj[:, :a.q_cols].view(3, a.heads, a.dk)
            want = (h[:, :d] @ w[p + "left.q"].float().T).view(3, a.heads, a.dim)
            half = s["left"]["rot"]["dims"] // 2
            assert torch.allclose(q[:, :, 0:2 * half:2], want[:, :, :half], atol=1e-4) and torch.allclose(q[:, :, 1:2 * half:2], want[:, :, half:2 * half], atol=1e-4)
            assert torch.allclose(q[:, :, 2 * half:a.dim], want[:, :, 2 * half:], atol=1e-4) and not q[:, :, a.dim:].any()
            assert torch.allclose(b.a_log2[:b.inner, :b.states], -torch.exp(w[p + "right.A_log"].float()) * 1.442695, rtol=1e-5) and not b.a_log2[b.inner:].any()
        if spec["mlp"] is not None:
            assert torch.equal(layer.mlp.w_gate_up[layer.mlp.cols:layer.mlp.cols + layer.mlp.ff, :d], w[f"l{i}.mlp.up"].float())


def test_random_weights_are_deterministic():
    from nanovllm_hip.models import build_model
    from nanovllm_hip.models.zaposun import ZaposunConfig
    cfg = ZaposunConfig.from_json(CONFIGS["odd"])
    a, b = build_model(cfg, seed=3), build_model(cfg, seed=3)
    assert all(torch.equal(x, y) for x, y in zip(a.buffers(), b.buffers())) and abs(a.layers[0].norm1[:72].mean() - 1) < 0.02


def test_what_a_sequence_keeps():
    """Pages for attention, and per slot: the previous token, the shift's rows, both recurrent states, the convolution's inputs."""
    from nanovllm_hip.engine.model_runner import ModelRunner
    from nanovllm_hip.models.zaposun import ZaposunConfig
    r = ModelRunner(ZaposunConfig.from_json(CONFIGS["odd"]), 5, device="cpu", max_model_len=512, max_num_seqs=3)
    assert len(r.kv_cache) == 3 and all(c.shape[:3] == (1, 5, 64) for c in r.kv_cache)
    shapes = {k: (tuple(v.shape), v.dtype) for k, v in r.state.items()}
    assert shapes["embed.last_token"] == ((3,), torch.int64)
    assert shapes["layers.0.shift.ring"] == ((3, 2, 128), torch.bfloat16) and shapes["layers.1.shift.ring"] == ((3, 3, 128), torch.bfloat16)
    assert shapes["layers.1.mixer.state"] == ((3, 3, 64, 64), torch.float32)
    assert shapes["layers.0.mixer.right.state"] == ((3, 64, 8), torch.float32) and shapes["layers.0.mixer.right.conv_state"] == ((3, 3, 64), torch.bfloat16)


def test_step_meta_tells_every_row_its_portion():
    from nanovllm_hip.engine.model_runner import build_step_meta
    from nanovllm_hip.engine.sequence import Sequence
    seqs = [Sequence(list(range(n)), block_size=64) for n in (70, 5, 9)]
    for i, (s, c) in enumerate(zip(seqs, (66, 4, 0))):
        s.num_cached_tokens, s.block_table, s.state_slot = c, [2 * i, 2 * i + 1], i
    m = build_step_meta([(seqs[0], 4), (seqs[1], 1), (seqs[2], 9)], 64)
    assert m["order"] == [1, 0, 2] and m["num_decode"] == 1
    assert m["cu_rows"].tolist() == [0, 1, 5, 14] and m["row_seq"].tolist() == [0] + [1] * 4 + [2] * 9 and m["state_slots"].tolist() == [1, 0, 2]
    assert m["positions"].tolist() == [4, 66, 67, 68, 69] + list(range(9))


def test_which_kernels_take_which_layers():
    from nanovllm_hip.models import build_model
    from nanovllm_hip.models.zaposun import ZaposunConfig
    layers = {n: build_model(ZaposunConfig.from_json(CONFIGS[n])).layers for n in ("wide", "plain")}
    assert all(l.mixer.step_ok for l in layers["wide"]) and all(l.mixer.left.fast_prompt for l in layers["wide"] if hasattr(l.mixer, "left"))
    assert [l.mixer.step_ok for l in layers["plain"]] == [False, False, True, False]
    assert wkv(2, 3)["mlp"] is None
