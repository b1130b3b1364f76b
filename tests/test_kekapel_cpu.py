"""Host side of the Kekapel model on the CPU: configuration, registry, checkpoint, layer runs, pools per pass — and the plain reference itself
(oracle/kekapel_ref.py) against closed forms, with planted mistakes that must show."""
import copy
import math

import pytest
import torch

from oracle import kekapel_ref as K
from kekapel_cases import CONFIGS, attention, config, weights
from zobasun_cases import save_checkpoint, tokens

F64 = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


# ------------------------------------------------------------------------------------------------ reference
def test_reference_norms_by_hand():
    x = torch.tensor([[1.0, 3.0]], dtype=F64)
    assert torch.allclose(K.layer_norm(x, torch.tensor([2.0, 4.0], dtype=F64), torch.tensor([0.5, 0.0], dtype=F64), 3.0), torch.tensor([[-0.5, 2.0]], dtype=F64))
    assert torch.allclose(K.unit_rms(torch.tensor([[3.0, 4.0]], dtype=F64), 3.5), torch.tensor([[0.75, 1.0]], dtype=F64))


def test_reference_poly_norm_scales():
    """Each power is divided by its own root mean square: a positive factor on z changes nothing (eps 0), a sign only the odd powers."""
    z, c = rnd(3, 40), torch.tensor([0.3, -1.2, 0.8, 0.1], dtype=F64)
    y = K.poly_norm(z, c, 0.0)
    assert torch.allclose(K.poly_norm(z * 7.0, c, 0.0), y)
    assert torch.allclose(K.poly_norm(-z, c, 0.0), 2 * (c[1] * K.unit_rms(z * z, 0.0) + c[3]) - y)
    one = K.poly_norm(torch.full((1, 9), 2.0, dtype=F64), c, 0.0)
    assert torch.allclose(one, torch.full_like(one, c.sum().item()))


def test_reference_cap_and_mixing():
    s = torch.tensor([-1e9, -0.001, 0.0, 0.001, 1e9], dtype=F64)
    assert torch.allclose(K.softcap(s, 5.0), torch.tensor([-5.0, -0.001, 0.0, 0.001, 5.0], dtype=F64), atol=1e-9)
    s, t = rnd(3, 4, 5), rnd(3, 3, seed=1)
    assert torch.allclose(K.mix_heads(s, t), torch.tensordot(t, s, dims=1)) and torch.equal(K.mix_heads(s, torch.eye(3, dtype=F64)), s)


def test_reference_mixing_decides_who_is_seen():
    """A head that takes another head's scores attends where that one does, over its own values."""
    q, k, v = rnd(1, 2, 8), rnd(6, 2, 8, seed=1), rnd(6, 2, 4, seed=2)
    ok = torch.ones(1, 6, dtype=torch.bool)
    eye, swap = torch.eye(2, dtype=F64), torch.eye(2, dtype=F64).flip(0)
    p = [torch.softmax(K.softcap(q[0, h] @ k[:, h].T * 0.5, 3.0), 0) for h in (0, 1)]
    assert torch.allclose(K.attend(q, k, v, eye, 0.5, 3.0, ok)[0, 0], p[0] @ v[:, 0])
    assert torch.allclose(K.attend(q, k, v, swap, 0.5, 3.0, ok)[0, 0], p[1] @ v[:, 0])


def test_reference_window():
    ok = K.visible(10, 3)
    assert ok[9].nonzero().flatten().tolist() == [7, 8, 9] and ok[1].nonzero().flatten().tolist() == [0, 1]
    assert torch.equal(K.visible(5, 1), torch.eye(5, dtype=torch.bool)) and torch.equal(K.visible(5, 9), torch.ones(5, 5, dtype=torch.bool).tril())


def test_reference_expert_unit_by_hand():
    g, u = torch.tensor([9.0, -9.0, 0.5], dtype=F64), torch.tensor([9.0, -9.0, 0.25], dtype=F64)
    sig = [1 / (1 + math.exp(-1.702 * t)) for t in (2.0, -9.0, 0.5)]
    assert torch.allclose(K.clamped_unit(g, u, 2.0), torch.tensor([2 * sig[0] * 3, -9 * sig[1] * -1, 0.5 * sig[2] * 1.25], dtype=F64))


def test_reference_route_by_hand():
    z = torch.tensor([0.1, 2.0, -1.0, 1.0], dtype=F64)
    chosen, w, gap = K.route(z, 2)
    e = math.exp(-1.0)
    assert chosen == [1, 3] and torch.allclose(w, torch.tensor([1 / (1 + e), e / (1 + e)], dtype=F64)) and math.isclose(gap, 0.9)
    assert K.route(z, 4)[2] == math.inf


def test_layer_runs_agree():
    from nanovllm_hip.models.kekapel import KekapelConfig
    for name, cfg in CONFIGS.items():
        c = KekapelConfig.from_json(cfg)
        assert [i for i, _ in c.runs()] == [i for i, _ in K.layer_runs(cfg)]
        for i in range(len(cfg["layers"])):
            assert [t for j, t in c.runs() if j == i] == list(range(c.passes(i)))
    assert K.layer_runs(CONFIGS["odd"]) == [(0, 0), (1, None), (2, None), (0, 1), (1, None), (2, None), (0, 2), (1, None), (2, None), (3, None), (4, None)]


def replaced(name, make):
    """Plants: the reference's function `name` gives way to what `make` builds from it."""
    def plant(monkeypatch):
        monkeypatch.setattr(K, name, make(getattr(K, name)))
    return plant


PLANTS = {
    "window one longer": replaced("visible", lambda f: lambda n, size: f(n, size + 1)),
    "window one shorter": replaced("visible", lambda f: lambda n, size: f(n, max(size - 1, 1))),
    "no cap": replaced("softcap", lambda f: lambda s, cap: s),
    "cap after mixing": replaced("mix_heads", lambda f: lambda s, t: 4.0 * torch.tanh(f(s, t) / 4.0)),
    "mixing transposed": replaced("mix_heads", lambda f: lambda s, t: f(s, t.T)),
    "no mixing": replaced("mix_heads", lambda f: lambda s, t: s),
    "mean kept in the norm": replaced("layer_norm", lambda f: lambda x, w, b, eps: K.unit_rms(x, eps) * w + b),
    "no norm bias": replaced("layer_norm", lambda f: lambda x, w, b, eps: f(x, w, torch.zeros_like(b), eps)),
    "powers of the normed value": replaced("poly_norm", lambda f: lambda z, c, eps: sum(c[k] * K.unit_rms(z, eps) ** (k + 1) for k in range(3)) + c[3]),
    "poly norm without its constant": replaced("poly_norm", lambda f: lambda z, c, eps: f(z, c, eps) - c[3]),
    "gate clamped below": replaced("clamped_unit", lambda f: lambda g, u, limit: f(torch.clamp(g, min=-limit), u, limit)),
    "no plus one": replaced("clamped_unit", lambda f: lambda g, u, limit: f(g, u, limit) - f(g, torch.zeros_like(u), limit)),
    "plain silu": replaced("clamped_unit", lambda f: lambda g, u, limit: (lambda a, b: a * torch.sigmoid(a) * (b + 1))(torch.clamp(g, max=limit), torch.clamp(u, -limit, limit))),
    # (a common factor of the weights is lost in the norm behind the experts: only their ratio shows)
    "equal expert weights": replaced("route", lambda f: lambda z, top: (f(z, top)[0], torch.full((top,), 1.0 / top, dtype=F64), f(z, top)[2])),
    "sigmoid expert weights": replaced("route", lambda f: lambda z, top: (f(z, top)[0], torch.sigmoid(z)[f(z, top)[0]], f(z, top)[2])),
    "positions scaled": replaced("embedding", lambda f: lambda cfg, w, toks: (f(cfg, w, toks) - w["pos"][:len(toks)]) + w["pos"][:len(toks)] * cfg["embedding"]["scale"]),
    "positions one off": replaced("embedding", lambda f: lambda cfg, w, toks: (f(cfg, w, toks) - w["pos"][:len(toks)]) + w["pos"][1:len(toks) + 1]),
}


@pytest.mark.parametrize("name", sorted(PLANTS))
def test_planted_mistakes_show(monkeypatch, name):
    """A reference with one equation wrong is far from the right one, so the comparisons of the GPU tests have teeth."""
    cfg, w = CONFIGS["odd"], weights("odd")
    toks = tokens(130, cfg["vocab"], 3)
    good = K.forward(cfg, w, toks)
    PLANTS[name](monkeypatch)
    bad = K.forward(cfg, w, toks)
    err = (bad - good).pow(2).mean(1).sqrt() / good.std()
    assert err.max() > 100 * 5e-5 and err.mean() > 1e-3


def _one_pass_less(cfg, w):
    cfg["loop"]["times"] -= 1


def _steps_swapped(cfg, w):
    w["loop.step"] = w["loop.step"].flip(0)


def _no_steps(cfg, w):
    w["loop.step"] = torch.zeros_like(w["loop.step"])


def _mult_on_both(cfg, w):
    cfg["residual_mult"] **= 2


def _no_router_bias(cfg, w):
    w["l0.mlp.router.b"] = torch.zeros_like(w["l0.mlp.router.b"])


def _no_second_norm(cfg, w):
    w["l1.norm1b"], w["l1.norm1b.b"] = torch.ones_like(w["l1.norm1b"]), torch.zeros_like(w["l1.norm1b.b"])


def _norm_weights_of_keys(cfg, w):
    w["l1.mix.q.norm"] = w["l1.mix.k.norm"]


@pytest.mark.parametrize("edit", [_one_pass_less, _steps_swapped, _no_steps, _mult_on_both, _no_router_bias, _no_second_norm, _norm_weights_of_keys], ids=lambda f: f.__name__[1:])
def test_planted_structure_shows(edit):
    cfg, w = copy.deepcopy(CONFIGS["odd"]), dict(weights("odd"))
    toks = tokens(60, cfg["vocab"], 3)
    good = K.forward(cfg, w, toks)
    edit(cfg, w)
    assert (K.forward(cfg, w, toks) - good).pow(2).mean().sqrt() > 0.01 * good.std()


# ------------------------------------------------------------------------------------------------ configuration, registry, checkpoint
def test_config_and_registry(tmp_path):
    from nanovllm_hip.models import load_config, model_class
    from nanovllm_hip.models.kekapel import KekapelConfig, KekapelForCausalLM
    save_checkpoint(tmp_path, CONFIGS["odd"], {"x": torch.zeros(1)})
    cfg = load_config(str(tmp_path), dtype=torch.float32)
    assert isinstance(cfg, KekapelConfig) and model_class(cfg) is KekapelForCausalLM and cfg.dtype == torch.float32
    assert (cfg.hidden_size, cfg.vocab_size, cfg.num_hidden_layers, cfg.norm_eps, cfg.embedding_scale, cfg.residual_mult) == (72, 101, 5, 1e-5, 3.0, 0.6)
    assert cfg.max_position_embeddings == 512
    assert load_config(str(tmp_path), max_position_embeddings=64).max_position_embeddings == 64
    assert load_config(str(tmp_path), max_position_embeddings=9999).max_position_embeddings == 512        # (the position table has no more rows)
    assert KekapelConfig.from_json(config(64, 10, [attention(1, 1, 8, 8, 5, 1.0, 1.0)])).runs() == [(0, 0)]


@pytest.mark.parametrize("edit,match", [
    (lambda c: c["layers"][0].update(type="other"), "unknown mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="other"), "unknown feed-forward"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mixer"].update(softcap=0.0), "softcap"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "top"),
    (lambda c: c["loop"].update(stop=6), "loop"),
    (lambda c: c["loop"].update(times=0), "loop"),
])
def test_config_refuses(edit, match):
    from nanovllm_hip.models.kekapel import KekapelConfig
    cfg = copy.deepcopy(CONFIGS["odd"])
    edit(cfg)
    with pytest.raises(ValueError, match=match):
        KekapelConfig.from_json(cfg)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_checkpoint_is_read_whole(name, tmp_path):
    """Every tensor lands somewhere, padding stays zero, and what the layers hold gives the reference's numbers back."""
    from nanovllm_hip.models import build_model, load_config
    from nanovllm_hip.utils import loader
    cfg, w = CONFIGS[name], weights(name)
    save_checkpoint(tmp_path, cfg, w)
    ckpt = loader.Checkpoint(str(tmp_path))
    c = load_config(str(tmp_path))
    model = build_model(c, str(tmp_path))
    type(model)(c).load_weights(ckpt)
    assert ckpt.unread() == []
    d = cfg["width"]
    assert torch.equal(model.pos[:, :d], w["pos"].float()) and not model.pos[:, d:].any()
    for i, layer in enumerate(model.layers):
        m, spec, p = layer.mixer, cfg["layers"][i], f"l{i}."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if spec["mlp"] is not None else ()):
            for t, name_ in zip(layer.norm(n), (p + n, p + n + ".b")):
                assert torch.equal(t[:d], w[name_].float()) and not t[d:].any()
        s = spec["mixer"]
        h = torch.randn(1, model.cols)
        h[:, d:] = 0
        rows = (h @ m.w_qkv.float().T)[:, m.q_cols:m.q_cols + m.k_cols].view(m.kv_heads, m.dk)
        want = h[:, :d] @ w[p + "mix.k"].float().T
        assert torch.allclose(rows[:, :s["dim"]].reshape(1, -1), want, atol=1e-4) and not rows[:, s["dim"]:].any()
        assert torch.equal(m.q_norm[:s["dim"]], w[p + "mix.q.norm"].float()) and not m.q_norm[s["dim"]:].any() and torch.equal(m.talk, w[p + "mix.talk"].float())
        if spec["mlp"] is not None and spec["mlp"]["kind"] == "moe":
            assert torch.equal(layer.mlp.w_gate_up[1, layer.mlp.cols:layer.mlp.cols + layer.mlp.ff, :d], w[p + "mlp.e1.up"])
        elif spec["mlp"] is not None:
            assert torch.equal(layer.mlp.w_up[:layer.mlp.ff, :d], w[p + "mlp.up"]) and torch.equal(layer.mlp.coef, w[p + "mlp.act"].float())


def test_random_weights_are_deterministic():
    from nanovllm_hip.models import build_model
    from nanovllm_hip.models.kekapel import KekapelConfig
    cfg = KekapelConfig.from_json(CONFIGS["odd"])
    a, b = build_model(cfg, seed=3), build_model(cfg, seed=3)
    assert all(torch.equal(x, y) for x, y in zip(a.buffers(), b.buffers())) and abs(a.layers[0].norm1[:72].mean() - 1) < 0.02


def test_pools_have_one_entry_per_pass():
    from nanovllm_hip.engine.model_runner import ModelRunner
    from nanovllm_hip.models.kekapel import KekapelConfig
    cfg = KekapelConfig.from_json(CONFIGS["odd"])
    r = ModelRunner(cfg, 5, device="cpu", max_model_len=512, max_num_seqs=3)
    m = [layer.mixer for layer in r.model.layers]
    assert [tuple(x.page_cache.shape[:3]) for x in m] == [(3, 5, 64)] * 3 + [(1, 5, 64)] * 2 and not r.state
    with pytest.raises(AssertionError):
        ModelRunner(cfg, 5, device="cpu", max_model_len=513, max_num_seqs=3)


def test_which_kernels_take_which_layers():
    from nanovllm_hip.models import build_model
    from nanovllm_hip.models.kekapel import KekapelConfig
    forms = {n: [(l.mixer.fast, l.mixer.fast_prompt) for l in build_model(KekapelConfig.from_json(CONFIGS[n])).layers] for n in ("wide", "plain")}
    assert forms["wide"] == [(True, True)] * 4
    assert forms["plain"] == [(False, False), (True, False), (False, False), (False, False)]
