"""Host side of the Galirax model on the CPU: configuration, registry, checkpoint, layer runs, pools per pass — and the plain reference itself
(oracle/galirax_ref.py) against closed forms, with planted mistakes that must show."""
import copy
import importlib.util
import math
import os

import pytest
import torch

from oracle import galirax_ref as G
from galirax_cases import CONFIGS, attention, config, lightning, weights
from zobasun_cases import save_checkpoint, tokens

F64 = torch.float64
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ------------------------------------------------------------------------------------------------ reference
def test_reference_recurrence_closed_form():
    """Constant k, v, q: S_t = k v^T (1 - d^t) / (1 - d)."""
    k, v, q, d = torch.tensor([1.0, -2.0], dtype=F64), torch.tensor([0.5, 3.0, 1.0], dtype=F64), torch.tensor([0.3, 0.7], dtype=F64), 0.9
    o, s = G.lightning_recurrence(q.expand(30, 2), k.expand(30, 2), v.expand(30, 3), d)
    gain = (1 - d ** torch.arange(1, 31, dtype=F64)) / (1 - d)
    assert torch.allclose(o, gain[:, None] * (q @ k) * v, rtol=1e-12) and torch.allclose(s, gain[-1] * k[:, None] * v, rtol=1e-12)
    o2, s2 = G.lightning_recurrence(q.expand(3, 2), k.expand(3, 2), v.expand(3, 3), d, s)
    assert torch.allclose(s2, (1 - d ** 33) / (1 - d) * k[:, None] * v, rtol=1e-12)


def test_reference_sink_is_one_more_entry():
    z = torch.randn(4, 7, dtype=F64)
    with_entry = torch.softmax(torch.cat([z, torch.full((4, 1), 1.3, dtype=F64)], dim=1), dim=1)[:, :7]
    assert torch.allclose(G.sink_softmax(z, torch.tensor(1.3, dtype=F64)), with_entry, rtol=1e-12)


def test_reference_window():
    ok = G.visible(10, {"size": 3, "keep_first": 2})
    assert ok[9].nonzero().flatten().tolist() == [0, 1, 7, 8, 9] and ok[3].nonzero().flatten().tolist() == [0, 1, 2, 3] and ok[0].nonzero().flatten().tolist() == [0]
    assert torch.equal(G.visible(5, None), torch.ones(5, 5, dtype=torch.bool).tril())


def test_reference_rotation_depends_on_distance_only():
    g = torch.Generator().manual_seed(0)
    q, k = torch.randn(1, 1, 16, generator=g, dtype=F64), torch.randn(1, 1, 16, generator=g, dtype=F64)
    freqs = G.frequencies(dict(dims=12, base=900.0, scaling=dict(factor=3.0, low=1.0, high=2.0, original=40)))

    def score(i, j):
        return (G.rotate_pairs(q, torch.tensor([i]), freqs) * G.rotate_pairs(k, torch.tensor([j]), freqs)).sum().item()
    assert math.isclose(score(70, 3), score(167, 100), rel_tol=1e-12) and not math.isclose(score(70, 3), score(70, 4), rel_tol=1e-6)
    assert torch.equal(G.rotate_pairs(q, torch.tensor([5]), freqs)[..., 12:], q[..., 12:])


def test_reference_route_by_hand():
    z = torch.logit(torch.tensor([0.9, 0.2, 0.6, 0.5, 0.8, 0.1], dtype=F64))
    corr = torch.tensor([-3.0, 0.1, 0.0, 0.05, -0.2, 0.3], dtype=F64)               # choice: -2.1 0.3 | 0.6 0.55 | 0.6 0.4
    chosen, w, gap = G.route(z, corr, dict(top=2, scale=2.0, groups=dict(count=3, keep=1)))
    assert chosen == [2, 3] and torch.allclose(w, torch.tensor([0.6, 0.5], dtype=F64) / 1.1 * 2) and math.isclose(gap, 0.15, rel_tol=1e-9)
    chosen, w, _ = G.route(z, corr, dict(top=5, scale=1.0, groups=dict(count=3, keep=3)))
    assert sorted(chosen) == [1, 2, 3, 4, 5] and torch.allclose(w.sum(), torch.tensor(1.0, dtype=F64))


def test_layer_runs_agree():
    from nanovllm_hip.models.galirax import GaliraxConfig
    for name, cfg in CONFIGS.items():
        c = GaliraxConfig.from_json(cfg)
        assert [i for i, _ in c.runs()] == G.layer_runs(cfg)
        for i in range(len(cfg["layers"])):
            assert [t for j, t in c.runs() if j == i] == list(range(c.passes(i)))
    assert G.layer_runs(CONFIGS["odd"]) == [0, 1, 2, 1, 2, 1, 2, 3, 4]


def _no_sink(monkeypatch):
    monkeypatch.setattr(G, "sink_softmax", lambda s, sink: torch.softmax(s, dim=-1))


def _scaled_sink(monkeypatch):
    soft = G.sink_softmax
    monkeypatch.setattr(G, "sink_softmax", lambda s, sink: soft(s, sink * 0.2))


def _window_off_by_one(monkeypatch):
    vis = G.visible
    monkeypatch.setattr(G, "visible", lambda n, m: vis(n, m if m is None else {**m, "size": m["size"] + 1}))


def _keep_one_less(monkeypatch):
    vis = G.visible
    monkeypatch.setattr(G, "visible", lambda n, m: vis(n, m if m is None else {**m, "keep_first": m["keep_first"] - 1}))


def _rotation_halves(monkeypatch):
    rot = G.rotate_pairs

    def halves(x, pos, freqs):
        n = len(freqs)
        perm = torch.stack([torch.arange(n), torch.arange(n) + n], 1).reshape(-1)
        y = x.clone()
        y[..., perm] = rot(x[..., perm], pos, freqs)
        return y
    monkeypatch.setattr(G, "rotate_pairs", halves)


def _no_scaling(monkeypatch):
    freqs = G.frequencies
    monkeypatch.setattr(G, "frequencies", lambda rot: freqs({k: v for k, v in rot.items() if k != "scaling"}))


def _norm_per_head(monkeypatch):
    rms = G.rms_norm

    def norm(x, w, eps):
        return rms(x.view(x.shape[0], 2, -1), w.view(2, -1), eps).flatten(1)
    monkeypatch.setattr(G, "rms_norm", norm)


def _correction_in_weights(monkeypatch):
    def route(z, c, r):
        chosen, _, gap = ROUTE(z, c, r)
        w = (torch.sigmoid(z) + c)[chosen]
        return chosen, w / (w.sum() + 1e-20) * r["scale"], gap
    ROUTE = G.route
    monkeypatch.setattr(G, "route", route)


def _no_groups(monkeypatch):
    route = G.route
    monkeypatch.setattr(G, "route", lambda z, c, r: route(z, c, {**r, "groups": dict(count=1, keep=1)}))


def _decay_after_adding(monkeypatch):
    rec = G.lightning_recurrence
    monkeypatch.setattr(G, "lightning_recurrence", lambda q, k, v, d, state=None: rec(q, k * d, v, d, state))


def _no_cap(monkeypatch):
    monkeypatch.setattr(G, "softcap", lambda z, cap: z)


def _rms_for_layer_norm(monkeypatch):
    monkeypatch.setattr(G, "layer_norm", lambda x, w, b, eps: G.rms_norm(x, w, eps) + b)


@pytest.mark.parametrize("plant", [_no_sink, _scaled_sink, _window_off_by_one, _keep_one_less, _rotation_halves, _no_scaling, _norm_per_head, _correction_in_weights,
                                   _no_groups, _decay_after_adding, _no_cap, _rms_for_layer_norm], ids=lambda f: f.__name__[1:])
def test_planted_mistakes_show(monkeypatch, plant):
    """A reference with one equation wrong is far from the right one, so the comparisons of the GPU tests have teeth."""
    cfg, w = CONFIGS["odd"], weights("odd")
    toks = tokens(130, cfg["vocab"], 3)
    good = G.forward(cfg, w, toks)
    plant(monkeypatch)
    bad = G.forward(cfg, w, toks)
    err = (bad - good).pow(2).mean(1).sqrt() / good.std()
    assert err.max() > 100 * 5e-5 and err.mean() > 1e-3


@pytest.mark.parametrize("edit", ["one pass less", "shared state", "experts read another input"])
def test_planted_structure_shows(edit, monkeypatch):
    cfg, w = copy.deepcopy(CONFIGS["odd"]), weights("odd")
    toks = tokens(60, cfg["vocab"], 3)
    good = G.forward(cfg, w, toks)
    if edit == "one pass less":
        cfg["loop"]["times"] -= 1
    elif edit == "shared state":                                          # a pass that goes on from the state of the one before
        kept = {}
        rec = G.lightning_recurrence

        def shared(q, k, v, d, state=None):
            o, kept[d] = rec(q, k, v, d, kept.get(d))
            return o, kept[d]
        monkeypatch.setattr(G, "lightning_recurrence", shared)
    else:
        moe = G.moe
        monkeypatch.setattr(G, "moe", lambda w, p, m, h, margins=None: moe(w, p, m, h * 1.1, margins))
    assert (G.forward(cfg, w, toks) - good).pow(2).mean().sqrt() > 0.01 * good.std()


# ------------------------------------------------------------------------------------------------ configuration, registry, checkpoint
def test_config_and_registry(tmp_path):
    from nanovllm_hip.models import load_config, model_class
    from nanovllm_hip.models.galirax import GaliraxConfig, GaliraxForCausalLM
    save_checkpoint(tmp_path, CONFIGS["odd"], {"x": torch.zeros(1)})
    cfg = load_config(str(tmp_path), dtype=torch.float32)
    assert isinstance(cfg, GaliraxConfig) and model_class(cfg) is GaliraxForCausalLM and cfg.dtype == torch.float32
    assert (cfg.hidden_size, cfg.vocab_size, cfg.num_hidden_layers, cfg.norm_eps, cfg.logit_softcap) == (72, 101, 5, 1e-5, 20.0)
    assert GaliraxConfig.from_json(config(64, 10, [lightning(1, 8, 8, [0.5])])).runs() == [(0, 0)]


@pytest.mark.parametrize("edit,match", [
    (lambda c: c["layers"][0].update(type="other"), "unknown mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "unknown feed-forward"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=22), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "top"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "groups"),
    (lambda c: c["layers"][1]["mixer"].update(heads=4), "decays"),
    (lambda c: c["loop"].update(stop=6), "loop"),
    (lambda c: c["loop"].update(times=0), "loop"),
])
def test_config_refuses(edit, match):
    from nanovllm_hip.models.galirax import GaliraxConfig
    cfg = copy.deepcopy(CONFIGS["odd"])
    edit(cfg)
    with pytest.raises(ValueError, match=match):
        GaliraxConfig.from_json(cfg)


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
    for i, layer in enumerate(model.layers):
        m, spec, p = layer.mixer, cfg["layers"][i], f"l{i}."
        assert torch.equal(layer.norm[:cfg["width"]], w[p + "norm1"].float()) and not layer.norm[cfg["width"]:].any()
        s = spec["mixer"]
        h = torch.randn(1, model.cols)
        h[:, cfg["width"]:] = 0
        if spec["type"] == "lightning":
            got = (h @ m.w_in.float().T)[:, m.qkv_cols:].view(m.heads, m.dv)
            want = h[:, :cfg["width"]] @ w[p + "mix.g"].float().T
            assert torch.allclose(got[:, :s["vdim"]].reshape(1, -1), want, atol=1e-4) and not got[:, s["vdim"]:].any()
        else:
            rows = (h @ m.w_qkv.float().T)[:, m.q_cols:m.q_cols + m.k_cols].view(m.kv_heads, m.dk)
            want = h[:, :cfg["width"]] @ w[p + "mix.k"].float().T
            assert torch.allclose(rows[:, :s["dim"]].reshape(1, -1), want, atol=1e-4) and not rows[:, s["dim"]:].any()
        if spec["mlp"] is not None:
            assert torch.equal(layer.mlp.w_gate_up[1, layer.mlp.cols:layer.mlp.cols + layer.mlp.ff, :cfg["width"]], w[p + "mlp.e1.up"])


def test_random_weights_are_deterministic():
    from nanovllm_hip.models import build_model
    from nanovllm_hip.models.galirax import GaliraxConfig
    cfg = GaliraxConfig.from_json(CONFIGS["odd"])
    a, b = build_model(cfg, seed=3), build_model(cfg, seed=3)
    assert all(torch.equal(x, y) for x, y in zip(a.buffers(), b.buffers())) and abs(a.layers[0].norm[:72].mean() - 1) < 0.02


def test_pools_have_one_entry_per_pass():
    from nanovllm_hip.engine.model_runner import ModelRunner
    from nanovllm_hip.models.galirax import GaliraxConfig
    cfg = GaliraxConfig.from_json(CONFIGS["odd"], max_position_embeddings=512)
    r = ModelRunner(cfg, 5, device="cpu", max_model_len=512, max_num_seqs=3)
    m = [layer.mixer for layer in r.model.layers]
    assert [tuple(x.page_cache.shape[:3]) for x in (m[0], m[2], m[4])] == [(1, 5, 64), (3, 5, 64), (1, 5, 64)]
    assert m[1].state.shape == (3, 3, 3, 64, 64) and m[3].state.shape == (1, 3, 2, 128, 64) and len(r.state) == 2


def test_padded_widths():
    from nanovllm_hip.layers.paged_attention import padded_widths
    assert [padded_widths(*d) for d in ((20, 12), (64, 65), (130, 64), (200, 128), (64, 129), (257, 8), (100, 300))] == [
        (64, 64), (64, 128), (192, 64), (256, 128), (256, 256), (264, 8), (104, 304)]


def test_attention_forms():
    """Which extras each form of attention has."""
    from nanovllm_hip.models import build_model
    from nanovllm_hip.models.galirax import GaliraxConfig
    m = [layer.mixer for layer in build_model(GaliraxConfig.from_json(CONFIGS["odd"])).layers]
    assert m[0].bias and m[0].qk_norm and m[0].has_sink and (m[0].window, m[0].keep_first) == (37, 3)
    assert not m[2].bias and not m[2].qk_norm and m[2].has_sink and (m[2].window, m[2].keep_first) == (0, 0)
    one = GaliraxConfig.from_json(config(64, 20, [attention(2, 1, 16, 16, 8, 0.3)]))
    assert build_model(one).layers[0].mlp is None


def test_every_model_has_its_sources():
    """The libraries of single models name files that exist and leave none of the whole library's out."""
    spec = importlib.util.spec_from_file_location("nvh_build", os.path.join(ROOT, "nano-vllm-learn_amd", "build.py"))
    build = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(build)
    names = sorted(f for f in os.listdir(build.CSRC) if f.endswith(".hip"))
    assert sorted(build.SOURCES) == names and len(set(build.SOURCES)) == len(build.SOURCES)
    assert all(os.path.exists(os.path.join(build.CSRC, h)) for h in build.HEADERS)
