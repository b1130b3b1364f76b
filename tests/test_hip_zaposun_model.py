"""GPU: Zaposun models of several sizes through the engine (checkpoint -> registry -> pages and state slots -> scheduler -> sampling), against the plain float64
reference on the CPU.  fp32 models are held to fp32 rounding, bf16 models to bf16's."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import zaposun_ref as Z
from zaposun_cases import CONFIGS, config, parallel, weights, wkv
from zobasun_cases import save_checkpoint, tokens

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BF16, F32 = torch.bfloat16, torch.float32
_FOLDERS, _PLAIN = {}, {}


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    def get(name):
        if name not in _FOLDERS:
            path = tmp_path_factory.mktemp(name)
            save_checkpoint(path, CONFIGS[name], weights(name))
            _FOLDERS[name] = str(path)
        return _FOLDERS[name]
    return get


def plain(name, toks):
    key = (name, tuple(toks))
    if key not in _PLAIN:
        _PLAIN[key] = Z.forward(CONFIGS[name], weights(name), toks)
    return _PLAIN[key]


def engine(folder, name, dtype, pool_tokens=1024, **kw):
    from nanovllm_hip.engine.llm_engine import LLMEngine
    kw = {**dict(max_num_seqs=4, max_model_len=512), **kw}
    return LLMEngine.from_folder(folder(name), dict(dtype=dtype), num_kvcache_blocks=pool_tokens // 64, **kw)


def row_errors(got, want):
    d = got.float().cpu().double() - want
    d = d - d.mean(1, keepdim=True)
    return d.pow(2).mean(1).sqrt() / want.std()


def check(got, want, dtype):
    e = row_errors(got, want)
    if dtype == F32:
        assert e.max() < 5e-5, f"worst row {e.max():.2e}"
    else:                                                                # (the first tokens' norms divide by little: their rows are the worst)
        assert e.median() < 0.04 and e.max() < 0.3, f"median {e.median():.3f} worst row {e.max():.3f} at {e.argmax()}"


def feed(eng, seq, toks, cuts):
    """Feed a sequence in portions ending at `cuts`; returns the logits of every token."""
    out, at = [], 0
    for hi in cuts:
        if at:
            for t in toks[at:hi]:
                seq.append_token(t)
        out.append(eng.feed([(seq, hi - at)], [list(range(hi - at))]))
        at = hi
    eng.release(seq)
    return torch.cat([o.float() for o in out])


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", ["odd", "plain", "strong", "wide"])
def test_prompts_portions_and_decoding(folder, name, dtype):
    """A whole prompt, the same prompt in portions of every kind (down to two tokens), and token by token: all against the reference."""
    eng = engine(folder, name, dtype)
    toks = tokens(203, CONFIGS[name]["vocab"], 1)
    want = plain(name, toks)
    for cuts in ([203], [1, 3, 5, 64, 66, 128, 130, 195, 203], [63, 65, 190, 192] + list(range(193, 204)), list(range(1, 204))):
        check(feed(eng, eng.sequence(toks[:cuts[0]]), toks, cuts), want, dtype)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", ["odd", "plain", "strong", "wide"])
def test_mixed_batches_with_reuse(folder, name, dtype):
    """Unequal requests in one batch — portions beside single tokens, requests left out of steps — on pages and state slots that are handed on several times; every
    row against the reference of its request alone."""
    eng = engine(folder, name, dtype, pool_tokens=448, max_num_seqs=3)
    vocab = CONFIGS[name]["vocab"]
    lengths = [130, 5, 70, 66, 1, 129, 64, 2, 90]
    reqs = [tokens(n, vocab, 20 + i) for i, n in enumerate(lengths)]
    pieces = [[60, 2, 5, 1, 1, 61], [1, 4], [70], [63, 1, 1, 1], [1], [2, 100, 27], [64], [2], [17, 3, 1, 1, 1, 1, 66]]
    waiting, live, got, step = list(range(len(reqs))), {}, {i: [] for i in range(len(reqs))}, 0
    while waiting or live:
        while waiting and len(live) < 3:
            live[waiting.pop(0)] = None
        batch = []
        for i in list(live):
            if live[i] is not None and (step + i) % 4 == 3 and len(live) > 1:
                continue                                              # left out of this step
            n = pieces[i].pop(0)
            if live[i] is None:
                live[i] = eng.sequence(reqs[i][:n])
            else:
                for t in reqs[i][len(live[i]):len(live[i]) + n]:
                    live[i].append_token(t)
            batch.append((i, live[i], n))
        step += 1
        if not batch:
            continue
        logits = eng.feed([(s, n) for _, s, n in batch], [list(range(n)) for *_, n in batch]).float().cpu()
        for (i, s, n), rows in zip(batch, logits.split([n for *_, n in batch])):
            got[i].append(rows)
            if not pieces[i]:
                eng.release(s)
                del live[i]
    check(torch.cat([torch.cat(got[i]) for i in range(len(reqs))]), torch.cat([plain(name, r) for r in reqs]), dtype)
    assert len(eng.block_manager.free_block_ids) == 7 and len(eng.state_slots.free) == 3


def test_wanted_rows_only(folder):
    eng = engine(folder, "odd", F32)
    toks = tokens(50, 101, 2)
    a, b = eng.sequence(toks), eng.sequence(toks[:20])
    got = eng.feed([(a, 50), (b, 20)], [[3, 49, 0], []])
    check(got, plain("odd", toks)[[3, 49, 0]], F32)
    assert eng.feed([(eng.sequence([1]), 1)], [[]]) is None


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_rows_do_not_depend_on_the_batch_or_the_pages(folder, dtype):
    """The same request alone and in company, on other pages and slots: equal up to rounding."""
    toks = tokens(140, CONFIGS["wide"]["vocab"], 4)
    eng = engine(folder, "wide", dtype)
    alone = feed(eng, eng.sequence(toks), toks, [140])
    eng = engine(folder, "wide", dtype)
    eng.block_manager.free_block_ids.rotate(5)
    eng.state_slots.free.rotate(1)
    others = [eng.sequence(tokens(n, CONFIGS["wide"]["vocab"], n)) for n in (64, 3)]
    seq = eng.sequence(toks)
    got = eng.feed([(others[0], 64), (seq, 140), (others[1], 3)], [[], list(range(140)), []])
    if dtype == F32:
        assert row_errors(got, alone.double().cpu()).max() < 5e-5
    check(got, plain("wide", toks), dtype)


def test_many_rows_at_once(folder):
    """A batch of more than a thousand rows (row kernels take several rows per thread), some of them single tokens, segments of recurrences over a thousand tokens."""
    eng = engine(folder, "odd", F32, pool_tokens=2048, max_model_len=1100)
    reqs = [tokens(n, 101, n) for n in (1100, 40, 300)]
    seqs = [eng.sequence(r[:n]) for r, n in zip(reqs, (7, 39, 2))]
    eng.feed([(s, len(s)) for s in seqs], [[], [], []])
    for s, r in zip(seqs, reqs):
        for t in r[len(s):]:
            s.append_token(t)
    got = eng.feed([(s, len(s) - s.num_cached_tokens) for s in seqs], [list(range(len(s) - s.num_cached_tokens)) for s in seqs])
    want = torch.cat([plain("odd", r)[n:] for r, n in zip(reqs, (7, 39, 2))])
    check(got, want, F32)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_smallest_models(dtype):
    """One layer of a kind, no feed-forward, constants at one, one stream; and a model without layers.  (Norm groups of one column are a sign: not for bf16.)"""
    from nanovllm_hip.engine.llm_engine import LLMEngine
    from nanovllm_hip.models.zaposun import ZaposunConfig
    for layers, kw in (([wkv(1, 8)], dict(streams=1, logit_scale=1.0, buckets=1, decay_rank=1)), ([parallel(1, 1, 8, 8, 8, 1000, 1.0, 8, 1, 1, 1, base=1.0)], dict(streams=1, groups=8 if dtype == F32 else 2)),
                       ([parallel(2, 1, 16, 2, 2, 3, 0.5, 16, 2, 1, 2, ff=8)], dict(streams=2, groups=2, buckets=3)), ([], dict(streams=4))):
        cfg = config(8, 11, layers, **kw)
        w = Z.random_weights(cfg, seed=2)
        eng = LLMEngine(ZaposunConfig.from_json(cfg, dtype=dtype, max_position_embeddings=70), 2, max_num_seqs=2, max_model_len=70)
        eng.runner.model.load_weights(lambda n: w[n].cuda())
        eng.runner.model.cuda()
        toks = tokens(70, 11, 1)
        got = feed(eng, eng.sequence(toks[:60]), toks, [60, 62] + list(range(63, 71)))
        check(got, Z.forward(cfg, w, toks), dtype)


def test_fused_decode_path_matches_the_plain_one(folder, monkeypatch):
    from nanovllm_hip.models import zaposun
    toks = tokens(90, CONFIGS["wide"]["vocab"], 5)
    for fused in (True, False):
        monkeypatch.setattr(zaposun, "FUSED_DECODE", fused)
        eng = engine(folder, "wide", BF16)
        check(feed(eng, eng.sequence(toks[:60]), toks, [60] + list(range(61, 91))), plain("wide", toks), BF16)


def test_long_contractions_decode(folder):
    """Widths above 1024: prompt, then decoding of several sequences through the fused path (split-K launches of many shapes on one workspace)."""
    reqs = [tokens(n, 300, n) for n in (40, 23, 31)]
    eng = engine(folder, "long", BF16)
    seqs = [eng.sequence(r[:-12]) for r in reqs]
    rows = [[r.float().cpu()] for r in eng.feed([(s, len(s)) for s in seqs], [list(range(len(s))) for s in seqs]).split([len(s) for s in seqs])]
    for t in range(12):
        for s, r in zip(seqs, reqs):
            s.append_token(r[len(s)])
        for out, row in zip(rows, eng.feed([(s, 1) for s in seqs]).float().cpu()):
            out.append(row[None])
    check(torch.cat([torch.cat(r) for r in rows]), torch.cat([plain("long", r) for r in reqs]), BF16)


@pytest.mark.parametrize("name,dtype", [("odd", F32), ("odd", BF16), ("wide", BF16)])
def test_more_single_tokens_than_the_fused_path_takes(folder, name, dtype):
    """Seventy sequences decoded together."""
    vocab = CONFIGS[name]["vocab"]
    reqs = [tokens(4 + i % 5, vocab, i) for i in range(70)]
    eng = engine(folder, name, dtype, pool_tokens=70 * 64, max_num_seqs=70)
    seqs = [eng.sequence(r[:-3]) for r in reqs]
    eng.feed([(s, len(s)) for s in seqs], [[] for _ in seqs])
    rows = []
    for _ in range(3):
        for s, r in zip(seqs, reqs):
            s.append_token(r[len(s)])
        rows.append(eng.feed([(s, 1) for s in seqs]).float().cpu())
    want = torch.stack([Z.forward(CONFIGS[name], weights(name), r)[-3:] for r in reqs], dim=1)
    check(torch.cat(rows), want.reshape(-1, vocab), dtype)


# ------------------------------------------------------------------------------------------------ generation
def follow(name, prompt, out, dtype):
    """Every generated token is the reference's arg-max after the same tokens, up to ties within rounding."""
    logits = Z.forward(CONFIGS[name], weights(name), prompt + out)[len(prompt) - 1:-1]
    slack = (1e-4 if dtype == F32 else 0.4) * logits.std()
    bad = [i for i, (row, t) in enumerate(zip(logits, out)) if row[t] < row.max() - slack]
    assert not bad, bad


@pytest.mark.parametrize("name,dtype", [("odd", F32), ("odd", BF16), ("wide", F32), ("wide", BF16), ("plain", BF16)])
def test_greedy_generation(folder, name, dtype):
    """Through generate(): more requests than slots, prompts cut by the token budget, long decoding in graph sessions across page and chunk borders."""
    prompts = [tokens(n, CONFIGS[name]["vocab"], 40 + n) for n in (90, 3, 150, 61, 33)]
    counts = [40, 150, 12, 30, 1]
    eng = engine(folder, name, dtype, max_num_batched_tokens=100)
    outs = eng.generate(prompts, counts)
    assert [len(o) for o in outs] == counts
    for p, o in zip(prompts, outs):
        follow(name, p, o, dtype)
    assert len(eng.block_manager.free_block_ids) == 16 and len(eng.state_slots.free) == 4


def test_generation_is_the_same_eager_graph_and_preempted(folder):
    """fp32: graph sessions, eager steps and a pool so small that a sequence has to start over all give the same tokens."""
    prompts = [tokens(n, 101, 60 + n) for n in (70, 20, 40)]
    outs = [engine(folder, "odd", F32, **kw).generate(prompts, 70) for kw in (dict(), dict(enforce_eager=True), dict(pool_tokens=320, enforce_eager=True),
                                                                              dict(pool_tokens=320))]
    assert outs[0] == outs[1] == outs[2] == outs[3]


def test_graph_session_replays(folder):
    """A captured decode step replayed many times, with other work on the device between the replays, equals eager steps; the state is put back by a rewind."""
    eng = engine(folder, "wide", BF16)
    seqs = [eng.sequence(tokens(n, 160, n)) for n in (80, 7)]
    eng.prefill(seqs, reserve_tokens=64)
    sess = eng.runner.decode_session(seqs, 40)
    assert sess.graph is not None
    saved = sess.state()
    logs = []
    for rep in range(3):
        for _ in range(10):
            sess.step(1)
            torch.randn(100, 100, device="cuda").sum()
        sess.step(8)
        torch.cuda.synchronize()
        logs.append(sess.tokens[:18].clone())
        sess.rewind(saved)
    assert torch.equal(logs[0], logs[1]) and torch.equal(logs[0], logs[2])
    eager = eng.runner.decode_session(seqs, 40, use_graph=False)
    eager.step(18)
    assert torch.equal(eager.tokens[:18], logs[0])


# ------------------------------------------------------------------------------------------------ programs
def test_trace_replay_program(folder, tmp_path):
    steps, reqs = [], {"a": tokens(70, 101, 1), "b": tokens(9, 101, 2)}
    steps.append(dict(entries=[dict(id="a", tokens=reqs["a"][:66], want=[0, 65]), dict(id="b", tokens=reqs["b"][:2], want=[])], end=[]))
    steps.append(dict(entries=[dict(id="b", tokens=reqs["b"][2:], want=[6]), dict(id="a", tokens=reqs["a"][66:67], want=[0])], end=["b"]))
    steps.append(dict(entries=[dict(id="a", tokens=reqs["a"][67:], want=[])], end=["a"]))
    text = "".join(json.dumps(dict(s, step=i)) + "\n" for i, s in enumerate(steps))
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder("odd"), "--dtype", "float32", "--out", str(tmp_path),
                        "--max-tokens", "256"], input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert not os.path.exists(tmp_path / "2.f32")
    rows = [torch.frombuffer(bytearray(open(tmp_path / f"{i}.f32", "rb").read()), dtype=F32).view(2, 101) for i in (0, 1)]
    wa, wb = plain("odd", reqs["a"]), plain("odd", reqs["b"])
    check(rows[0], wa[[0, 65]], F32)
    check(rows[1], torch.stack([wb[8], wa[66]]), F32)


def test_generate_program(folder):
    p = tokens(12, 101, 9)
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "generate"), "--model", folder("odd"), "--prompt-ids", ",".join(map(str, p)), "--prompt-ids", "5",
                        "--max-tokens", "10", "--dtype", "float32"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    lines = [json.loads(l) for l in r.stdout.splitlines() if l.startswith("{")]
    assert [l["prompt"] for l in lines] == [p, [5]]
    for l in lines:
        follow("odd", l["prompt"], l["completion"], F32)
