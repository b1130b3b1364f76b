"""Plain restatement of the Galirax decoder (softmax attention with sinks, windows and kept first tokens; lightning attention; a sigmoid-routed
mixture of experts beside the mixer) in float64 on the CPU: one function per mechanism, token loops where the mechanism is sequential, no cache, no
paging, no batching.  It shares no code with nanovllm_hip; tests compare the framework with it.

Weights are a dict name -> tensor under the checkpoint's names ("embed", "l0.mix.q", ...), the configuration is the parsed config.json.
"""
import math

import torch

F64 = torch.float64


def layer_norm(x, w, b, eps):
    c = x - x.mean(dim=-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(dim=-1, keepdim=True) + eps) * w + b


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def frequencies(rot):
    """Turns per token (radians) of every pair; with `scaling`, long wavelengths are stretched by `factor`, short ones kept, a linear ramp between."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        s = rot.get("scaling")
        if s is not None:
            turns = s["original"] * f / (2.0 * math.pi)          # turns over the original length
            if turns < s["low"]:
                f = f / s["factor"]
            elif turns <= s["high"]:
                t = (turns - s["low"]) / (s["high"] - s["low"])
                f = (1.0 - t) * f / s["factor"] + t * f
        out.append(f)
    return out


def rotate_pairs(x, positions, freqs):
    """x [T, heads, D]: neighbours (2i, 2i + 1) turn by positions * freqs[i]; dimensions past the pairs pass."""
    out = x.clone()
    for i, f in enumerate(freqs):
        ang = positions.to(F64)[:, None] * f
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(ang) - v * torch.sin(ang)
        out[..., 2 * i + 1] = v * torch.cos(ang) + u * torch.sin(ang)
    return out


def visible(n, mask):
    """[query, key]: causal; with a mask also (nearer than `size`, or among the first `keep_first` tokens)."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    ok = j <= i
    if mask is not None:
        ok = ok & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    return ok


def sink_softmax(scores, sink):
    """Softmax over the last dimension whose denominator also holds exp(sink)."""
    top = torch.clamp(scores.max(dim=-1, keepdim=True).values, min=sink)
    e = torch.exp(scores - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink - top))


def attention_mixer(w, p, kind, m, h, eps):
    n, heads, kvh, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w[p + t].T for t in "qkv")
    if kind == "attention_2":
        q, k, v = (a + w[p + t + ".b"] for a, t in zip((q, k, v), "qkv"))
        q, k = rms_norm(q, w[p + "q.norm"], eps), rms_norm(k, w[p + "k.norm"], eps)
    pos, freqs = torch.arange(n), frequencies(m["rot"])
    q = rotate_pairs(q.view(n, heads, dim), pos, freqs)
    k = rotate_pairs(k.view(n, kvh, dim), pos, freqs)
    v = v.view(n, kvh, vdim)
    ok = visible(n, m["mask"] if kind == "attention_2" else None)
    out = []
    for g in range(heads):
        src = g // (heads // kvh)
        s = (q[:, g] @ k[:, src].T) * m["scale"]
        out.append(sink_softmax(s.masked_fill(~ok, float("-inf")), w[p + "sink"][g]) @ v[:, src])
    return torch.cat(out, dim=1) @ w[p + "o"].T


def silu(z):
    return z * torch.sigmoid(z)


def lightning_recurrence(q, k, v, decay, state=None):
    """One head.  S = decay S + k v^T, o = S^T q per token.  Returns (o [T, vdim], last S)."""
    s = torch.zeros(k.shape[1], v.shape[1], dtype=F64) if state is None else state
    out = []
    for t in range(q.shape[0]):
        s = decay * s + k[t][:, None] * v[t][None, :]
        out.append(s.T @ q[t])
    return torch.stack(out), s


def lightning_mixer(w, p, m, h, eps):
    n, heads, dim, vdim = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (silu(h @ w[p + t].T) for t in "qkv")
    outs = []
    for g in range(heads):
        a, b = slice(g * dim, (g + 1) * dim), slice(g * vdim, (g + 1) * vdim)
        outs.append(lightning_recurrence(q[:, a], k[:, a], v[:, b], m["decay"][g])[0])
    o = rms_norm(torch.cat(outs, dim=1), w[p + "norm"], eps)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def route(z, correction, r):
    """One token: logits [experts] -> (chosen experts, their weights, how far the nearest other choice was)."""
    s = torch.sigmoid(z)
    choice = (s + correction).tolist()
    groups, keep, top = r["groups"]["count"], r["groups"]["keep"], r["top"]
    size = len(z) // groups
    score = [sum(sorted(choice[g * size:(g + 1) * size])[-2:]) for g in range(groups)]
    rank = sorted(range(groups), key=lambda g: -score[g])
    open_to = sorted((e for e in range(len(z)) if e // size in rank[:keep]), key=lambda e: -choice[e])
    chosen = open_to[:top]
    gaps = [choice[chosen[-1]] - choice[open_to[top]]] if top < len(open_to) else []
    if keep < groups:
        gaps.append(score[rank[keep - 1]] - score[rank[keep]])
    weights = s[chosen]
    return chosen, weights / (weights.sum() + 1e-20) * r["scale"], min(gaps, default=math.inf)


def expert(w, p, h):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def moe(w, p, m, h, margins=None):
    out = torch.zeros_like(h)
    z = h @ w[p + "router"].T
    picks = {}
    for t in range(h.shape[0]):
        chosen, weights, gap = route(z[t], w[p + "correction"], m["router"])
        for e, g in zip(chosen, weights):
            picks.setdefault(e, []).append((t, g))
        if margins is not None:
            margins[t] = min(margins[t], gap)
    for e, rows in picks.items():
        t = [r[0] for r in rows]
        out[t] += torch.stack([r[1] for r in rows])[:, None] * expert(w, f"{p}e{e}.", h[t])
    return out


def layer_runs(cfg):
    """Layer indices in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return list(range(n))
    return list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n))


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


def forward(cfg, weights, tokens, collect=None, margins=None):
    """Logits [T, vocab] of one whole sequence; `collect`, a list, receives the residual stream after every layer run, `margins`, a list of a number per
    token, the closest call of its expert choices."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    for i in layer_runs(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        m = layer["mixer"]
        y = lightning_mixer(w, p + "mix.", m, h, eps) if layer["type"] == "lightning" else attention_mixer(w, p + "mix.", layer["type"], m, h, eps)
        if layer["mlp"] is not None:
            y = y + moe(w, p + "mlp.", layer["mlp"], h, margins)
        x = x + y
        if collect is not None:
            collect.append(x.clone())
    return softcap(layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T, cfg["logit_softcap"])


def random_weights(cfg, seed=0):
    """Small random bfloat16 weights of every tensor the configuration implies; norm weights, biases, sinks and corrections away from neutral."""
    gen = torch.Generator().manual_seed(seed)

    def rnd(*shape, scale=None):
        return (torch.randn(*shape, generator=gen) * (scale if scale is not None else shape[-1] ** -0.5)).bfloat16()

    def norm(name, n):
        w[name], w[name + ".b"] = 1.0 + rnd(n, scale=0.2), rnd(n, scale=0.2)

    d, w = cfg["width"], {}
    w["embed"] = rnd(cfg["vocab"], d, scale=1.0)
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        norm(f"l{i}.norm1", d)
        if layer["type"] == "lightning":
            a, b = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            w[p + "q"], w[p + "k"], w[p + "v"], w[p + "g"], w[p + "o"] = rnd(a, d), rnd(a, d), rnd(b, d), rnd(b, d), rnd(d, b)
            w[p + "norm"] = 1.0 + rnd(b, scale=0.2)
        else:
            a, c, b = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
            w[p + "q"], w[p + "k"], w[p + "v"], w[p + "o"] = rnd(a, d), rnd(c, d), rnd(b, d), rnd(d, m["heads"] * m["vdim"])
            w[p + "sink"] = 1.0 + rnd(m["heads"], scale=1.0)
            if layer["type"] == "attention_2":
                w[p + "q.b"], w[p + "k.b"], w[p + "v.b"] = rnd(a, scale=0.3), rnd(c, scale=0.3), rnd(b, scale=0.3)
                w[p + "q.norm"], w[p + "k.norm"] = 1.0 + rnd(a, scale=0.2), 1.0 + rnd(c, scale=0.2)
        if layer["mlp"] is not None:
            ff, r, q = layer["mlp"]["expert"]["ff"], layer["mlp"]["router"], f"l{i}.mlp."
            w[q + "router"], w[q + "correction"] = rnd(r["experts"], d), rnd(r["experts"], scale=0.5)
            for e in range(r["experts"]):
                w[f"{q}e{e}.gate"], w[f"{q}e{e}.up"], w[f"{q}e{e}.down"] = rnd(ff, d), rnd(ff, d), rnd(d, ff)
    norm("final.norm", d)
    w["head"] = rnd(cfg["vocab"], d, scale=2.0 * d ** -0.5)
    return w
