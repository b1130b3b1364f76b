"""Plain restatement of the Kekapel decoder (windowed softmax attention whose soft-capped scores are mixed across the heads, dense PolyNorm feed-forwards or a
softmax-routed mixture of clamped gated experts, layer norms before and after every sublayer, a looped run of layers) in float64 on the CPU: one function per
mechanism, no cache, no paging, no batching.  It shares no code with nanovllm_hip; tests compare the framework with it.

Weights are a dict name -> tensor under the checkpoint's names ("embed", "l0.mix.q", ...), the configuration is the parsed config.json.
"""
import math

import torch

F64 = torch.float64


def layer_norm(x, w, b, eps):
    c = x - x.mean(dim=-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(dim=-1, keepdim=True) + eps) * w + b


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def softcap(s, cap):
    return cap * torch.tanh(s / cap)


def mix_heads(s, talk):
    """s [heads, queries, keys] -> row h is the sum over g of talk[h, g] s[g]."""
    out = torch.zeros_like(s)
    for h in range(s.shape[0]):
        for g in range(s.shape[0]):
            out[h] += talk[h, g] * s[g]
    return out


def visible(n, size):
    """[query, key]: a token sees itself and the size - 1 tokens before it."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & (i - j < size)


def attend(q, k, v, talk, scale, cap, ok):
    """q [T, heads, dim], k and v [S, kv heads, .] already normed, ok [T, S] -> [T, heads, vdim]."""
    heads, ratio = q.shape[1], q.shape[1] // k.shape[1]
    s = torch.stack([softcap(q[:, h] @ k[:, h // ratio].T * scale, cap) for h in range(heads)])
    p = torch.softmax(mix_heads(s, talk).masked_fill(~ok, float("-inf")), dim=-1)
    return torch.stack([p[h] @ v[:, h // ratio] for h in range(heads)], dim=1)


def attention_mixer(w, p, m, h, eps):
    n = h.shape[0]
    q, k, v = ((h @ w[p + t].T).view(n, c, d) for t, c, d in (("q", m["heads"], m["dim"]), ("k", m["kv_heads"], m["dim"]), ("v", m["kv_heads"], m["vdim"])))
    q, k = unit_rms(q, eps) * w[p + "q.norm"], unit_rms(k, eps) * w[p + "k.norm"]
    o = attend(q, k, v, w[p + "talk"], m["scale"], m["softcap"], visible(n, m["mask"]["size"]))
    return o.reshape(n, -1) @ w[p + "o"].T


def poly_norm(z, coef, eps):
    return coef[0] * unit_rms(z, eps) + coef[1] * unit_rms(z ** 2, eps) + coef[2] * unit_rms(z ** 3, eps) + coef[3]


def dense(w, p, h, eps):
    return poly_norm(h @ w[p + "up"].T, w[p + "act"], eps) @ w[p + "down"].T


def clamped_unit(g, u, limit):
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def expert(w, p, h, limit):
    return clamped_unit(h @ w[p + "gate"].T, h @ w[p + "up"].T, limit) @ w[p + "down"].T


def route(z, top):
    """One token: logits [experts] -> (chosen experts, their weights, how far the nearest other choice was)."""
    order = sorted(range(len(z)), key=lambda e: -z[e].item())
    gap = (z[order[top - 1]] - z[order[top]]).item() if top < len(z) else math.inf
    return order[:top], torch.softmax(z[order[:top]], dim=0), gap


def moe(w, p, m, h, margins=None):
    out = torch.zeros_like(h)
    z = h @ w[p + "router"].T + w[p + "router.b"]
    picks = {}
    for t in range(h.shape[0]):
        chosen, weights, gap = route(z[t], m["router"]["top"])
        for e, g in zip(chosen, weights):
            picks.setdefault(e, []).append((t, g))
        if margins is not None:
            margins[t] = min(margins[t], gap)
    for e, rows in picks.items():
        t = [r[0] for r in rows]
        out[t] += torch.stack([r[1] for r in rows])[:, None] * expert(w, f"{p}e{e}.", h[t], m["expert"]["limit"])
    return out


def layer_runs(cfg):
    """(layer, pass if the layer starts one) in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return [(i, None) for i in range(a)] + [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)] + [(i, None) for i in range(b, n)]


def embedding(cfg, w, tokens):
    return w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"] + w["pos"][:len(tokens)]


def forward(cfg, weights, tokens, collect=None, margins=None):
    """Logits [T, vocab] of one whole sequence; `collect`, a list, receives the residual stream after every layer run, `margins`, a list of a number per
    token, the closest call of its expert choices."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    first = x = embedding(cfg, w, tokens)

    def norm(name, t):
        return layer_norm(t, w[name], w[name + ".b"], eps)
    for i, start in layer_runs(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        if start is not None:
            x = x + w["loop.step"][start] + (first if start > 0 else 0.0)
        x = x + mult * norm(p + "norm1b", attention_mixer(w, p + "mix.", layer["mixer"], norm(p + "norm1", x), eps))
        if layer["mlp"] is not None:
            h = norm(p + "norm2", x)
            y = dense(w, p + "mlp.", h, eps) if layer["mlp"]["kind"] == "dense" else moe(w, p + "mlp.", layer["mlp"], h, margins)
            x = x + mult * norm(p + "norm2b", y)
        if collect is not None:
            collect.append(x.clone())
    return norm("final.norm", x) @ w["head"].T


def random_weights(cfg, seed=0):
    """Small random bfloat16 weights of every tensor the configuration implies; norm weights, biases and mixing matrices away from neutral."""
    gen = torch.Generator().manual_seed(seed)

    def rnd(*shape, scale=None):
        return (torch.randn(*shape, generator=gen) * (scale if scale is not None else shape[-1] ** -0.5)).bfloat16()

    def norm(name, n):
        w[name], w[name + ".b"] = 1.0 + rnd(n, scale=0.2), rnd(n, scale=0.2)

    d, w = cfg["width"], {}
    w["embed"], w["pos"] = rnd(cfg["vocab"], d, scale=1.0 / cfg["embedding"]["scale"]), rnd(cfg["max_positions"], d, scale=0.5)
    if cfg.get("loop") is not None:
        w["loop.step"] = rnd(cfg["loop"]["times"], d, scale=0.5)
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if layer["mlp"] is not None else ()):
            norm(f"l{i}.{n}", d)
        h, g, a, b = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        w[p + "q"], w[p + "k"], w[p + "v"], w[p + "o"] = rnd(h * a, d), rnd(g * a, d), rnd(g * b, d), rnd(d, h * b)
        w[p + "q.norm"], w[p + "k.norm"] = 1.0 + rnd(a, scale=0.3), 1.0 + rnd(a, scale=0.3)
        w[p + "talk"] = torch.eye(h).bfloat16() + rnd(h, h, scale=0.6 * h ** -0.5)
        if layer["mlp"] is not None:
            q, mlp = f"l{i}.mlp.", layer["mlp"]
            if mlp["kind"] == "dense":
                w[q + "up"], w[q + "down"], w[q + "act"] = rnd(mlp["ff"], d), rnd(d, mlp["ff"]), torch.tensor([0.7, -0.4, 0.5, 0.2]).bfloat16() + rnd(4, scale=0.2)
            else:
                ff, e = mlp["expert"]["ff"], mlp["router"]["experts"]
                w[q + "router"], w[q + "router.b"] = rnd(e, d), rnd(e, scale=0.5)
                for k in range(e):
                    w[f"{q}e{k}.gate"], w[f"{q}e{k}.up"], w[f"{q}e{k}.down"] = rnd(ff, d), rnd(ff, d), rnd(d, ff)
    norm("final.norm", d)
    w["head"] = rnd(cfg["vocab"], d, scale=2.0 * d ** -0.5)
    return w
