"""Plain restatement of the Zaposun decoder (RWKV-style time mixing; chunked softmax attention with rotated values beside a selective scan; hyper-connections, grouped
norms, token shift, a bigram embedding) in float64 on the CPU: one function per mechanism, token by token where the mechanism is a recurrence, no cache, no paging,
no batching.  It shares no code with nanovllm_hip; tests compare the framework with it.

Weights are a dict name -> tensor under the checkpoint's names ("embed", "l0.mix.r", ...), the configuration is the parsed config.json.
"""
import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    """Every one of `groups` equal consecutive parts of the last dimension by its own root mean square, the whole times w."""
    part = x.shape[-1] // groups
    return torch.cat([rms(x[..., g * part:(g + 1) * part], eps) for g in range(groups)], dim=-1) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0.0)


# ---------------------------------------------------------------- embedding, streams, shift
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    return [buckets if i == 0 else (tokens[i - 1] * mul_prev + t * mul_cur) % buckets for i, t in enumerate(tokens)]


def embedding(cfg, w, tokens):
    b = cfg["embedding"]["bigram"]
    return w["embed"][torch.as_tensor(tokens)] + w["bigram"][torch.as_tensor(bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"]))]


def read_streams(xs, weights):
    """xs [streams, T, width] -> what a sublayer reads."""
    return sum(weights[s] * xs[s] for s in range(xs.shape[0]))


def update_streams(xs, mix, out, y):
    """mix is indexed [from, to]."""
    n = xs.shape[0]
    return torch.stack([sum(mix[s, t] * xs[s] for s in range(n)) + out[t] * y for t in range(n)])


def previous(h):
    """Row t holds row t - 1, row 0 zeros."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def lerp_previous(h, mu):
    return h + (previous(h) - h) * mu


# ---------------------------------------------------------------- time mixing with data-dependent decay
def wkv_scan(r, k, v, decay, u, state=None):
    """One head: r, k, decay [T, dk], v [T, dv], u [dk] -> (o [T, dv], state behind the last token)."""
    s = torch.zeros(k.shape[1], v.shape[1], dtype=F64) if state is None else state
    o = []
    for t in range(r.shape[0]):
        kv = torch.outer(k[t], v[t])
        o.append((s + u[:, None] * kv).T @ r[t])
        s = decay[t][:, None] * s + kv
    return torch.stack(o), s


def wkv_decay(w, p, mixed):
    return torch.exp(-torch.exp(torch.tanh(mixed @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]))


def wkv_mixer(w, p, m, h, eps):
    n, heads, dim = h.shape[0], m["heads"], m["dim"]
    mixed = {c: lerp_previous(h, w[p + "mu." + c]) for c in "rkvgw"}
    r, k, v = ((mixed[c] @ w[p + c].T).view(n, heads, dim) for c in "rkv")
    decay = wkv_decay(w, p, mixed["w"]).view(n, heads, dim)
    o = torch.stack([wkv_scan(r[:, i], k[:, i], v[:, i], decay[:, i], w[p + "u"][i])[0] for i in range(heads)], dim=1)
    return (rms(o, eps).reshape(n, -1) * w[p + "norm"] * silu(mixed["g"] @ w[p + "g"].T)) @ w[p + "o"].T


# ---------------------------------------------------------------- chunked attention with rotated values
def rotate_half(x, positions, dims, base):
    """x [T, heads, d]: dimension i turns with dimension i + dims / 2, i < dims / 2; the rest passes."""
    half = dims // 2
    angle = positions[:, None].double() * torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=F64)
    c, s = angle.cos()[:, None], angle.sin()[:, None]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def visible(n, size):
    """[query, key]: no later token, none of another chunk."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & (i // size == j // size)


def attend(q, k, v, scale, ok):
    """q [T, heads, dim], k and v [S, kv heads, .] -> [T, heads, vdim]."""
    ratio = q.shape[1] // k.shape[1]
    out = []
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h // ratio].T * scale).masked_fill(~ok, float("-inf"))
        out.append(torch.softmax(s, dim=-1) @ v[:, h // ratio])
    return torch.stack(out, dim=1)


def attention_mixer(w, p, m, h, eps):
    n, pos, base = h.shape[0], torch.arange(h.shape[0]), m["rot"]["base"]
    q, k, v = ((h @ w[p + t].T).view(n, c, d) for t, c, d in (("q", m["heads"], m["dim"]), ("k", m["kv_heads"], m["dim"]), ("v", m["kv_heads"], m["vdim"])))
    q, k = (rotate_half(rms(t, eps) * w[p + name], pos, m["rot"]["dims"], base) for t, name in ((q, "q.norm"), (k, "k.norm")))
    o = attend(q, k, rotate_half(v, pos, m["vdim"], base), m["scale"], visible(n, m["mask"]["size"]))
    return rotate_half(o, -pos, m["vdim"], base).reshape(n, -1) @ w[p + "o"].T


# ---------------------------------------------------------------- selective scan
def causal_conv(x, w, b):
    """x [T, channels], w [channels, taps], the last column on the current token."""
    taps, out = w.shape[1], torch.zeros_like(x) + b
    for back in range(taps):
        if back < x.shape[0]:
            out[back:] += x[:x.shape[0] - back] * w[:, taps - 1 - back]
    return out


def selective_scan(x, dt, a, b, c, d, state=None):
    """x, dt [T, channels], a [channels, n], b, c [T, n], d [channels] -> (y [T, channels], state behind the last token)."""
    s = torch.zeros_like(a) if state is None else state
    y = []
    for t in range(x.shape[0]):
        s = torch.exp(dt[t][:, None] * a) * s + (dt[t] * x[t])[:, None] * b[t][None, :]
        y.append(s @ c[t] + d * x[t])
    return torch.stack(y), s


def mamba_mixer(w, p, m, h):
    inner, rank, n = m["inner"], m["dt_rank"], m["state"]
    x, z = (h @ w[p + "in"].T).split(inner, dim=1)
    x = silu(causal_conv(x, w[p + "conv"], w[p + "conv.b"]))
    dt, b, c = (x @ w[p + "x"].T).split([rank, n, n], dim=1)
    dt = softplus(dt @ w[p + "dt"].T + w[p + "dt.b"])
    y, _ = selective_scan(x, dt, -torch.exp(w[p + "A_log"]), b, c, w[p + "D"])
    return (y * silu(z)) @ w[p + "o"].T


def parallel_mixer(w, p, m, h, eps):
    left, right = attention_mixer(w, p + "left.", m["left"], h, eps), mamba_mixer(w, p + "right.", m["right"], h)
    return 0.5 * (rms(left, eps) * w[p + "left.out"] + rms(right, eps) * w[p + "right.out"])


def dense(w, p, h):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


# ---------------------------------------------------------------- the model
def forward(cfg, weights, tokens, collect=None):
    """Logits [T, vocab] of one whole sequence; `collect`, a list, receives the sum of the streams after every layer."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    xs = torch.stack([embedding(cfg, w, tokens)] * cfg["streams"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = lerp_previous(group_norm(read_streams(xs, w[p + "hc1.in"]), w[p + "norm1"], groups, eps), w[p + "shift"])
        y = (wkv_mixer if layer["type"] == "wkv" else parallel_mixer)(w, p + "mix.", layer["mixer"], h, eps)
        xs = update_streams(xs, w[p + "hc1.mix"], w[p + "hc1.out"], y)
        if layer["mlp"] is not None:
            y = dense(w, p + "mlp.", group_norm(read_streams(xs, w[p + "hc2.in"]), w[p + "norm2"], groups, eps))
            xs = update_streams(xs, w[p + "hc2.mix"], w[p + "hc2.out"], y)
        if collect is not None:
            collect.append(xs.sum(dim=0))
    return group_norm(xs.sum(dim=0), w["final.norm"], groups, eps) @ w["head"].T * cfg["logit_scale"]


def random_weights(cfg, seed=0):
    """Small random bfloat16 weights of every tensor the configuration implies; norms, mixes and constants away from neutral."""
    gen = torch.Generator().manual_seed(seed)

    def rnd(*shape, scale=None):
        return (torch.randn(*shape, generator=gen) * (scale if scale is not None else shape[-1] ** -0.5)).bfloat16()

    def uni(*shape, lo=0.0, hi=1.0):
        return (torch.rand(*shape, generator=gen) * (hi - lo) + lo).bfloat16()

    d, n, w = cfg["width"], cfg["streams"], {}
    w["embed"], w["bigram"] = rnd(cfg["vocab"], d, scale=1.0), rnd(cfg["embedding"]["bigram"]["buckets"] + 1, d, scale=0.6)
    for i, layer in enumerate(cfg["layers"]):
        m, l, p = layer["mixer"], f"l{i}.", f"l{i}.mix."
        w[l + "shift"] = uni(d, lo=0.0, hi=0.8)
        for q in ("1", "2") if layer["mlp"] is not None else ("1",):
            w[l + "norm" + q] = 1.0 + rnd(d, scale=0.2)
            w[f"{l}hc{q}.in"], w[f"{l}hc{q}.out"] = 1.0 / n + rnd(n, scale=0.15), 1.0 + rnd(n, scale=0.3)
            w[f"{l}hc{q}.mix"] = (0.8 * torch.eye(n)).bfloat16() + rnd(n, n, scale=0.15)
        if layer["type"] == "wkv":
            a, rank = m["heads"] * m["dim"], cfg.get("_decay_rank", 12)
            for c in "rkvgw":
                w[p + "mu." + c] = uni(d, hi=0.9)
            for c in "rkvg":
                w[p + c] = rnd(a, d)
            w[p + "w1"], w[p + "w2"], w[p + "w0"] = rnd(rank, d), rnd(a, rank, scale=0.7 * rank ** -0.5), uni(a, lo=-6.0, hi=0.0)
            w[p + "u"], w[p + "norm"], w[p + "o"] = 0.5 + rnd(m["heads"], m["dim"], scale=0.5), 1.0 + rnd(a, scale=0.2), rnd(d, a)
        else:
            q, f = m["left"], p + "left."
            w[f + "q"], w[f + "k"], w[f + "v"] = rnd(q["heads"] * q["dim"], d), rnd(q["kv_heads"] * q["dim"], d), rnd(q["kv_heads"] * q["vdim"], d)
            w[f + "q.norm"], w[f + "k.norm"] = 1.2 + rnd(q["dim"], scale=0.4), 1.2 + rnd(q["dim"], scale=0.4)
            w[f + "o"], w[f + "out"] = rnd(d, q["heads"] * q["vdim"]), 0.9 + rnd(d, scale=0.2)
            q, f = m["right"], p + "right."
            e, s = q["inner"], q["state"]
            w[f + "in"], w[f + "conv"], w[f + "conv.b"] = rnd(2 * e, d), rnd(e, q["conv"], scale=0.6), rnd(e, scale=0.1)
            w[f + "x"], w[f + "dt"], w[f + "dt.b"] = rnd(q["dt_rank"] + 2 * s, e), rnd(e, q["dt_rank"]), uni(e, lo=-4.0, hi=-0.5)
            w[f + "A_log"], w[f + "D"] = uni(e, s, lo=-4.0, hi=1.5), 0.8 + rnd(e, scale=0.2)
            w[f + "o"], w[f + "out"] = rnd(d, e), 0.9 + rnd(d, scale=0.2)
        if layer["mlp"] is not None:
            f = layer["mlp"]["ff"]
            w[l + "mlp.gate"], w[l + "mlp.up"], w[l + "mlp.down"] = rnd(f, d), rnd(f, d), rnd(d, f)
    w["final.norm"], w["head"] = 1.0 + rnd(d, scale=0.3), rnd(cfg["vocab"], d, scale=2.0 * d ** -0.5)
    return w
