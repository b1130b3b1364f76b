"""Plain restatement of the Zobasun decoder (gated linear recurrence blocks + latent attention) in float64 on the CPU: one function
per mechanism, token loops where the mechanism is sequential, no cache, no paging, no batching.  It shares no code with nanovllm_hip;
tests compare the framework with it.

Weights are a dict name -> tensor under the checkpoint's names ("embed", "l0.mix.x", ...), the configuration is the parsed config.json.
"""
import math

import torch

F64 = torch.float64


def rms_norm(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def zero_centred_norm(x, w, eps):
    """RMS norm whose stored weight is the deviation from one."""
    return rms_norm(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(v, taps, bias):
    """v [T, C], taps [C, K]: out[t] = sum_j taps[:, j] * v[t - (K - 1) + j] + bias, rows before the start count as zero."""
    n, k = v.shape[0], taps.shape[1]
    out = torch.zeros_like(v)
    for t in range(n):
        for j in range(k):
            s = t - (k - 1) + j
            if s >= 0:
                out[t] += taps[:, j] * v[s]
    return out + bias


def block_gate(u, w, b):
    """sigmoid of a block-diagonal linear map: u [T, B*S], w [B, S, S] ([out, in]), b [B, S]."""
    blocks, size = b.shape
    parts = [u[:, i * size:(i + 1) * size] @ w[i].T + b[i] for i in range(blocks)]
    return torch.sigmoid(torch.cat(parts, dim=1))


def rglru_recurrence(u, r, i, lam, state=None):
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t with log a_t = -8 r_t softplus(lam).  Returns (all S [T, W], last S)."""
    s = torch.zeros_like(u[0]) if state is None else state
    rate = torch.log1p(torch.exp(-lam.abs())) + lam.clamp(min=0)
    out = []
    for t in range(u.shape[0]):
        log_a = -8.0 * r[t] * rate
        s = torch.exp(log_a) * s + torch.sqrt(-torch.expm1(2.0 * log_a)) * i[t] * u[t]
        out.append(s)
    return torch.stack(out), s


def rglru_mixer(w, p, h):
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"])
    r = block_gate(u, w[p + "ra"], w[p + "ra.b"])
    i = block_gate(u, w[p + "ri"], w[p + "ri.b"])
    s, _ = rglru_recurrence(u, r, i, w[p + "lam"])
    return (s * y) @ w[p + "o"].T


def rotate_pairs(x, positions, dims, base):
    """x [..., T, D]: the pair (2i, 2i+1), i < dims/2, turns by positions * base^(-2i/dims); the rest passes."""
    out = x.clone()
    for i in range(dims // 2):
        ang = positions.to(F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(ang), torch.sin(ang)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def latent_rows(w, p, m, h, eps):
    """What a latent-attention layer caches per token: (normed latent [T, kv_rank], rotated shared key part [T, rot_dim])."""
    a = h @ w[p + "dkv"].T
    c = rms_norm(a[:, :m["kv_rank"]], eps) * w[p + "dkv.norm"]
    k = rotate_pairs(a[:, m["kv_rank"]:], torch.arange(h.shape[0]), m["rot"]["dims"], m["rot"]["base"])
    return c, k


def latent_mixer(w, p, m, h, eps, rows):
    n, heads, dim, rot, vdim = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, k_rot = rows
    q = (rms_norm(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T
    q = q.view(n, heads, dim + rot)
    k = (c @ w[p + "uk"].T).view(n, heads, dim)
    v = (c @ w[p + "uv"].T).view(n, heads, vdim)
    visible = torch.ones(n, n, dtype=torch.bool).tril()
    pos = torch.arange(n)
    out = []
    for g in range(heads):
        q_rot = rotate_pairs(q[:, g, dim:], pos, m["rot"]["dims"], m["rot"]["base"])
        score = (q[:, g, :dim] @ k[:, g].T + q_rot @ k_rot.T) * m["scale"]
        out.append(torch.softmax(score.masked_fill(~visible, float("-inf")), dim=-1) @ v[:, g])
    return torch.cat(out, dim=1) @ w[p + "o"].T


def clamped_glu(gate, up, limit):
    g = torch.clamp(gate, max=limit)
    u = torch.clamp(up, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def dense_mlp(w, p, m, h):
    return clamped_glu(h @ w[p + "gate"].T, h @ w[p + "up"].T, m["limit"]) @ w[p + "down"].T


def forward(cfg, weights, tokens, collect=None):
    """Logits [T, vocab] of one whole sequence; `collect`, a list, receives the residual stream after every layer."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    latents = {}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        if layer["type"] == "rglru":
            y = rglru_mixer(w, p, x)
        else:
            if "kv_from" in m:
                rows = latents[m["kv_from"]]
            else:
                rows = latents[i] = latent_rows(w, p, m, x, eps)
            y = latent_mixer(w, p, m, x, eps, rows)
        x = x + zero_centred_norm(y, w[f"l{i}.norm1"], eps)
        if layer["mlp"] is not None:
            x = x + zero_centred_norm(dense_mlp(w, f"l{i}.mlp.", layer["mlp"], x), w[f"l{i}.norm2"], eps)
        if collect is not None:
            collect.append(x.clone())
    return zero_centred_norm(x, w["final.norm"], eps) @ w["head"].T


def random_weights(cfg, seed=0):
    """Small random bfloat16 weights of every tensor the configuration implies; decay rates spread so that both short and long memories
    occur, norm weights away from their neutral value."""
    gen = torch.Generator().manual_seed(seed)

    def rnd(*shape, scale=None):
        return (torch.randn(*shape, generator=gen) * (scale if scale is not None else shape[-1] ** -0.5)).bfloat16()

    d, w = cfg["width"], {}
    w["embed"] = rnd(cfg["vocab"], d, scale=1.0)
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        w[f"l{i}.norm1"] = rnd(d, scale=0.2)
        if layer["type"] == "rglru":
            width, blocks, size = m["width"], m["blocks"], m["width"] // m["blocks"]
            for n in "yx":
                w[p + n], w[p + n + ".b"] = rnd(width, d), rnd(width, scale=0.3)
            w[p + "conv"], w[p + "conv.b"] = rnd(width, m["conv"]), rnd(width, scale=0.3)
            for n in ("ra", "ri"):
                w[p + n], w[p + n + ".b"] = rnd(blocks, size, size), rnd(blocks, size, scale=0.5)
            w[p + "lam"] = (torch.rand(width, generator=gen) * 8.0 - 7.0).bfloat16()
            w[p + "o"] = rnd(d, width)
        else:
            h, qr, kr = m["heads"], m["q_rank"], m["kv_rank"]
            w[p + "dq"], w[p + "dq.norm"] = rnd(qr, d), 1.0 + rnd(qr, scale=0.2)
            w[p + "uq"] = rnd(h * (m["dim"] + m["rot_dim"]), qr)
            if "kv_from" not in m:
                w[p + "dkv"], w[p + "dkv.norm"] = rnd(kr + m["rot_dim"], d), 1.0 + rnd(kr, scale=0.2)
            w[p + "uk"], w[p + "uv"] = rnd(h * m["dim"], kr), rnd(h * m["vdim"], kr)
            w[p + "o"] = rnd(d, h * m["vdim"])
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            w[f"l{i}.norm2"] = rnd(d, scale=0.2)
            w[f"l{i}.mlp.gate"], w[f"l{i}.mlp.up"], w[f"l{i}.mlp.down"] = rnd(ff, d), rnd(ff, d), rnd(d, ff)
    w["final.norm"] = rnd(d, scale=0.2)
    w["head"] = rnd(cfg["vocab"], d)
    return w
