"""Small configurations the Galirax tests share."""

from oracle import galirax_ref as G


def attention(heads, kv_heads, dim, vdim, rot, scale, base=10000.0, scaling=None, mlp=None):
    r = {"base": base, "dims": rot}
    if scaling is not None:
        r["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": r, "scale": scale}, "mlp": mlp}


def attention_2(heads, kv_heads, dim, vdim, rot, scale, size, keep, base=10000.0, mlp=None):
    layer = attention(heads, kv_heads, dim, vdim, rot, scale, base, mlp=mlp)
    layer["type"], layer["mixer"]["mask"] = "attention_2", {"size": size, "keep_first": keep}
    return layer


def lightning(heads, dim, vdim, decay, mlp=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def experts(ff, count, top, groups=1, keep=1, scale=1.0):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": count, "top": top, "groups": {"count": groups, "keep": keep}, "scale": scale}}


def config(width, vocab, layers, eps=1e-5, cap=20.0, loop=None):
    cfg = {"architecture": "Galirax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers, "logit_softcap": cap}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


CONFIGS = {
    # nothing a power of two, every layer unlike the others, layers without experts, a loop in the middle
    "odd": config(72, 101, [attention_2(6, 2, 20, 12, 12, 0.21, 37, 3, mlp=experts(20, 6, 3, 3, 2, 1.7)),
                            lightning(3, 12, 20, [0.5, 0.93, 0.999], mlp=experts(36, 9, 1, scale=0.8)),
                            attention(5, 1, 28, 36, 28, 0.17, base=500.0, scaling=(4.0, 1.0, 4.0, 64), mlp=experts(70, 10, 4, 5, 3, 2.0)),
                            lightning(2, 70, 50, [0.0, 1.0]),
                            attention_2(4, 4, 72, 130, 70, 0.1, 100, 70, base=300.0)], loop=(1, 3, 3)),
    # more query heads per key head than a pass takes, windows at page borders, wider heads, many experts
    "wide": config(192, 160, [lightning(2, 128, 128, [0.9, 0.998], mlp=experts(64, 32, 6, 8, 3, 2.5)),
                              attention_2(20, 2, 64, 128, 32, 0.11, 64, 1, mlp=experts(128, 16, 2, 2, 2, 1.0)),
                              attention(4, 1, 128, 64, 128, 0.09, mlp=experts(64, 70, 5, 7, 7, 1.0))], eps=1e-6, cap=8.0, loop=(0, 3, 1)),
    # beyond the fast kernels: wide keys, wide values, a wide state; these layers run on the plain kernels in bf16 too
    "plain": config(136, 90, [attention_2(2, 1, 270, 40, 100, 0.05, 30, 0, mlp=experts(40, 4, 2)), lightning(1, 300, 72, [0.97]), attention(3, 3, 40, 264, 8, 0.15)],
                    loop=(0, 2, 2)),
    # contractions longer than 1024 in every projection: the decode path's split-K workspace
    "long": config(1280, 300, [attention_2(12, 3, 128, 128, 64, 0.09, 50, 2, mlp=experts(300, 12, 3, 4, 2, 1.5)), lightning(9, 60, 128, [0.8 + 0.02 * i for i in range(9)]),
                               attention(20, 4, 64, 64, 64, 0.12, mlp=experts(1100, 3, 2))]),
}
_WEIGHTS = {}


def weights(name):
    if name not in _WEIGHTS:
        _WEIGHTS[name] = G.random_weights(CONFIGS[name], seed=len(name))
    return _WEIGHTS[name]
