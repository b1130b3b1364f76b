"""Small configurations the Kekapel tests share."""

from oracle import kekapel_ref as K


def attention(heads, kv_heads, dim, vdim, size, cap, scale, mlp=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size}, "softcap": cap, "scale": scale}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def experts(ff, limit, count, top):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": count, "top": top}}


def config(width, vocab, layers, eps=1e-5, scale=3.0, mult=0.6, positions=512, loop=None):
    cfg = {"architecture": "Kekapel", "width": width, "vocab": vocab, "embedding": {"scale": scale}, "norm": {"eps": eps}, "residual_mult": mult, "max_positions": positions,
           "layers": layers}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


CONFIGS = {
    # nothing a power of two, every layer unlike the others, a layer without a feed-forward, a loop that starts the model
    "odd": config(72, 101, [attention(6, 2, 20, 12, 37, 5.0, 0.31, mlp=experts(20, 0.7, 6, 3)), attention(5, 1, 28, 36, 100, 2.5, 0.17, mlp=dense(50)),
                            attention(3, 3, 40, 24, 1, 9.0, 0.2), attention(4, 4, 72, 130, 64, 1.5, 0.25, mlp=experts(36, 3.0, 9, 1)),
                            attention(2, 1, 64, 64, 300, 30.0, 0.4, mlp=dense(70))], loop=(0, 3, 3)),
    # more query heads per key head than a pass takes, more heads than a tile of the mixing product, windows at page borders, wide heads, many experts
    "wide": config(192, 160, [attention(20, 2, 64, 128, 64, 8.0, 0.2, mlp=experts(64, 1.5, 32, 6)), attention(4, 1, 128, 64, 129, 15.0, 0.1, mlp=dense(192)),
                              attention(12, 3, 192, 64, 65, 4.0, 0.1, mlp=experts(128, 0.4, 70, 5)), attention(8, 4, 70, 200, 128, 6.0, 0.15, mlp=dense(320))],
                   eps=1e-6, scale=1.0, mult=1.0, positions=1024, loop=(1, 3, 2)),
    # beyond the fast kernels: wide keys, wide values, many heads; in bf16 too these layers, or their prompts, run on the plain kernels
    "plain": config(136, 90, [attention(2, 1, 270, 40, 30, 3.0, 0.1, mlp=experts(40, 2.0, 4, 2)), attention(40, 8, 16, 24, 90, 4.0, 0.3, mlp=dense(100)),
                              attention(70, 10, 8, 8, 50, 4.0, 0.4), attention(3, 3, 40, 264, 150, 6.0, 0.2)], loop=(1, 2, 4)),
    # contractions longer than 1024 in every projection: the decode path's split-K workspace
    "long": config(1280, 300, [attention(12, 3, 128, 128, 50, 7.0, 0.12, mlp=experts(300, 1.0, 12, 3)), attention(20, 4, 64, 64, 70, 7.0, 0.12, mlp=dense(1100))], scale=2.0),
}
_WEIGHTS = {}


def weights(name):
    if name not in _WEIGHTS:
        _WEIGHTS[name] = K.random_weights(CONFIGS[name], seed=len(name))
    return _WEIGHTS[name]
