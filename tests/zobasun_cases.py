"""Small configurations and helpers the Zobasun tests share."""
import json
import os

import torch
from safetensors.torch import save_file

from oracle import zobasun_ref as Z


def recurrent(width, blocks, conv, mlp=None):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": mlp}


def latent(heads, dim, rot, vdim, q_rank, kv_rank, scale, base=10000.0, mlp=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
         "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def config(width, vocab, layers, eps=1e-5, scale=3.0):
    return {"architecture": "Zobasun", "width": width, "vocab": vocab, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # nothing a power of two, every layer unlike the others, a shared cache two layers on, feed-forwards in other places
    "odd": config(72, 101, [latent(3, 20, 12, 40, 28, 36, 0.21, mlp=dense(100, 0.7)), recurrent(132, 3, 3, mlp=dense(52, 2.0)),
                            latent(5, 44, 12, 24, 50, 36, 0.13, kv_from=0), recurrent(60, 2, 2), latent(2, 70, 30, 90, 33, 130, 0.3, base=500.0)]),
    # sizes of the MFMA kernels with more heads than one tile, a single-block recurrence, one-tap convolution, attention first and last
    "wide": config(192, 160, [recurrent(128, 1, 1), latent(20, 64, 64, 128, 96, 256, 0.1, mlp=dense(192, 1.5)), recurrent(256, 2, 5),
                              latent(4, 128, 64, 64, 64, 512, 0.07)], eps=1e-6, scale=1.0),
    # beyond the MFMA kernels: wide latent, wide rotation, wide keys; these layers run on the plain kernels in bf16 too
    "plain": config(136, 90, [latent(2, 210, 80, 150, 40, 530, 0.08), recurrent(40, 5, 4, mlp=dense(72, 1.0)), latent(3, 30, 80, 20, 24, 530, 0.1, kv_from=0)]),
    # contractions longer than 1024, each projection with its own split: the decode path's shared split-K workspace
    "long": config(1280, 300, [recurrent(1536, 6, 4, mlp=dense(1700, 1.0)), latent(10, 64, 32, 128, 1100, 320, 0.1, mlp=dense(2100, 2.0)), recurrent(1100, 5, 3)],
                   scale=2.0),
}


def save_checkpoint(path, cfg, weights):
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


_WEIGHTS = {}


def weights(name):
    if name not in _WEIGHTS:
        _WEIGHTS[name] = Z.random_weights(CONFIGS[name], seed=len(name))
    return _WEIGHTS[name]
