"""Small random hybrid models and error measures shared by the hybrid tests."""
from __future__ import annotations

import torch


def attention(heads=4, kv_heads=2, dim=32, vdim=24, rot=8, base=1000.0, scale=None, ff=72):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "scale": 4.0 / dim ** 0.5 if scale is None else scale,
                      "rot": {"dims": rot, "base": base}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads=4, kv_heads=2, dim=24, vdim=40, conv=4, ff=72):
    return {"type": "delta",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(layers, width=96, vocab=131, loop=None, mult=0.6, eps=1e-5, **kw):
    d = {"architecture": "Fonapel", "layers": layers, "norm": {"eps": eps},
         "residual_mult": mult, "vocab": vocab, "width": width, **kw}
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


# sizes that are not multiples of anything, equal and unequal head sizes, every loop position
CASES = {
    "mixed": model([attention(), delta(), attention(heads=2, kv_heads=2), delta()],
                   loop=(1, 3, 2)),
    "loop_first": model([delta(heads=6, kv_heads=3, dim=20, vdim=12, conv=3),
                         attention(heads=6, kv_heads=1, dim=40, vdim=72, rot=40, ff=50)],
                        width=76, vocab=97, loop=(0, 2, 3)),
    "loop_last_once": model([attention(dim=20, vdim=20, rot=4, ff=0), delta(conv=1, ff=33)],
                            width=61, vocab=83, loop=(1, 2, 1), mult=1.0),
    "no_loop": model([attention(heads=3, kv_heads=3, dim=66, vdim=30, rot=64, ff=128),
                      delta(heads=3, kv_heads=3, dim=64, vdim=64, conv=2, ff=0)],
                     width=128, vocab=256, mult=0.35, eps=1e-3),
    "wide_heads": model([attention(heads=20, kv_heads=1, dim=128, vdim=128, rot=128),
                         delta(heads=2, kv_heads=1, dim=128, vdim=128, conv=7),
                         attention(heads=2, kv_heads=1, dim=192, vdim=136, rot=0)],
                        width=64, vocab=70, loop=(0, 1, 2)),
}


def weights_of(cfg_dict, seed=0):
    """(config, getter, {name: tensor}) of seeded random bf16 weights."""
    from cake_amd.models.hybrid.config import from_config
    from cake_amd.models.hybrid.weights import random_tensors, tensor_shapes
    cfg = from_config(cfg_dict)
    get = random_tensors(cfg, seed=seed)
    return cfg, get, {n: get(n) for n in tensor_shapes(cfg)}


def tokens(n, vocab, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def rel_rms(got, want):
    """Largest per-row rms of the difference (mean taken off) over the rows' overall rms."""
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return float(d.pow(2).mean(-1).sqrt().max() / want.pow(2).mean().sqrt())
