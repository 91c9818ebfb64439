"""Small random Nubosun models for the tests (saved and checked by _layer_stack)."""
from __future__ import annotations

import numpy as np

import _layer_stack as T

YARN = {"factor": 3.0, "original": 64, "fast": 8.0, "slow": 0.5}


def latent(heads=4, dim=24, rot=8, vdim=16, rank=40, base=1000.0, scaling=YARN, scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
         "scale": scale or (dim + rot) ** -0.5, "rot": {"base": base, "dims": rot}}
    if scaling:
        m["rot"]["scaling"] = dict(scaling)
    return m


def mamba(inner=72, state=12, dt_rank=6, conv=4):
    return {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}


def dense(ff=56, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def config(layers, *, width=88, vocab=150, streams=3, scale=3.0, cap=8.0, loop=None, eps=1e-5):
    """layers: (mixer, feed-forward or None)."""
    c = {"architecture": "Nubosun", "vocab": vocab, "width": width, "norm": {"eps": eps},
         "embedding": {"scale": scale}, "streams": streams, "logit_softcap": cap,
         "layers": [{"type": "mamba1" if "inner" in a else "latent_attention", "mixer": a, "mlp": m}
                    for a, m in layers]}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


def weights(cfg, seed):
    """Random bf16 values; every vector away from the value that would hide it."""
    rng = np.random.default_rng(seed)
    W, S, w = cfg["width"], cfg["streams"], {}

    def normal(name, *shape, mean=0.0, std=1.0):
        w[name] = (mean + std * rng.standard_normal(shape)).astype(np.float32)

    def lin(name, n, k, g=1.0):
        normal(name, n, k, std=g / np.sqrt(k))

    def sublayer(p, q):
        normal(f"{p}norm{q}", W, mean=1.0, std=0.3)
        normal(f"{p}ls{q}", W, mean=0.8, std=0.3)
        normal(f"{p}hc{q}.in", S, mean=0.6, std=0.15)
        normal(f"{p}hc{q}.out", S, mean=0.6, std=0.3)
        w[f"{p}hc{q}.mix"] = (0.8 * np.eye(S) + 0.2 / np.sqrt(S) * rng.standard_normal((S, S))
                              ).astype(np.float32)

    normal("embed", cfg["vocab"], W)
    for i, L in enumerate(cfg["layers"]):
        p, a, f = f"l{i}.", L["mixer"], L.get("mlp")
        sublayer(p, 1)
        if L["type"] == "mamba1":
            n, s, r = a["inner"], a["state"], a["dt_rank"]
            lin(p + "mix.in", 2 * n, W)
            lin(p + "mix.conv", n, a["conv"])
            normal(p + "mix.conv.b", n, std=0.3)
            lin(p + "mix.x", r + 2 * s, n, 1.2)
            lin(p + "mix.dt", n, r)
            normal(p + "mix.dt.b", n, mean=-2.0)
            w[p + "mix.A_log"] = np.log(rng.uniform(0.1, 4.0, (n, s))).astype(np.float32)
            normal(p + "mix.D", n, std=0.4)
            lin(p + "mix.o", W, n, 1.5)
        else:
            H, D, R, V, K = (a[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
            lin(p + "mix.q", H * (D + R), W, 1.5)
            lin(p + "mix.dkv", K + R, W, 1.5)
            normal(p + "mix.dkv.norm", K, mean=1.0, std=0.3)
            lin(p + "mix.uk", H * D, K, 1.5)
            lin(p + "mix.uv", H * V, K)
            normal(p + "mix.sink", H, mean=1.0)
            lin(p + "mix.o", W, H * V)
        if f:
            sublayer(p, 2)
            lin(p + "mlp.gate", f["ff"], W, 1.5)
            lin(p + "mlp.up", f["ff"], W, 1.5)
            lin(p + "mlp.down", W, f["ff"])
    normal("final.norm", W, mean=1.0, std=0.3)
    lin("head", cfg["vocab"], W, 3.0)
    return {k: T.to_bf16(v) for k, v in w.items()}
