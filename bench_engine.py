"""Prefill and decode throughput of a layer-stack model beside the closest other
model at equal width, heads, depth, vocabulary and context:
`bench.py --engine [small|large|all] [--engine-model gefarax|nubosun]`.

Gefarax stands beside the dense FP16 CUDADecoder, Nubosun (half its layers latent
attention with a feed-forward, half selective scans) beside Gefarax.  Random
weights and tokens.  The layer-stack models are driven through the serving
engine's own step (host metadata, cache bookkeeping, logits and all), the dense
model through its own prefill and step graph.
"""
from __future__ import annotations

import json
import struct
import sys
import tempfile
import time
from pathlib import Path

import numpy as np

HBM_PEAK = 8.0e12

SIZES = {
    "small": dict(width=1024, heads=16, kv_heads=2, dim=64, layers=4, vocab=32768, experts=32,
                  top=4, ff=512, shared=1024, prompt=2048, decode=[(16, 2048), (64, 2048)]),
    "large": dict(width=2048, heads=16, kv_heads=2, dim=128, layers=4, vocab=32768, experts=32,
                  top=4, ff=1024, shared=2048, prompt=2048, decode=[(16, 4096), (64, 4096)]),
}

# what Nubosun needs besides: the feed-forward is as wide as the experts a Gefarax
# token passes
NUBOSUN = {
    "small": dict(dim=64, rot=32, vdim=64, rank=256, ff=3072, inner=2048, state=16, dt_rank=64),
    "large": dict(dim=128, rot=64, vdim=128, rank=512, ff=6144, inner=4096, state=16, dt_rank=128),
}


def gefarax_config(s):
    layer = {"type": "attention",
             "mixer": {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"],
                       "vdim": s["dim"], "scale": s["dim"] ** -0.5,
                       "rot": {"base": 1e5, "dims": s["dim"] // 2,
                               "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0,
                                           "slow": 1.0}}},
             "mlp": {"kind": "moe", "expert": {"ff": s["ff"], "limit": 7.0},
                     "router": {"experts": s["experts"], "top": s["top"], "scale": 1.0},
                     "shared": {"ff": s["shared"], "limit": 7.0}}}
    return {"architecture": "Gefarax", "vocab": s["vocab"], "width": s["width"],
            "norm": {"eps": 1e-5}, "layers": [layer] * s["layers"]}


def nubosun_config(s, n):
    rot = {"base": 1e5, "dims": n["rot"],
           "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
    latent = {"type": "latent_attention",
              "mixer": {"heads": s["heads"], "dim": n["dim"], "rot_dim": n["rot"],
                        "vdim": n["vdim"], "kv_rank": n["rank"],
                        "scale": (n["dim"] + n["rot"]) ** -0.5, "rot": rot},
              "mlp": {"kind": "dense", "ff": n["ff"], "limit": 7.0}}
    scan = {"type": "mamba1", "mlp": None,
            "mixer": {"inner": n["inner"], "state": n["state"], "dt_rank": n["dt_rank"], "conv": 4}}
    order = [latent, scan, scan, latent]
    return {"architecture": "Nubosun", "vocab": s["vocab"], "width": s["width"],
            "norm": {"eps": 1e-5}, "embedding": {"scale": 12.0}, "streams": 4,
            "logit_softcap": 30.0, "layers": [order[i % 4] for i in range(s["layers"])]}


def random_bf16(rng, shape, scale):
    """Random signs and mantissas around `scale` (bf16 bits)."""
    n = int(np.prod(shape))
    e = int(np.floor(np.log2(scale))) + 127
    bits = rng.integers(0, 1 << 16, n, dtype=np.uint16)
    return (bits & np.uint16(0x807F)) | np.uint16(e << 7)


def gefarax_tensors(cfg):
    """(name, shape, all ones?) of every weight."""
    W, names = cfg["width"], []

    def t(name, *shape, one=False):
        names.append((name, shape, one))
    t("embed", cfg["vocab"], W)
    for i, L in enumerate(cfg["layers"]):
        a, f, p = L["mixer"], L["mlp"], f"l{i}."
        for n in ("norm1", "norm1b", "norm2", "norm2b"):
            t(p + n, W, one=True)
        t(p + "mix.q", a["heads"] * a["dim"], W)
        t(p + "mix.k", a["kv_heads"] * a["dim"], W)
        t(p + "mix.v", a["kv_heads"] * a["vdim"], W)
        t(p + "mix.o", W, a["heads"] * a["vdim"])
        t(p + "mix.sink", a["heads"])
        t(p + "mlp.router", f["router"]["experts"], W)
        t(p + "mlp.correction", f["router"]["experts"])
        for e in [f"e{k}" for k in range(f["router"]["experts"])] + ["shared"]:
            ff = f["shared"]["ff"] if e == "shared" else f["expert"]["ff"]
            t(f"{p}mlp.{e}.gate", ff, W)
            t(f"{p}mlp.{e}.up", ff, W)
            t(f"{p}mlp.{e}.down", W, ff)
    t("final.norm", W, one=True)
    t("head", cfg["vocab"], W)
    return names


def nubosun_tensors(cfg):
    W, S, names = cfg["width"], cfg["streams"], []

    def t(name, *shape, one=False):
        names.append((name, shape, one))
    t("embed", cfg["vocab"], W)
    for i, L in enumerate(cfg["layers"]):
        a, f, p = L["mixer"], L["mlp"], f"l{i}."
        for q in (1, 2) if f else (1,):
            for n in (f"norm{q}", f"ls{q}"):
                t(p + n, W, one=True)
            t(f"{p}hc{q}.in", S)
            t(f"{p}hc{q}.out", S)
            t(f"{p}hc{q}.mix", S, S)
        if L["type"] == "mamba1":
            n, state, rank = a["inner"], a["state"], a["dt_rank"]
            t(p + "mix.in", 2 * n, W)
            t(p + "mix.conv", n, a["conv"])
            t(p + "mix.conv.b", n)
            t(p + "mix.x", rank + 2 * state, n)
            t(p + "mix.dt", n, rank)
            t(p + "mix.dt.b", n)
            t(p + "mix.A_log", n, state)
            t(p + "mix.D", n, one=True)
            t(p + "mix.o", W, n)
        else:
            H, D, R, V, K = (a[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
            t(p + "mix.q", H * (D + R), W)
            t(p + "mix.dkv", K + R, W)
            t(p + "mix.dkv.norm", K, one=True)
            t(p + "mix.uk", H * D, K)
            t(p + "mix.uv", H * V, K)
            t(p + "mix.sink", H)
            t(p + "mix.o", W, H * V)
        if f:
            t(p + "mlp.gate", f["ff"], W)
            t(p + "mlp.up", f["ff"], W)
            t(p + "mlp.down", W, f["ff"])
    t("final.norm", W, one=True)
    t("head", cfg["vocab"], W)
    return names


def write_model(folder, cfg, seed):
    """config.json and random weights, streamed to model.safetensors."""
    (folder / "config.json").write_text(json.dumps(cfg))
    names = (nubosun_tensors if cfg["architecture"] == "Nubosun" else gefarax_tensors)(cfg)
    head, at = {}, 0
    for name, shape, _ in names:
        n = 2 * int(np.prod(shape))
        head[name] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [at, at + n]}
        at += n
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    rng = np.random.default_rng(seed)
    with open(folder / "model.safetensors", "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h)
        for name, shape, one in names:
            x = np.full(shape, 0x3F80, np.uint16) if one else \
                random_bf16(rng, shape, 1.0 if name == "embed" else shape[-1] ** -0.5)
            x.tofile(f)


def log(*a):
    print(*a, file=sys.stderr, flush=True)


def timed(fn, n, sync=lambda: None):
    sync()
    t0 = time.perf_counter()
    for _ in range(n):
        fn()
    sync()
    return (time.perf_counter() - t0) / n


def bench_stack(cfg, s, steps, seed=0):
    """Through the scheduler: a prompt that generates one token (prefill), then
    batches of requests once all of them decode."""
    from engine import Engine
    name = cfg["architecture"]
    rng = np.random.default_rng(seed)
    B = max(b for b, _ in s["decode"])
    T = max(t for _, t in s["decode"])
    res = {"model": name, "dtype": "bf16"}
    new = 4 * steps + 2 * B * (T // 2048 + 2)  # decode tokens while the last prompts fill
    with tempfile.TemporaryDirectory() as d:
        t0 = time.time()
        write_model(Path(d), cfg, seed)
        per_seq = -(-(T + new) // 64) * 64
        eng = Engine(d, max_seqs=B, max_tokens=B * per_seq, max_seq_len=per_seq)
        log(f"{name}: setup {time.time() - t0:.1f}s")
    prompt = rng.integers(0, s["vocab"], s["prompt"])

    def one_prefill():
        eng.generate_batch([prompt], 1)
    one_prefill()
    one_prefill()
    t = timed(one_prefill, 5)
    res["prefill"] = {"prompt": s["prompt"], "ms": round(t * 1e3, 3),
                      "tokens_per_s": round(s["prompt"] / t, 1)}
    res["decode"] = []
    for b, ctx in s["decode"]:
        ids = [eng.submit(rng.integers(0, s["vocab"], ctx), new) for _ in range(b)]
        while any(not eng.result(i)[0] for i in ids):
            eng.run()
        for _ in range(8):
            eng.run()
        t = timed(eng.run, steps)
        res["decode"].append({"batch": b, "context": ctx, "ms_per_step": round(t * 1e3, 4),
                              "tokens_per_s": round(b / t, 1)})
        while eng.run():
            pass
        for i in ids:
            eng.result(i)
        log(f"{name} decode {b} x {ctx}: {t * 1e3:.3f} ms")
    eng.close()
    return res


def bench_dense(s, steps, seed=0):
    import llm_decoder
    import torch
    L, H, D, V = s["layers"], s["heads"], s["dim"], s["vocab"]
    hid, inter = H * D, 4 * H * D
    rng = np.random.default_rng(seed)
    B = max(b for b, _ in s["decode"])
    T = max(t for _, t in s["decode"]) + 4 * steps + 64
    dec = llm_decoder.CUDADecoder(L, H, D, hid, V, T, max_batch=B, attn_scale=D ** -0.5)
    w = {"emb": rng.standard_normal((V, hid), dtype=np.float32).astype(np.float16).view(np.uint16)}
    for n in ("ln1", "ln2"):
        w[n + "_g"], w[n + "_b"] = np.ones((L, hid), np.float32), np.zeros((L, hid), np.float32)
    w["b1"], w["b2"] = np.zeros((L, inter), np.float32), np.zeros((L, hid), np.float32)
    for k, (K, N) in {"wqkv": (hid, 3 * hid), "wo": (hid, hid), "w1": (hid, inter),
                      "w2": (inter, hid)}.items():
        w[k] = (rng.standard_normal((L, K, N), dtype=np.float32) * K ** -0.5).astype(
            np.float16).view(np.uint16)
    dec.set_weights(w)
    res = {"model": "CUDADecoder", "dtype": "fp16"}
    prompt = rng.integers(0, V, s["prompt"]).tolist()
    ts = []
    for _ in range(4):
        dec.begin_synthetic(1, 0, 0, False)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        dec.prefill(0, prompt)
        ts.append(time.perf_counter() - t0)
    t = min(ts[1:])
    res["prefill"] = {"prompt": s["prompt"], "ms": round(t * 1e3, 3),
                      "tokens_per_s": round(s["prompt"] / t, 1)}
    res["decode"] = []
    for b, ctx in s["decode"]:
        dec.begin_synthetic(b, ctx, 0, True)
        for _ in range(4):
            dec.step(None, 0, 0, False)
        t = timed(lambda: dec.step(None, 0, 0, True), steps, dec.sync)
        res["decode"].append({"batch": b, "context": ctx, "ms_per_step": round(t * 1e3, 4),
                              "tokens_per_s": round(b / t, 1)})
        log(f"dense decode {b} x {ctx}: {t * 1e3:.3f} ms")
    return res


def decode_bytes(s, b, ctx, model):
    """Bytes a decode step must move: weights once, K and V (or latent rows, or
    state) of every row."""
    L, W, H, D, V = s["layers"], s["width"], s["heads"], s["dim"], s["vocab"]
    if model == "CUDADecoder":
        return 2 * (L * (12 * W * W + b * ctx * 2 * H * D) + V * W)
    if model == "Nubosun":
        n = s["nubosun"]
        row = n["rank"] + n["rot"]
        latent = (W * (H * (n["dim"] + n["rot"]) + row) + n["rank"] * H * (n["dim"] + n["vdim"]) +
                  W * H * n["vdim"] + 3 * W * n["ff"] + b * ctx * row)
        scan = (3 * W * n["inner"] + n["inner"] * (2 * n["dt_rank"] + 2 * n["state"]) +
                b * 2 * 2 * n["inner"] * n["state"])  # fp32 state read and written
        return 2 * (L // 2 * (latent + scan) + V * W)
    G, E, k = s["kv_heads"], s["experts"], s["top"]
    hit = E * (1 - (1 - k / E) ** b)  # experts a batch is expected to touch
    per = W * (H + 2 * G) * D + W * H * D + 3 * W * (hit * s["ff"] + s["shared"]) + E * W
    return 2 * (L * (per + b * ctx * 2 * G * D) + V * W)


def run(which, steps, model="gefarax"):
    """The JSON object of `bench.py --engine`."""
    beside = {"gefarax": "the dense decoder", "nubosun": "Gefarax"}[model]
    out = {"metric": "prefill and decode tokens/s, layer-stack model beside " + beside,
           "data": "synthetic (random weights and tokens)", "sizes": {}}
    for name in (sorted(SIZES) if which == "all" else [which]):
        s = dict(SIZES[name], nubosun=NUBOSUN[name])
        gefarax = bench_stack(gefarax_config(s), s, steps)
        if model == "nubosun":
            rows = {"nubosun": bench_stack(nubosun_config(s, NUBOSUN[name]), s, steps),
                    "gefarax": gefarax}
        else:
            rows = {"gefarax": gefarax, "dense": bench_dense(s, steps)}
        for r in rows.values():
            for x in r["decode"]:
                by = decode_bytes(s, x["batch"], x["context"], r["model"])
                x["step_bytes"] = int(by)
                x["hbm_frac"] = round(by / (x["ms_per_step"] * 1e-3) / HBM_PEAK, 4)
        drop = ("decode", "prompt") + (() if model == "nubosun" else ("nubosun",))
        out["sizes"][name] = {"shape": {k: v for k, v in s.items() if k not in drop}, **rows}
    return out
