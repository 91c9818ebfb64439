"""Small random layer-stack models for the tests: a configuration, weights, and
the folder (config.json + model.safetensors) the product loads."""
from __future__ import annotations

import json
import struct

import numpy as np

from oracle import layer_stack as ls

YARN = {"factor": 3.0, "original": 64, "fast": 8.0, "slow": 0.5}


def attn(heads=4, kv_heads=2, dim=32, vdim=32, rot=16, base=1000.0, scaling=YARN, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "scale": scale or dim ** -0.5}
    if rot:
        m["rot"] = {"base": base, "dims": rot}
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    return m


def moe(experts=8, top=2, ff=40, limit=1.5, scale=1.7, shared=48, shared_limit=0.9):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
         "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        m["shared"] = {"ff": shared, "limit": shared_limit}
    return m


def config(layers, *, width=96, vocab=150, loop=None, eps=1e-5):
    c = {"architecture": "Gefarax", "vocab": vocab, "width": width, "norm": {"eps": eps},
         "layers": [{"type": "attention", "mixer": a, "mlp": m} for a, m in layers]}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


def to_bf16(x):
    """fp32 values rounded to bf16 (kept as fp32)."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
    return u.view(np.float32)


def weights(cfg, seed, gain=1.0):
    """Random weights, all bf16 values: unit-variance products, norm weights and
    sinks away from 1 and 0."""
    rng = np.random.default_rng(seed)
    W, w = cfg["width"], {}

    def lin(name, n, k, g=1.0):
        w[name] = rng.standard_normal((n, k), dtype=np.float32) * (g * gain / np.sqrt(k))

    def norm(name):
        w[name] = (1.0 + 0.3 * rng.standard_normal(W)).astype(np.float32)

    w["embed"] = rng.standard_normal((cfg["vocab"], W), dtype=np.float32)
    for i, L in enumerate(cfg["layers"]):
        p, a, f = f"l{i}.", L["mixer"], L.get("mlp")
        norm(p + "norm1")
        norm(p + "norm1b")
        lin(p + "mix.q", a["heads"] * a["dim"], W, 1.5)
        lin(p + "mix.k", a["kv_heads"] * a["dim"], W, 1.5)
        lin(p + "mix.v", a["kv_heads"] * a["vdim"], W)
        lin(p + "mix.o", W, a["heads"] * a["vdim"])
        w[p + "mix.sink"] = rng.standard_normal(a["heads"]).astype(np.float32) + 1.0
        if not f:
            continue
        norm(p + "norm2")
        norm(p + "norm2b")
        r = f["router"]
        lin(p + "mlp.router", r["experts"], W)
        w[p + "mlp.correction"] = (0.2 * rng.standard_normal(r["experts"])).astype(np.float32)
        for e in [f"e{k}" for k in range(r["experts"])] + (["shared"] if f.get("shared") else []):
            ff = f["shared"]["ff"] if e == "shared" else f["expert"]["ff"]
            lin(f"{p}mlp.{e}.gate", ff, W, 1.5)
            lin(f"{p}mlp.{e}.up", ff, W, 1.5)
            lin(f"{p}mlp.{e}.down", W, ff)
    norm("final.norm")
    lin("head", cfg["vocab"], W)
    return {k: to_bf16(v) for k, v in w.items()}


def save(folder, cfg, w):
    """config.json and model.safetensors (bf16)."""
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    head, at, data = {}, 0, []
    for k, v in w.items():
        b = (np.ascontiguousarray(v, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[k] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [at, at + len(b)]}
        at += len(b)
        data.append(b)
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    (folder / "model.safetensors").write_bytes(struct.pack("<Q", len(h)) + h + b"".join(data))
    return folder


def row_error(got, want):
    """Per-row rms difference (the mean taken off) over the rms of the logits."""
    d = got.astype(np.float64) - want
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((want * want).mean())


FP32_TOL = 2e-5    # fp32 rounding through a few layers, relative to the logits' rms
BF16_TOL = 0.06    # bf16 products and activations


def clear_choices(w, seed=0):
    """Corrections so far apart that rounding never changes an expert choice
    (bf16 runs of whole models; the fp32 runs keep the open router)."""
    rng = np.random.default_rng(seed)
    for k in w:
        if k.endswith("mlp.correction"):
            w[k] = to_bf16(1.25 * rng.permutation(len(w[k])))
    return w


def check_rows(got, want, dtype, close_calls=False):
    """Every row.  close_calls: in bf16 a row whose experts are a close call may
    choose others, so up to one row in ten is left out."""
    e = row_error(got, want)
    tol = FP32_TOL if dtype == "float32" else BF16_TOL
    worst = e.max()
    if close_calls and dtype != "float32":
        worst = np.sort(e)[max(0, int(0.9 * len(e)) - 1)]
    assert worst < tol, f"row {e.argmax()} of {len(e)}: {e.max():.2e}, checked {worst:.2e}"


def logits(cfg, w, tokens):
    f = ls.forward_streams if cfg["architecture"] == "Nubosun" else ls.forward
    return f(cfg, w, tokens)


def replay(eng, requests, schedule):
    """Run steps [[(request, n tokens), ...], ...]; every position's logits per
    request.  A request ends (its pages and slot go back) with its last token."""
    got = {i: [] for i in requests}
    seq, at = {}, {i: 0 for i in requests}
    for step in schedule:
        entries = []
        for i, n in step:
            if i not in seq:
                seq[i] = eng.open_seq()
            t = requests[i][at[i]:at[i] + n]
            entries.append((seq[i], t, range(len(t))))
        out = eng.step(entries)
        row = 0
        for i, n in step:
            m = len(requests[i][at[i]:at[i] + n])
            got[i].append(out[row:row + m])
            row += m
            at[i] += m
            if at[i] == len(requests[i]):
                eng.close_seq(seq.pop(i))
    for s in seq.values():
        eng.close_seq(s)
    return {i: np.concatenate(v) for i, v in got.items() if v}


def random_schedule(requests, live, seed):
    """Mixed steps: some requests decode, others bring portions, some pause."""
    rng = np.random.default_rng(seed)
    waiting, left, running, steps = list(requests), {i: len(t) for i, t in requests.items()}, [], []
    while waiting or running:
        while waiting and len(running) < live:
            running.append(waiting.pop(0))
        step = []
        for i in rng.permutation(running).tolist():
            if rng.random() < 0.15 and len(running) > 1:
                continue
            n = int(rng.choice([1, 1, 1, 2, 3, 5, 16, 40, 64, 90]))
            step.append((i, min(n, left[i])))
        for i, n in step:
            left[i] -= n
            if left[i] == 0:
                running.remove(i)
        if step:
            steps.append(step)
    return steps


def most_pages(requests, steps, page=64):
    """The most pages the schedule's live requests hold at once."""
    at, most = {}, 0
    for step in steps:
        for i, n in step:
            at[i] = at.get(i, 0) + n
        most = max(most, sum(-(-n // page) for n in at.values()))
        for i, _ in step:
            if at[i] == len(requests[i]):
                del at[i]
    return most


def greedy(cfg, w, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(logits(cfg, w, np.array(t))[-1].argmax()))
    return t[len(prompt):]


def portions(total, sizes):
    """Cut `total` tokens by the cycled sizes."""
    out, k = [], 0
    while total > 0:
        n = min(sizes[k % len(sizes)], total)
        out.append(n)
        total -= n
        k += 1
    return out
