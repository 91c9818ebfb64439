"""Plain restatement of the layer-stack models (csrc/layer_stack.cpp): one slow
numpy function per mechanism, whole sequences, no cache.

Everything runs in `dtype` (float64 by default), so the product's rounding is
what a comparison sees.  Weights are a dict name -> array, the configuration
the parsed config.json of the model.
"""
from __future__ import annotations

import math

import numpy as np


def rms_norm(x, w, eps):
    """x / rms(x) * w over the last axis, eps inside the root."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def rope_frequencies(rot):
    """Frequency of each rotated pair and the factor on its cosine and sine.

    With `scaling` (YaRN) the frequencies between the pair that turns `fast`
    times in the original context and the one that turns `slow` times go
    linearly from unchanged to divided by `factor`."""
    dims, base = rot["dims"], rot["base"]
    i = np.arange(dims // 2, dtype=np.float64)
    f = base ** (-2.0 * i / dims)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def turns_at(t):
        return dims * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))

    lo = max(math.floor(turns_at(sc["fast"])), 0)
    hi = min(math.ceil(turns_at(sc["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [T][heads][dim]: pairs (i, i + dims/2) of the first dims dimensions turned."""
    half = rot["dims"] // 2
    f, mul = rope_frequencies(rot)
    a = positions[:, None].astype(np.float64) * f
    c, s = (np.cos(a) * mul)[:, None, :], (np.sin(a) * mul)[:, None, :]
    c, s = c.astype(x.dtype), s.astype(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    out = x.copy()
    out[..., :half] = u * c - v * s
    out[..., half:2 * half] = v * c + u * s
    return out


def sink_softmax(scores, sink):
    """softmax over the last axis whose denominator also holds exp(sink).
    scores [heads][queries][keys] with -inf where masked; sink [heads] or None."""
    m = scores.max(-1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink[:, None, None])
    e = np.exp(scores - m)
    den = e.sum(-1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink[:, None, None] - m)
    return e / den


def attention(h, w, mixer, positions):
    """Causal grouped-query attention of one whole sequence (h [T][width])."""
    T = h.shape[0]
    H, G, D, Dv = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    q = (h @ w["q"].T).reshape(T, H, D)
    k = (h @ w["k"].T).reshape(T, G, D)
    v = (h @ w["v"].T).reshape(T, G, Dv)
    if mixer.get("rot"):
        q, k = rotate(q, positions, mixer["rot"]), rotate(k, positions, mixer["rot"])
    group = np.arange(H) // (H // G)
    out = np.empty((T, H, Dv), h.dtype)
    for b in range(0, T, 256):  # query blocks bound the score matrix
        s = np.einsum("qhd,khd->hqk", q[b:b + 256], k[:, group]) * mixer["scale"]
        s = np.where(positions[None, None, :] <= positions[None, b:b + 256, None], s, -np.inf)
        p = sink_softmax(s, w.get("sink"))
        out[b:b + 256] = np.einsum("hqk,khd->qhd", p, v[:, group])
    return out.reshape(T, H * Dv) @ w["o"].T


def clamped_glu(h, gate, up, down, limit):
    """down( g sigmoid(1.702 g) (u + 1) ), gate clamped above, up on both sides."""
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g / (1 + np.exp(-1.702 * g)) * (u + 1)) @ down.T


def route(h, router_w, correction, top, scale):
    """(chosen experts [T][top], their weights [T][top])."""
    s = 1 / (1 + np.exp(-(h @ router_w.T)))
    ids = np.argsort(-(s + correction), axis=-1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, -1) * scale


def moe(h, w, mlp):
    r = mlp["router"]
    ids, wt = route(h, w["router"], w["correction"], r["top"], r["scale"])
    out = np.zeros_like(h)
    for e in range(r["experts"]):
        tok, slot = np.nonzero(ids == e)
        if tok.size:
            y = clamped_glu(h[tok], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"],
                            mlp["expert"]["limit"])
            out[tok] += wt[tok, slot][:, None] * y
    if mlp.get("shared"):
        out += clamped_glu(h, w["shared.gate"], w["shared.up"], w["shared.down"],
                           mlp["shared"]["limit"])
    return out


def layer_runs(cfg):
    """[(layer, first layer of a repeated pass?)] in the order they run."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, False) for i in range(a)]
    for p in range(loop["times"]):
        runs += [(i, p > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(cfg, weights, tokens, dtype=np.float64, taps=None):
    """Logits [T][vocab] of one sequence from position 0.  taps: a list that
    receives the residual after every layer run."""
    cache = {}

    def get(name):
        if name not in cache:
            cache[name] = np.asarray(weights[name]).astype(dtype)
        return cache[name]

    def sub(prefix):
        return {n[len(prefix):]: get(n) for n in weights if n.startswith(prefix)}

    eps = cfg["norm"]["eps"]
    tokens = np.asarray(tokens)
    positions = np.arange(len(tokens))
    emb = get("embed")[tokens]
    x = emb
    for i, again in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + emb
        y = attention(rms_norm(x, get(p + "norm1"), eps), sub(p + "mix."), L["mixer"], positions)
        x = x + rms_norm(y, get(p + "norm1b"), eps)
        if L.get("mlp"):
            y = moe(rms_norm(x, get(p + "norm2"), eps), sub(p + "mlp."), L["mlp"])
            x = x + rms_norm(y, get(p + "norm2b"), eps)
        if taps is not None:
            taps.append(x)
    return rms_norm(x, get("final.norm"), eps) @ get("head").T
