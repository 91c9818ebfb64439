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


def rotate_pairs(x, positions, rot):
    """x [T][heads][dim]: pairs (2i, 2i + 1) of the first dims dimensions turned."""
    f, mul = rope_frequencies(rot)
    a = positions[:, None].astype(np.float64) * f
    c, s = (np.cos(a) * mul)[:, None, :], (np.sin(a) * mul)[:, None, :]
    c, s = c.astype(x.dtype), s.astype(x.dtype)
    n = rot["dims"]
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out = x.copy()
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


def latent_attention(h, w, mixer, positions, eps):
    """Causal attention whose keys and values are products of one normed latent
    per token; a rotated key part is shared by the heads."""
    T = h.shape[0]
    H, D, Dr, Dv, R = (mixer[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    rot = dict(mixer["rot"], dims=Dr)
    q = (h @ w["q"].T).reshape(T, H, D + Dr)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :R], w["dkv.norm"], eps)
    k_rot = rotate_pairs(down[:, None, R:], positions, rot)[:, 0]
    q_rot = rotate_pairs(q[..., D:], positions, rot)
    k = (c @ w["uk"].T).reshape(T, H, D)
    v = (c @ w["uv"].T).reshape(T, H, Dv)
    out = np.empty((T, H, Dv), h.dtype)
    for b in range(0, T, 256):
        s = np.matmul(q[b:b + 256, :, :D].transpose(1, 0, 2), k.transpose(1, 2, 0))
        s = (s + np.matmul(q_rot[b:b + 256].transpose(1, 0, 2), k_rot.T)) * mixer["scale"]
        s = np.where(positions[None, None, :] <= positions[None, b:b + 256, None], s, -np.inf)
        out[b:b + 256] = np.matmul(sink_softmax(s, w.get("sink")),
                                   v.transpose(1, 0, 2)).transpose(1, 0, 2)
    return out.reshape(T, H * Dv) @ w["o"].T


def silu(x):
    return x / (1 + np.exp(-x))


def causal_conv(x, taps, bias):
    """x [T][channels], taps [channels][n]: the last tap meets the current token,
    zeros stand before the first."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, x.shape[1]), x.dtype), x])
    return sum(padded[k:k + len(x)] * taps[:, k] for k in range(n)) + bias


def selective_scan(x, dt, A, B, C, D):
    """S <- exp(dt A) S + dt x B, y = S C + D x, token by token from S = 0.
    x, dt [T][channels], A [channels][state], B, C [T][state], D [channels]."""
    S = np.zeros(A.shape, x.dtype)
    y = np.empty_like(x)
    for t in range(len(x)):
        S = np.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba1(h, w, mixer):
    inner, rank, state = mixer["inner"], mixer["dt_rank"], mixer["state"]
    xz = h @ w["in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, w["conv"], w["conv.b"]))
    low = x @ w["x"].T
    dt = np.logaddexp(0, low[:, :rank] @ w["dt"].T + w["dt.b"])
    y = selective_scan(x, dt, -np.exp(w["A_log"]), low[:, rank:rank + state],
                       low[:, rank + state:], w["D"])
    return (y * silu(z)) @ w["o"].T


def mix_streams(x, y, hc_mix, hc_out):
    """x [streams][T][width] -> sum over s of mix[s, t] x_s + out[t] y."""
    return np.tensordot(hc_mix.T, x, 1) + hc_out[:, None, None] * y


def softcap(x, cap):
    return cap * np.tanh(x / cap)


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


def forward_streams(cfg, weights, tokens, dtype=np.float64, taps=None):
    """Logits [T][vocab] of a model with several residual streams (Nubosun)."""
    cache = {}

    def get(name):
        if name not in cache:
            cache[name] = np.asarray(weights[name]).astype(dtype)
        return cache[name]

    def sub(prefix):
        return {n[len(prefix):]: get(n) for n in weights if n.startswith(prefix)}

    eps = cfg["norm"]["eps"]
    positions = np.arange(len(tokens))
    emb = get("embed")[np.asarray(tokens)] * dtype(cfg["embedding"]["scale"])
    x = np.repeat(emb[None], cfg["streams"], 0)

    def sublayer(x, p, q, f):
        u = np.tensordot(get(f"{p}hc{q}.in"), x, 1)
        y = f(rms_norm(u, get(f"{p}norm{q}"), eps)) * get(f"{p}ls{q}")
        return mix_streams(x, y, get(f"{p}hc{q}.mix"), get(f"{p}hc{q}.out"))

    for i, _ in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        w = sub(p + "mix.")
        if L["type"] == "mamba1":
            x = sublayer(x, p, 1, lambda h: mamba1(h, w, L["mixer"]))
        else:
            x = sublayer(x, p, 1, lambda h: latent_attention(h, w, L["mixer"], positions, eps))
        if L.get("mlp"):
            m = sub(p + "mlp.")
            x = sublayer(x, p, 2, lambda h: clamped_glu(h, m["gate"], m["up"], m["down"],
                                                        L["mlp"]["limit"]))
        if taps is not None:
            taps.append(x.sum(0))
    z = rms_norm(x.sum(0), get("final.norm"), eps) @ get("head").T
    return softcap(z, cfg["logit_softcap"]) if cfg.get("logit_softcap") else z
