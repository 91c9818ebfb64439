"""CPU checks of the Nubosun mechanisms: the restatement (oracle/layer_stack.py)
against independent forms, and configurations the product refuses."""
import json
import math

import numpy as np
import pytest

import _layer_stack as T
import _nubosun as N
from oracle import layer_stack as ls
from test_layer_stack import create, lib  # noqa: F401  (fixture)


def test_pair_rotation_is_the_half_rotation_reordered():
    rng = np.random.default_rng(0)
    x = rng.standard_normal((5, 2, 14))
    rot = {"dims": 10, "base": 50.0, "scaling": N.YARN}
    order = [0, 2, 4, 6, 8, 1, 3, 5, 7, 9, 10, 11, 12, 13]
    pos = np.array([0, 1, 7, 63, 200])
    assert np.allclose(ls.rotate_pairs(x, pos, rot)[..., order], ls.rotate(x[..., order], pos, rot))
    p = ls.rotate_pairs(x, pos, {"dims": 10, "base": 50.0})
    angle = 7 * 50.0 ** (-2 / 10)  # position 7, pair 1
    u, v = x[2, 0, 2:4]
    assert np.allclose(p[2, 0, 2:4], [u * math.cos(angle) - v * math.sin(angle),
                                      v * math.cos(angle) + u * math.sin(angle)])


def test_latent_attention_is_grouped_attention_over_written_out_keys():
    """With keys and values written out per head, the layer is attention with a
    key/value head per head; queries taken into the latent space give the same
    scores."""
    m = N.latent(heads=3, dim=6, rot=4, vdim=5, rank=9)
    cfg = N.config([(m, None)], width=20)
    w = {k[7:]: v.astype(np.float64) for k, v in N.weights(cfg, 1).items() if k.startswith("l0.mix.")}
    h = np.random.default_rng(2).standard_normal((11, 20))
    pos = np.arange(11)
    got = ls.latent_attention(h, w, m, pos, 1e-5)
    c = ls.rms_norm(h @ w["dkv"][:9].T, w["dkv.norm"], 1e-5)
    kr = ls.rotate_pairs((h @ w["dkv"][9:].T)[:, None], pos, m["rot"])[:, 0]
    out = np.zeros((11, 3, 5))
    for head in range(3):
        q = h @ w["q"][10 * head:10 * head + 10].T
        qr = ls.rotate_pairs(q[:, None, 6:], pos, m["rot"])[:, 0]
        in_latent = q[:, :6] @ w["uk"][6 * head:6 * head + 6]
        for i in range(11):
            s = (c[:i + 1] @ in_latent[i] + kr[:i + 1] @ qr[i]) * m["scale"]
            e = np.exp(s)
            p = e / (e.sum() + math.exp(w["sink"][head]))
            out[i, head] = w["uv"][5 * head:5 * head + 5] @ (p @ c[:i + 1])
    assert np.allclose(got, out.reshape(11, 15) @ w["o"].T)


def test_causal_conv_by_hand():
    x = np.array([[1.0], [2.0], [4.0], [8.0]])
    got = ls.causal_conv(x, np.array([[0.5, 10.0, 100.0]]), np.array([0.25]))
    assert got[:, 0].tolist() == [100.25, 210.25, 420.75, 841.25]


def test_selective_scan_is_a_sum_over_the_past():
    rng = np.random.default_rng(3)
    T_, C, S = 9, 4, 3
    x, dt = rng.standard_normal((T_, C)), rng.uniform(0.1, 1, (T_, C))
    A, B, Cm, D = -rng.uniform(0.1, 2, (C, S)), *rng.standard_normal((2, T_, S)), rng.standard_normal(C)
    y = ls.selective_scan(x, dt, A, B, Cm, D)
    for t in range(T_):
        want = D * x[t]
        for j in range(t + 1):
            decay = np.exp(dt[j + 1:t + 1].sum(0)[:, None] * A)
            want = want + (decay * (dt[j] * x[j])[:, None] * B[j] * Cm[t]).sum(1)
        assert np.allclose(y[t], want)


def test_streams_mix_from_first_index_to_second():
    x = np.array([[[1.0]], [[10.0]]])
    got = ls.mix_streams(x, np.array([[100.0]]), np.array([[1.0, 2.0], [3.0, 5.0]]), np.array([7.0, 0.5]))
    assert got[:, 0, 0].tolist() == [1 + 30 + 700, 2 + 50 + 50]


def test_one_token_through_one_layer_by_hand():
    cfg = N.config([(N.mamba(inner=4, state=2, dt_rank=1, conv=2), N.dense(ff=3, limit=0.4))],
                   width=8, vocab=7, streams=2, scale=2.5, cap=3.0)
    w = {k: v.astype(np.float64) for k, v in N.weights(cfg, 4).items()}
    x = [2.5 * w["embed"][5]] * 2

    def rms(v, g):
        return v / math.sqrt((v * v).mean() + 1e-5) * g

    def around(q, f):
        hc = {n: w[f"l0.hc{q}.{n}"] for n in ("in", "out", "mix")}
        y = f(rms(hc["in"][0] * x[0] + hc["in"][1] * x[1], w[f"l0.norm{q}"])) * w[f"l0.ls{q}"]
        return [hc["mix"][0, t] * x[0] + hc["mix"][1, t] * x[1] + hc["out"][t] * y for t in range(2)]

    def mixer(h):
        xz = w["l0.mix.in"] @ h
        c = xz[:4] * w["l0.mix.conv"][:, 1] + w["l0.mix.conv.b"]
        c = c / (1 + np.exp(-c))
        low = w["l0.mix.x"] @ c
        dt = np.log1p(np.exp(w["l0.mix.dt"] @ low[:1] + w["l0.mix.dt.b"]))
        y = dt * c * (low[1:3] @ low[3:5]) + w["l0.mix.D"] * c
        return w["l0.mix.o"] @ (y * xz[4:] / (1 + np.exp(-xz[4:])))

    def ffn(h):
        g, u = np.minimum(w["l0.mlp.gate"] @ h, 0.4), np.clip(w["l0.mlp.up"] @ h, -0.4, 0.4)
        return w["l0.mlp.down"] @ (g / (1 + np.exp(-1.702 * g)) * (u + 1))

    x = around(1, mixer)
    x = around(2, ffn)
    z = w["head"] @ rms(x[0] + x[1], w["final.norm"])
    assert np.allclose(ls.forward_streams(cfg, w, [5])[0], 3 * np.tanh(z / 3))


def test_a_position_does_not_see_later_tokens():
    cfg = N.config([(N.latent(), N.dense()), (N.mamba(), None)], loop=(0, 2, 2))
    w = N.weights(cfg, 5)
    t = np.arange(20) % cfg["vocab"]
    u = t.copy()
    u[12:] = 7
    a, b = T.logits(cfg, w, t), T.logits(cfg, w, u)
    assert np.allclose(a[:12], b[:12]) and not np.allclose(a[12:], b[12:])


def test_repeated_passes_run_the_same_weights_again():
    one = N.config([(N.latent(), N.dense()), (N.mamba(), None)], loop=(0, 2, 2))
    w = N.weights(one, 6)
    two = N.config([(N.latent(), N.dense()), (N.mamba(), None)] * 2)
    w2 = dict(w, **{k.replace(a, b): w[k] for a, b in (("l0.", "l2."), ("l1.", "l3."))
                    for k in w if k.startswith(a)})
    t = [3, 1, 4, 1, 5]
    assert np.allclose(T.logits(one, w, t), T.logits(two, w2, t))


def test_config_faults_are_named(lib, tmp_path):  # noqa: F811
    def bad(change, status=1):
        c = N.config([(N.latent(), N.dense()), (N.mamba(), None)])
        change(c)
        (tmp_path / "config.json").write_text(json.dumps(c))
        rc, msg = create(lib, tmp_path)
        assert rc == status, (rc, msg)
        return msg

    L = lambda c, i=0: c["layers"][i]  # noqa: E731
    assert "width" in bad(lambda c: c.pop("width"))
    assert "embedding.scale" in bad(lambda c: c.pop("embedding"))
    assert "streams" in bad(lambda c: c.pop("streams"))
    assert "streams" in bad(lambda c: c.update(streams=0))
    assert "streams" in bad(lambda c: c.update(streams=17))
    assert "kv_rank" in bad(lambda c: L(c)["mixer"].pop("kv_rank"))
    assert "kv_rank" in bad(lambda c: L(c)["mixer"].update(kv_rank=513))
    assert "rot_dim" in bad(lambda c: L(c)["mixer"].update(rot_dim=7))
    assert "base" in bad(lambda c: L(c)["mixer"].pop("rot"))
    assert "scaling.fast" in bad(lambda c: L(c)["mixer"]["rot"]["scaling"].pop("fast"))
    assert "limit" in bad(lambda c: L(c)["mlp"].pop("limit"))
    assert "kind" in bad(lambda c: L(c)["mlp"].update(kind="moe"), 2)
    assert "type" in bad(lambda c: L(c).update(type="attention"), 2)
    assert "state" in bad(lambda c: L(c, 1)["mixer"].update(state=257))
    assert "conv" in bad(lambda c: L(c, 1)["mixer"].pop("conv"))
    assert "loop" in bad(lambda c: c.update(loop={"start": 1, "stop": 3, "times": 2}))


@pytest.mark.parametrize("cap", [None, 0.5])
def test_softcap_bounds_the_logits(cap):
    cfg = N.config([(N.mamba(), None)], cap=cap)
    z = T.logits(cfg, N.weights(cfg, 8), [1, 2, 3])
    assert (np.abs(z).max() <= 0.5) if cap else (np.abs(z).max() > 1)
