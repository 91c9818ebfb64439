"""CPU checks of the layer-stack models: the restatement's mechanisms against
independent forms, the registry, and configurations and weight files that are
refused before anything touches a device."""
import ctypes
import json
import math
import os
import struct
import subprocess
import sys

import numpy as np
import pytest

import _layer_stack as T
from conftest import ROOT
from oracle import layer_stack as ls


def test_yarn_keeps_fast_pairs_and_slows_slow_ones():
    rot = {"dims": 64, "base": 10000.0,
           "scaling": {"factor": 8.0, "original": 512, "fast": 16.0, "slow": 1.0}}
    f, mul = ls.rope_frequencies(rot)
    plain, one = ls.rope_frequencies({"dims": 64, "base": 10000.0})
    turns = 512 * plain / (2 * math.pi)
    assert one == 1.0 and mul == pytest.approx(0.1 * math.log(8.0) + 1)
    assert np.allclose(f[turns > 32], plain[turns > 32])
    assert np.allclose(f[turns < 0.5], plain[turns < 0.5] / 8)
    assert np.all(np.diff(f) < 0)


def test_rotation_depends_on_distance_only():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((2, 1, 1, 24))
    rot = {"dims": 16, "base": 100.0}
    at = lambda x, p: ls.rotate(x, np.array([p]), rot)[0, 0]  # noqa: E731
    assert at(q, 9) @ at(k, 4) == pytest.approx(at(q, 25) @ at(k, 20))
    assert np.array_equal(at(q, 9)[16:], q[0, 0, 16:])


def test_sink_is_one_more_key_without_a_value():
    rng = np.random.default_rng(1)
    s, sink = rng.standard_normal((3, 5, 7)), rng.standard_normal(3)
    with_key = np.concatenate([s, np.broadcast_to(sink[:, None, None], (3, 5, 1))], -1)
    e = np.exp(with_key)
    assert np.allclose(ls.sink_softmax(s, sink), (e / e.sum(-1, keepdims=True))[..., :-1])


def test_one_token_by_hand():
    """A single token attends to itself and the sink."""
    cfg = T.config([(T.attn(heads=2, kv_heads=1, dim=8, vdim=4, rot=4), None)], width=32, vocab=9)
    w = T.weights(cfg, 2)
    w = {k: v.astype(np.float64) for k, v in w.items()}
    x = w["embed"][5]
    h = ls.rms_norm(x, w["l0.norm1"], 1e-5)
    q, k, v = (w[f"l0.mix.{n}"] @ h for n in "qkv")
    y = []
    for head in range(2):
        score = q[8 * head:8 * head + 8] @ k * 8 ** -0.5
        # at position 0 the rotation only scales: the YaRN factor on both sides
        mul = 0.1 * math.log(T.YARN["factor"]) + 1
        rot = q[8 * head:8 * head + 4] @ k[:4] * 8 ** -0.5
        score = score - rot + rot * mul * mul
        y.append(v * math.exp(score) / (math.exp(score) + math.exp(w["l0.mix.sink"][head])))
    x = x + ls.rms_norm(w["l0.mix.o"] @ np.concatenate(y), w["l0.norm1b"], 1e-5)
    want = w["head"] @ ls.rms_norm(x, w["final.norm"], 1e-5)
    assert np.allclose(ls.forward(cfg, w, [5])[0], want)


def test_route_prefers_corrected_scores_and_weighs_plain_ones():
    z = np.array([[0.0, 2.0, -2.0, 1.0]])
    ids, wt = ls.route(z, np.eye(4), np.array([0.9, 0, 0, -0.9]), 2, 3.0)
    s = 1 / (1 + np.exp(-z[0]))
    assert ids.tolist() == [[0, 1]]
    assert np.allclose(wt, [[3 * s[0], 3 * s[1]]])


def test_clamped_glu_limits():
    one = np.ones((1, 1))
    for g, u in ((5.0, 5.0), (-5.0, -5.0), (0.3, -0.2)):
        got = ls.clamped_glu(one, one * g, one * u, one, 2.0)[0, 0]
        gc, uc = min(g, 2.0), max(min(u, 2.0), -2.0)
        assert got == pytest.approx(gc / (1 + math.exp(-1.702 * gc)) * (uc + 1))


def test_layer_runs_of_a_loop():
    cfg = T.config([(T.attn(), None)] * 4, loop=(1, 3, 2))
    assert ls.layer_runs(cfg) == [(0, False), (1, False), (2, False), (1, True), (2, False),
                                  (3, False)]


def test_a_position_does_not_see_later_tokens():
    cfg = T.config([(T.attn(), T.moe(experts=3, top=1))] * 2, loop=(0, 2, 2))
    w = T.weights(cfg, 3)
    t = np.arange(20) % cfg["vocab"]
    u = t.copy()
    u[12:] = 7
    assert np.allclose(ls.forward(cfg, w, t)[:12], ls.forward(cfg, w, u)[:12])


# ----------------------------------------------------- the product, on the host
@pytest.fixture(scope="module")
def lib():
    import llm_capi
    return llm_capi.load()


def create(lib, folder, **kw):
    import engine
    cfg = engine.EngineConfig(kw.get("dtype", 3), kw.get("max_seqs", 1), kw.get("max_tokens", 64), 0, 0)
    h = ctypes.c_void_p()
    rc = lib.llm_engine_create(os.fsencode(str(folder)), ctypes.byref(cfg), ctypes.byref(h))
    return rc, lib.llm_last_error().decode()


def test_registry_lists_every_architecture(lib):
    assert lib.llm_model_architectures().decode().split(",") == ["CUDADecoder", "Gefarax",
                                                                "INT8Decoder", "Nubosun"]


def test_config_faults_are_named(lib, tmp_path):
    rc, msg = create(lib, tmp_path / "none")
    assert rc == 5 and "config.json" in msg
    (tmp_path / "config.json").write_text("{")
    assert create(lib, tmp_path)[0] == 5
    (tmp_path / "config.json").write_text('{"architecture": "Other"}')
    rc, msg = create(lib, tmp_path)
    assert rc == 2 and "Other" in msg and "Gefarax" in msg

    def bad(change, status=1):
        c = T.config([(T.attn(), T.moe())])
        change(c)
        (tmp_path / "config.json").write_text(json.dumps(c))
        rc, msg = create(lib, tmp_path)
        assert rc == status, (rc, msg)
        return msg

    L = lambda c: c["layers"][0]  # noqa: E731
    assert "width" in bad(lambda c: c.pop("width"))
    assert "eps" in bad(lambda c: c.pop("norm"))
    assert "kv_heads" in bad(lambda c: L(c)["mixer"].update(kv_heads=3))
    assert "head sizes" in bad(lambda c: L(c)["mixer"].update(dim=258))
    assert "rot.dims" in bad(lambda c: L(c)["mixer"]["rot"].update(dims=7))
    assert "expert" in bad(lambda c: L(c)["mlp"]["router"].update(top=9))
    assert "loop" in bad(lambda c: c.update(loop={"start": 0, "stop": 2, "times": 2}))
    assert "type" in bad(lambda c: L(c).update(type="other"), 2)
    assert "kind" in bad(lambda c: L(c)["mlp"].update(kind="other"), 2)
    assert "limit" in bad(lambda c: L(c)["mlp"]["expert"].pop("limit"))
    assert "dtype" in create(lib, T.save(tmp_path / "m", T.config([(T.attn(), None)]), {}), dtype=0)[1]


def test_trace_run_refuses_bad_arguments():
    run = [sys.executable, str(ROOT / "bin" / "trace_run")]
    assert subprocess.run(run + ["--help"], capture_output=True).returncode == 0
    r = subprocess.run(run + ["--model", "x", "--dtype", "int8", "--out", ".", "--max-tokens", "1"],
                       capture_output=True, text=True)
    assert r.returncode == 2 and "dtype" in r.stderr
    assert os.access(ROOT / "bin" / "trace_run", os.X_OK)
    assert os.access(ROOT / "bin" / "generate", os.X_OK)


def test_safetensors_writer_layout(tmp_path):
    """The tests' own files are what they say (8-byte length, JSON, data)."""
    cfg = T.config([(T.attn(), None)], width=32, vocab=5)
    w = T.weights(cfg, 1)
    b = (T.save(tmp_path / "m", cfg, w) / "model.safetensors").read_bytes()
    n = struct.unpack("<Q", b[:8])[0]
    head = json.loads(b[8:8 + n])
    lo, hi = head["embed"]["data_offsets"]
    x = (np.frombuffer(b[8 + n + lo:8 + n + hi], "<u2").astype(np.uint32) << 16).view(np.float32)
    assert np.array_equal(x.reshape(5, 32), w["embed"])
