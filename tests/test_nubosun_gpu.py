"""Nubosun (latent attention, selective scan, mixed residual streams) on the
serving engine against the plain restatement (oracle/layer_stack.py): each
mechanism alone and at its size limits, every way of cutting a prompt, mixed
batches with pages and slots used again, keys that stand out, long memories,
long decoding, and generation through the scheduler."""
import json
import subprocess
import sys

import numpy as np
import pytest

import _layer_stack as T
import _nubosun as N
from conftest import ROOT
from oracle import layer_stack as ls
from test_layer_stack_gpu import DTYPES, run_whole, serve, tokens  # noqa: F401  (fixture)

pytestmark = pytest.mark.gpu


def silent(w, *layers):
    """Sublayers that put out nothing."""
    for i in layers:
        for n in (f"l{i}.ls1", f"l{i}.ls2"):
            if n in w:
                w[n] = 0 * w[n]
    return w


def check_cuts(eng, cfg, w, t, dtype, steps):
    want = T.logits(cfg, w, t)
    T.check_rows(run_whole(eng, t), want, dtype)
    T.check_rows(T.replay(eng, {0: t}, [[(0, n)] for n in steps])[0], want, dtype)


# ---------------------------------------------------------------- mechanisms
@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_norm_head_and_cap_alone(serve, dtype):  # noqa: F811
    for cap, scale in ((2.0, 0.3), (None, 5.0), (40.0, 1.0)):
        cfg = N.config([(N.mamba(), None)], width=72, eps=0.3, cap=cap, scale=scale, streams=2)
        w = silent(N.weights(cfg, 1), 0)
        t = tokens(cfg, 30, 2)
        T.check_rows(run_whole(serve(cfg, w, dtype, name=f"m{scale}"), t), T.logits(cfg, w, t), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 7, 16])
def test_streams(serve, streams, dtype):  # noqa: F811
    """Unlike mixing in every sublayer; streams that are swapped, summed early or
    mixed the other way round show."""
    cfg = N.config([(N.mamba(inner=40), N.dense(ff=24)), (N.latent(), N.dense(ff=24)),
                    (N.mamba(inner=40), None)], streams=streams)
    w = N.weights(cfg, 3)
    t = tokens(cfg, 70, 4)
    check_cuts(serve(cfg, w, dtype), cfg, w, t, dtype, [30, 1, 2] + [1] * 37)
    if streams > 1:
        turned = dict(w, **{k: v.T for k, v in w.items() if k.endswith(".mix") and v.ndim == 2
                            and v.shape == (streams, streams)})
        assert np.median(T.row_error(T.logits(cfg, turned, t), T.logits(cfg, w, t))) > 0.01


def test_residual_widths(serve):  # noqa: F811
    for width in (37, 264, 700, 1101, 2500):
        cfg = N.config([(N.mamba(inner=20), N.dense(ff=10))], width=width, vocab=41)
        w = N.weights(cfg, 5)
        t = tokens(cfg, 20, 6)
        T.check_rows(run_whole(serve(cfg, w, name=f"w{width}"), t), T.logits(cfg, w, t), "float32")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff,limit", [(56, 1.5), (33, 0.05), (1, 7.0), (200, 0.4)])
def test_feed_forward_alone(serve, ff, limit, dtype):  # noqa: F811
    cfg = N.config([(N.mamba(), N.dense(ff=ff, limit=limit))])
    w = N.weights(cfg, 7)
    w["l0.ls1"] = 0 * w["l0.ls1"]
    eng = serve(cfg, w, dtype)
    for n in (1, 19, 300):
        t = tokens(cfg, n, n)
        T.check_rows(run_whole(eng, t), T.logits(cfg, w, t), dtype)


# portions from 65 tokens on take expanded keys where the latent is much wider
# than the heads
LATENT = {
    "plain": N.latent(),
    "no_scaling": N.latent(scaling=None),
    "narrow_ramp": N.latent(rot=16, scaling=dict(factor=8.0, original=4096, fast=1.0, slow=1.0)),
    "factor_one": N.latent(scaling=dict(factor=1.0, original=64, fast=8.0, slow=0.5)),
    "not_rotated": N.latent(rot=0),
    "one_head": N.latent(heads=1),
    "twenty_heads": N.latent(heads=20, dim=8, vdim=8),
    "forty_heads": N.latent(heads=40, dim=8, vdim=4),
    "odd_sizes": N.latent(heads=3, dim=9, rot=6, vdim=7, rank=29),
    "one_dim": N.latent(dim=1, rot=2, vdim=1, rank=1),
    "scale": N.latent(scale=0.5),
    "expanded": N.latent(heads=5, dim=16, rot=8, vdim=16, rank=128),
    "expanded_odd": N.latent(heads=3, dim=15, rot=10, vdim=9, rank=101),
    "row_320": N.latent(heads=2, dim=40, rot=24, vdim=24, rank=250),
    "row_576": N.latent(heads=18, dim=32, rot=64, vdim=40, rank=512),
    "heads_past_256": N.latent(heads=2, dim=260, rot=16, vdim=270, rank=300),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(LATENT))
def test_latent_attention_alone(serve, name, dtype):  # noqa: F811
    cfg = N.config([(LATENT[name], None)])
    w = N.weights(cfg, 9)
    t = tokens(cfg, 230, 10)
    eng = serve(cfg, w, dtype)
    check_cuts(eng, cfg, w, t, dtype, [17, 66, 3, 70, 2, 1, 47] + [1] * 24)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["plain", "expanded"])
@pytest.mark.parametrize("sink", [-30.0, 0.0, 6.0, 40.0])
def test_sink(serve, name, sink, dtype):  # noqa: F811
    cfg = N.config([(LATENT[name], None)])
    w = N.weights(cfg, 11)
    w["l0.mix.sink"] = T.to_bf16(sink + np.linspace(-1, 1, len(w["l0.mix.sink"])))
    t = tokens(cfg, 140, 12)
    want = T.logits(cfg, w, t)
    check_cuts(serve(cfg, w, dtype), cfg, w, t, dtype, [100] + [1] * 40)
    if -30 < sink < 40:
        w2 = dict(w, **{"l0.mix.sink": w["l0.mix.sink"] - 100})
        assert T.row_error(T.logits(cfg, w2, t), want)[:20].max() > 0.02


MAMBA = {
    "plain": N.mamba(),
    "one_tap": N.mamba(conv=1),
    "two_taps": N.mamba(conv=2),
    "three_taps": N.mamba(conv=3),
    "seven_taps": N.mamba(conv=7),
    "one_state": N.mamba(state=1),
    "state_8": N.mamba(state=8),
    "state_16": N.mamba(state=16, inner=96),
    "state_31": N.mamba(state=31),
    "state_64": N.mamba(state=64, inner=130),
    "state_100": N.mamba(state=100),
    "state_256": N.mamba(state=256, inner=40),
    "odd_sizes": N.mamba(inner=77, state=5, dt_rank=3),
    "one_rank": N.mamba(dt_rank=1),
    "wide_rank": N.mamba(dt_rank=50),
    "one_channel": N.mamba(inner=1),
    "many_channels": N.mamba(inner=600, state=4),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MAMBA))
def test_selective_scan_alone(serve, name, dtype):  # noqa: F811
    """Prompts of several chunks, portions shorter than the convolution, single
    tokens."""
    cfg = N.config([(MAMBA[name], None)])
    w = N.weights(cfg, 13)
    t = tokens(cfg, 230, 14)
    check_cuts(serve(cfg, w, dtype), cfg, w, t, dtype, [2, 1, 2, 2, 1, 3, 66, 5, 64, 1, 1, 2, 60] + [1] * 20)


@pytest.mark.parametrize("state", [8, 128])
def test_memory_of_the_first_token(serve, state):  # noqa: F811
    """Slow decay and a strong first input: the token at position 0 decides rows
    hundreds of tokens later, over chunks, portions and decoded tokens."""
    cfg = N.config([(N.mamba(state=state, inner=64), None)], cap=None, streams=2)
    w = N.weights(cfg, 15)
    w["l0.mix.A_log"][:] = T.to_bf16(np.full(1, np.log(2e-4)))[0]
    w["l0.mix.D"][:] = 0
    w["embed"][0] *= 8
    t = tokens(cfg, 400, 16)
    t[t == 0] = 1
    t[0] = 0
    other = t.copy()
    other[0] = 2
    want = T.logits(cfg, w, t)
    assert T.row_error(T.logits(cfg, w, other), want)[350:].min() > 20 * T.FP32_TOL
    check_cuts(serve(cfg, w), cfg, w, t, "float32", [1, 130, 2, 64, 63, 65, 1, 40] + [1] * 34)


def test_fast_decay_and_large_steps(serve):  # noqa: F811
    """Decays that vanish and step sizes past the softplus' bend."""
    cfg = N.config([(N.mamba(), None)])
    w = N.weights(cfg, 17)
    w["l0.mix.A_log"] = T.to_bf16(w["l0.mix.A_log"] + 4)
    w["l0.mix.dt.b"] = T.to_bf16(np.linspace(-40, 40, len(w["l0.mix.dt.b"])))
    t = tokens(cfg, 150, 18)
    check_cuts(serve(cfg, w), cfg, w, t, "float32", [70, 3, 60] + [1] * 17)


@pytest.mark.parametrize("loop", [(0, 1, 3), (1, 3, 2), (0, 3, 2), (2, 3, 4), (1, 2, 1), (1, 1, 2)])
def test_repeated_layers(serve, loop):  # noqa: F811
    cfg = N.config([(N.latent(), None), (N.mamba(), N.dense()), (N.latent(rank=24), N.dense())],
                   loop=loop)
    w = N.weights(cfg, 19)
    t = tokens(cfg, 90, 20)
    check_cuts(serve(cfg, w), cfg, w, t, "float32", [50] + [1] * 40)


def test_residual_after_every_layer(serve):  # noqa: F811
    cfg = N.config([(N.latent(), N.dense()), (N.mamba(), None)], loop=(0, 2, 2), width=100)
    w = N.weights(cfg, 21)
    t = tokens(cfg, 25, 22)
    eng = serve(cfg, w)
    s = eng.open_seq()
    got, tap = eng.step_taps([(s, t, range(25))])
    want = []
    T.check_rows(got, ls.forward_streams(cfg, w, t, taps=want), "float32")
    assert tap.shape == (4, 25, 100) and len(want) == 4
    for a, b in zip(tap, want):
        assert np.abs(a - b).max() < 1e-4 * np.abs(b).max()


# ------------------------------------------------------------- whole models
MODELS = {
    "plain": N.config([(N.latent(), N.dense()), (N.mamba(), None), (N.mamba(), N.dense()),
                       (N.latent(), N.dense())], loop=(0, 2, 2)),
    "unlike_layers": N.config(
        [(N.mamba(inner=50, state=33, dt_rank=5, conv=2), N.dense(ff=20)),
         (N.latent(heads=5, dim=16, rot=8, vdim=16, rank=128), None),
         (N.latent(heads=18, dim=8, rot=4, vdim=6, rank=20, base=50.0, scaling=None), N.dense(ff=70)),
         (N.mamba(inner=90, state=7, conv=6), None),
         (N.latent(heads=2, dim=11, rot=2, vdim=30, rank=200), N.dense(ff=9))],
        width=84, vocab=211, streams=4, loop=(1, 4, 2)),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
@pytest.mark.parametrize("sizes", [[2], [3, 2, 7], [16], [64], [63, 65], [1], [70, 1, 66]])
def test_portions(serve, name, sizes, dtype):  # noqa: F811
    cfg = MODELS[name]
    w = N.weights(cfg, 23)
    t = tokens(cfg, 140, 24)
    eng = serve(cfg, w, dtype)
    got = T.replay(eng, {0: t}, [[(0, n)] for n in T.portions(len(t), sizes)])[0]
    T.check_rows(got, T.logits(cfg, w, t), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
@pytest.mark.parametrize("seed", [1, 2])
def test_mixed_batches_with_pages_and_slots_used_again(serve, name, dtype, seed):  # noqa: F811
    cfg = MODELS[name]
    w = N.weights(cfg, 25)
    req = {i: tokens(cfg, n, 26 + i) for i, n in
           enumerate([1, 70, 190, 5, 128, 64, 33, 150, 65, 2, 100, 129])}
    steps = T.random_schedule(req, 4, seed)
    eng = serve(cfg, w, dtype, max_tokens=64 * T.most_pages(req, steps), max_seqs=4)
    free = eng.free_tokens
    got = T.replay(eng, req, steps)
    assert eng.free_tokens == free
    for i, t in req.items():
        T.check_rows(got[i], T.logits(cfg, w, t), dtype)


def test_a_slot_starts_from_nothing(serve):  # noqa: F811
    """One slot, sequences of all lengths after one another, one cut short."""
    cfg = MODELS["plain"]
    w = N.weights(cfg, 27)
    eng = serve(cfg, w, max_seqs=1, max_tokens=192)
    for n, cut in ((150, [150]), (1, [1]), (2, [1, 1]), (3, [2, 1]), (90, [1, 89]), (5, [3, 2])):
        t = tokens(cfg, n, n)
        got = T.replay(eng, {0: t}, [[(0, k)] for k in cut])[0]
        T.check_rows(got, T.logits(cfg, w, t), "float32")
        s = eng.open_seq()  # left unfinished
        eng.step([(s, t[:n // 2 + 1], [])])
        eng.close_seq(s)


def test_batch_alone_and_step_size_give_the_same(serve):  # noqa: F811
    cfg = MODELS["unlike_layers"]
    w = N.weights(cfg, 29)
    a, b, c = (tokens(cfg, n, n) for n in (130, 77, 20))
    eng = serve(cfg, w, max_seqs=3)
    small = serve(cfg, w, max_seqs=3, max_step_tokens=24, name="small")
    alone = run_whole(eng, a)
    for e in (eng, small):
        together = T.replay(e, {0: c, 1: a, 2: b}, [[(0, 20), (1, 130), (2, 77)]])[1]
        assert T.row_error(together, alone).max() < T.FP32_TOL


def test_models_without_attention_or_without_scan(serve):  # noqa: F811
    for name, mix in (("scan", N.mamba()), ("attention", N.latent())):
        cfg = N.config([(mix, N.dense()), (mix, None)])
        w = N.weights(cfg, 31)
        req = {i: tokens(cfg, n, i) for i, n in enumerate((90, 20, 3))}
        eng = serve(cfg, w, name=name, max_seqs=3)
        got = T.replay(eng, req, T.random_schedule(req, 3, 1))
        for i, t in req.items():
            T.check_rows(got[i], T.logits(cfg, w, t), "float32")


# --------------------------------------------------------- keys that stand out
def needle_model(seed, mixer, width=64):
    """Token 1 looks for token 0 wherever it is: only token 0 reaches latent
    dimension 0, whose key meets token 1's query far above every other score and
    whose value is unlike the others'."""
    cfg = N.config([(mixer, None)], width=width, vocab=60, cap=None, scale=1.0)
    w = N.weights(cfg, seed)
    H, D, R, V, K = (mixer[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    w["embed"][:, :2] = 0
    for i in range(2):
        w["embed"][i] = 0
        w["embed"][i, i] = np.sqrt(width)
    w["l0.norm1"][:2] = 1
    w["l0.hc1.in"] = np.abs(w["l0.hc1.in"])
    w["l0.mix.q"][:, :2] = 0
    w["l0.mix.dkv"][:, :2] = 0
    w["l0.mix.dkv"][0] = 0
    w["l0.mix.dkv"][0, 0] = 2.0
    w["l0.mix.dkv.norm"][0] = 1
    w["l0.mix.uk"][:, 0] = 0
    w["l0.mix.uv"][:, 0] = np.tile(np.linspace(-1, 1, V), H)
    for h in range(H):
        w["l0.mix.q"][h * (D + R)] = 0
        w["l0.mix.q"][h * (D + R), 1] = 1.0
        w["l0.mix.uk"][h * D] = 0
        # the score of the pair is 40
        w["l0.mix.uk"][h * D, 0] = 40 / (mixer["scale"] * np.sqrt(width) * np.sqrt(K))
    return cfg, {k: T.to_bf16(v) for k, v in w.items()}


NEEDLES = [0, 1, 31, 32, 62, 63, 64, 65, 127, 128, 191, 192, 250]
FORMS = {"in_latent_space": N.latent(), "expanded": LATENT["expanded"], "row_576": LATENT["row_576"]}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("form", sorted(FORMS))
def test_one_key_at_page_borders_and_far_away(serve, dtype, decoded, form):  # noqa: F811
    cfg, w = needle_model(33, FORMS[form])
    n = 260
    eng = serve(cfg, w, dtype, max_tokens=8 * 320, max_seqs=8)
    base = 2 + np.random.default_rng(34).integers(0, cfg["vocab"] - 2, n).astype(np.int32)
    for at in NEEDLES[::2] if form == "row_576" else NEEDLES:
        t = base.copy()
        t[at] = 0
        asked = [p for p in (2, 33, 63, 64, 66, 127, 129, 193, 251, 259) if p > at]
        t[asked] = 1
        cut = min(asked)
        steps = [[(0, cut)]] + [[(0, 1)]] * (n - cut) if decoded else [[(0, n)]]
        got = T.replay(eng, {0: t}, steps)[0][asked]
        want = T.logits(cfg, w, t)
        gone = t.copy()
        gone[at] = base[at]
        assert T.row_error(T.logits(cfg, w, gone)[asked], want[asked]).min() > 0.2
        e = T.row_error(got, want[asked])
        assert e.max() < (T.FP32_TOL if dtype == "float32" else T.BF16_TOL), (at, e)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("form", sorted(FORMS))
def test_far_keys_in_long_contexts(serve, dtype, form):  # noqa: F811
    """Contexts long enough that every launch form splits the keys; a heavy sink
    that counts once whatever the splits."""
    cfg, w = needle_model(35, FORMS[form])
    w["l0.mix.sink"] = T.to_bf16(np.linspace(37, 41, len(w["l0.mix.sink"])))
    n = 1200
    base = 2 + np.random.default_rng(36).integers(0, cfg["vocab"] - 2, n).astype(np.int32)
    eng = serve(cfg, w, dtype, max_tokens=2 * 1536, max_seqs=2, max_step_tokens=700)
    for at, asked in ((3, [700, 1199]), (1023, [1024, 1190])):
        t = base.copy()
        t[at], t[asked] = 0, 1
        want = T.logits(cfg, w, t)[asked]
        gone = np.where(np.arange(n) == at, base, t)
        assert T.row_error(T.logits(cfg, w, gone)[asked], want).min() > 0.1
        for steps in ([[(0, n)]],
                      [[(0, 400)], [(0, 300)], [(0, 3)], [(0, 460)]] + [[(0, 2)]] * 10 + [[(0, 1)]] * 17):
            got = T.replay(eng, {0: t}, steps)[0][asked]
            T.check_rows(got, want, dtype)


def test_key_just_ahead_is_not_seen(serve):  # noqa: F811
    for form in ("in_latent_space", "expanded"):
        cfg, w = needle_model(37, FORMS[form])
        eng = serve(cfg, w, name=form)
        for p in (5, 62, 63, 64, 127):
            t = 2 + np.random.default_rng(p).integers(0, cfg["vocab"] - 2, 140).astype(np.int32)
            t[p], t[p + 1] = 1, 0
            want = T.logits(cfg, w, t)
            for steps in ([[(0, 140)]], [[(0, p + 1)], [(0, 139 - p)]], [[(0, p)]] + [[(0, 1)]] * 5,
                          [[(0, 138)], [(0, 2)]]):
                got = T.replay(eng, {0: t}, steps)[0]
                T.check_rows(got, want[:len(got)], "float32")


def test_far_positions_turn_alike(serve):  # noqa: F811
    """Rotated scores alone, thousands of positions out."""
    cfg = N.config([(N.latent(dim=2, rot=32, vdim=8, rank=16, base=10000.0, scale=0.4), None)],
                   width=32, vocab=30, streams=1)
    w = N.weights(cfg, 39)
    t = tokens(cfg, 2600, 40)
    eng = serve(cfg, w, max_tokens=2624)
    want = T.logits(cfg, w, t)
    s = eng.open_seq()
    eng.step([(s, t[:2590], [])])
    got = np.concatenate([eng.step([(s, t[i:i + 1], [0])]) for i in range(2590, 2600)])
    assert T.row_error(got, want[2590:]).max() < 2e-4  # fp32 angles


# ------------------------------------------------------------------ decoding
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_long_decoding_of_a_batch(serve, name, dtype):  # noqa: F811
    """Hundreds of decode steps (replayed graphs) of three sequences, other work
    in between, every step against the restatement."""
    cfg = MODELS[name]
    w = N.weights(cfg, 41)
    req = {0: tokens(cfg, 300, 1), 1: tokens(cfg, 330, 2), 2: tokens(cfg, 270, 3)}
    steps = [[(0, 20), (1, 50)], [(2, 3)]]
    for k in range(267):
        steps.append([(0, 1), (1, 1), (2, 1)])
        if k % 60 == 30:
            steps.append([(1, 2)])
    at = {0: 20 + 267, 1: 50 + 2 * 4 + 267, 2: 3 + 267}
    steps.append([(i, len(req[i]) - at[i]) for i in req if at[i] < len(req[i])])
    got = T.replay(serve(cfg, w, dtype, max_seqs=3), req, steps)
    for i, t in req.items():
        T.check_rows(got[i], T.logits(cfg, w, t), dtype)


@pytest.mark.parametrize("batch", [20, 70])
def test_decoding_of_many(serve, batch):  # noqa: F811
    """Row counts of the larger product forms, every row its own sequence."""
    cfg = MODELS["plain"]
    w = N.weights(cfg, 43)
    eng = serve(cfg, w, max_seqs=batch, max_tokens=64 * batch)
    req = {i: tokens(cfg, 3 + i % 5 + 8, i) for i in range(batch)}
    steps = [[(i, 3 + i % 5) for i in req]] + [[(i, 1) for i in req]] * 8
    got = T.replay(eng, req, steps)
    for i, t in req.items():
        T.check_rows(got[i], T.logits(cfg, w, t), "float32")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("vocab,ff,inner", [(33001, 6144, 8192), (12288, 4096, 6144), (8200, 3100, 4100)])
def test_wide_products(serve, vocab, ff, inner, dtype):  # noqa: F811
    """Few rows against many columns: every tile form of the row counts up to 64,
    as portions and as decoded batches."""
    cfg = N.config([(N.mamba(inner=inner, state=2), N.dense(ff=ff)),
                    (N.latent(heads=40, dim=90, rot=8, vdim=8, rank=16), None)],
                   width=40, vocab=vocab, streams=2)
    w = N.weights(cfg, 44)
    eng = serve(cfg, w, dtype, max_seqs=40, max_tokens=64 * 40)
    for n in (16, 30, 47, 64):
        t = tokens(cfg, n, n)
        T.check_rows(run_whole(eng, t), T.logits(cfg, w, t), dtype)
    req = {i: tokens(cfg, 3, i) for i in range(40)}
    rows = (range(40), range(25), range(40), range(25, 40))
    got = T.replay(eng, req, [[(i, 1) for i in r] for r in rows])
    for i, t in req.items():
        T.check_rows(got[i], T.logits(cfg, w, t), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompts_of_wide_layers(serve, dtype):  # noqa: F811
    """Every product in its prompt form, alone and beside single tokens; expanded
    keys of several portions in one step, over pages that are not whole."""
    cfg = N.config([(N.mamba(inner=4100, state=2), N.dense(ff=4096)),
                    (N.latent(heads=40, dim=160, rot=8, vdim=24, rank=128), None)],
                   width=40, vocab=200, streams=2)
    w = N.weights(cfg, 46)
    eng = serve(cfg, w, dtype, max_seqs=4, max_tokens=64 * 60)
    req = {i: tokens(cfg, n, n) for i, n in enumerate((1030, 901, 400, 70))}
    want = {i: T.logits(cfg, w, t) for i, t in req.items()}
    T.check_rows(run_whole(eng, req[0]), want[0], dtype)
    got = T.replay(eng, req, [[(2, 30), (0, 355), (3, 69), (1, 401)], [(1, 331), (3, 1), (0, 330), (2, 370)],
                              [(0, 1), (1, 1)], [(1, 168), (0, 344)]])
    for i in req:
        T.check_rows(got[i], want[i], dtype)


def test_greedy_generation_through_the_scheduler(serve):  # noqa: F811
    cfg = MODELS["plain"]
    w = N.weights(cfg, 45)
    prompts = [tokens(cfg, n, 50 + n).tolist() for n in (1, 9, 70, 64, 130, 3, 40)]
    eng = serve(cfg, w, max_seqs=3, max_tokens=64 * 6, max_step_tokens=48)
    out = eng.generate_batch(prompts, 12)
    for p, o in zip(prompts, out):
        assert o == T.greedy(cfg, w, p, 12)
    assert eng.free_tokens == 64 * 6


def test_commands(gpu, tmp_path):
    cfg = MODELS["unlike_layers"]
    w = N.weights(cfg, 47)
    T.save(tmp_path / "m", cfg, w)
    a, b = tokens(cfg, 75, 1), tokens(cfg, 40, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:70].tolist(), "want": [0, 69]},
                                {"id": "b", "tokens": b[:2].tolist(), "want": []}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[2:].tolist(), "want": [37]}], "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": a[70:].tolist(), "want": [4]}], "end": ["a"]}]
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model",
                        str(tmp_path / "m"), "--dtype", "float32", "--out", str(tmp_path),
                        "--max-tokens", "192"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                       text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    la, lb = T.logits(cfg, w, a), T.logits(cfg, w, b)
    for i, want in enumerate((la[[0, 69]], lb[39:], la[74:])):
        got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(want.shape)
        T.check_rows(got, want, "float32")
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "generate"), "--model",
                        str(tmp_path / "m"), "--dtype", "float32", "--max-new", "6",
                        "--max-tokens", "512", ",".join(map(str, b))],
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [int(t) for t in r.stdout.strip().split(",")] == T.greedy(cfg, w, b.tolist(), 6)
