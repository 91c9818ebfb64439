"""Layer-stack models (csrc/layer_stack.cpp) and the serving engine against the
plain restatement (oracle/layer_stack.py): each mechanism alone, every way of
cutting a prompt, mixed batches, reused pages and slots, far and near keys, and
generation through the scheduler."""
import json
import subprocess
import sys

import numpy as np
import pytest

import _layer_stack as T
from conftest import ROOT

pytestmark = pytest.mark.gpu


@pytest.fixture
def serve(gpu, tmp_path):
    """serve(cfg, w, dtype, ...) -> Engine of a saved model."""
    import engine
    made = []

    def make(cfg, w, dtype="float32", max_tokens=1024, name="m", **kw):
        T.save(tmp_path / name, cfg, w)
        e = engine.Engine(tmp_path / name, dtype=dtype, max_tokens=max_tokens, **kw)
        made.append(e)
        return e
    yield make
    for e in made:
        e.close()


def tokens(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.int32)


def run_whole(eng, toks):
    s = eng.open_seq()
    out = eng.step([(s, toks, range(len(toks)))])
    eng.close_seq(s)
    return out


DTYPES = ["float32", "bfloat16"]


def model_weights(cfg, seed, dtype):
    w = T.weights(cfg, seed)
    return T.clear_choices(w) if dtype == "bfloat16" else w


# ---------------------------------------------------------------- mechanisms
def one_layer(a=None, m=None, **kw):
    return T.config([(a or T.attn(), m)], **kw)


@pytest.mark.parametrize("dtype", DTYPES)
def test_norm_and_head_alone(serve, dtype):
    """A mixer that puts out nothing: embedding, final norm, head (the norm of a
    zero row is zero)."""
    cfg = one_layer(width=72, eps=0.3)
    w = T.weights(cfg, 1)
    w["l0.mix.o"][:] = 0
    t = tokens(cfg, 30, 2)
    T.check_rows(run_whole(serve(cfg, w, dtype), t), T.logits(cfg, w, t), dtype)


ATTENTION = {
    "plain": T.attn(rot=0),
    "rotary": T.attn(scaling=None),
    "rotary_all_dims": T.attn(rot=32, scaling=None),
    "yarn": T.attn(),
    "yarn_narrow_ramp": T.attn(rot=32, scaling=dict(factor=8.0, original=4096, fast=1.0, slow=1.0)),
    "one_key_head": T.attn(heads=8, kv_heads=1),
    "head_each": T.attn(heads=4, kv_heads=4),
    "group_of_three": T.attn(heads=6, kv_heads=2),
    "group_of_twenty": T.attn(heads=20, kv_heads=1, dim=16, vdim=16, rot=8),
    "small_odd_values": T.attn(dim=24, vdim=7, rot=10),
    "value_wider": T.attn(dim=40, vdim=72, rot=20),
    "dim_128": T.attn(dim=128, vdim=112, rot=64),
    "dim_256": T.attn(heads=2, kv_heads=1, dim=256, vdim=200, rot=96),
    "scale": T.attn(scale=0.6),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(ATTENTION))
def test_attention_alone(serve, name, dtype):
    cfg = one_layer(ATTENTION[name])
    w = T.weights(cfg, 3)
    t = tokens(cfg, 150, 4)
    eng = serve(cfg, w, dtype)
    want = T.logits(cfg, w, t)
    T.check_rows(run_whole(eng, t), want, dtype)
    got = T.replay(eng, {0: t}, [[(0, n)] for n in T.portions(130, [17]) + [1] * 20])[0]
    T.check_rows(got, want, dtype)


@pytest.mark.parametrize("sink", [-30.0, 0.0, 6.0, 40.0])
def test_sink(serve, sink):
    """From no weight to nearly all of it; a sink that is left out, scaled or
    counted per key shows in the first positions."""
    cfg = one_layer(T.attn(heads=8, kv_heads=2, scale=0.4))
    w = T.weights(cfg, 5)
    w["l0.mix.sink"] = T.to_bf16(sink + np.linspace(-1, 1, 8))
    t = tokens(cfg, 140, 6)
    eng = serve(cfg, w)
    want = T.logits(cfg, w, t)
    T.check_rows(run_whole(eng, t), want, "float32")
    got = T.replay(eng, {0: t}, [[(0, 100)]] + [[(0, 1)]] * 40)[0]
    T.check_rows(got, want, "float32")
    if sink > -30:  # the test sees the sink
        w2 = dict(w, **{"l0.mix.sink": w["l0.mix.sink"] - 100})
        assert T.row_error(T.logits(cfg, w2, t), want)[:20].max() > 100 * T.FP32_TOL


MOE = {
    "plain": T.moe(shared=0),
    "shared": T.moe(),
    "one_of_one": T.moe(experts=1, top=1),
    "all_of_five": T.moe(experts=5, top=5, ff=33, shared=65),
    "many": T.moe(experts=130, top=6, ff=8, shared=16),
    "odd_sizes": T.moe(experts=7, top=3, ff=29, shared=31),
    "tight_limit": T.moe(limit=0.05, shared_limit=0.2),
    "wide_shared": T.moe(ff=16, shared=200),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MOE))
def test_experts_alone(serve, name, dtype):
    """The mixer puts out nothing, so the layer is its feed-forward."""
    cfg = one_layer(m=MOE[name])
    w = T.weights(cfg, 7)
    w["l0.mix.o"][:] = 0
    eng = serve(cfg, w, dtype)
    for n, seed in ((1, 8), (19, 9), (300, 10)):  # one token, small and large routing forms
        t = tokens(cfg, n, seed)
        T.check_rows(run_whole(eng, t), T.logits(cfg, w, t), dtype, close_calls=True)


def test_correction_chooses_but_does_not_weigh(serve):
    cfg = one_layer(m=T.moe(experts=6, top=2, shared=0))
    w = T.weights(cfg, 11)
    w["l0.mix.o"][:] = 0
    w["l0.mlp.correction"] = T.to_bf16(np.array([0, 3, 0, 0, 3.5, 0]))  # 1 and 4 always
    t = tokens(cfg, 40, 12)
    want = T.logits(cfg, w, t)
    T.check_rows(run_whole(serve(cfg, w), t), want, "float32")
    w2 = dict(w, **{"l0.mlp.correction": 0 * w["l0.mlp.correction"]})
    assert np.median(T.row_error(T.logits(cfg, w2, t), want)) > 0.01


@pytest.mark.parametrize("loop", [(0, 1, 3), (1, 3, 2), (0, 3, 2), (2, 3, 4), (1, 2, 1), (1, 1, 2)])
def test_repeated_layers(serve, loop):
    """Each pass has its own cache and starts with the embedding added again."""
    cfg = T.config([(T.attn(), None), (T.attn(), T.moe(experts=4)), (T.attn(), None)], loop=loop)
    w = T.weights(cfg, 13)
    t = tokens(cfg, 90, 14)
    eng = serve(cfg, w)
    want = T.logits(cfg, w, t)
    T.check_rows(run_whole(eng, t), want, "float32")
    T.check_rows(T.replay(eng, {0: t}, [[(0, 50)]] + [[(0, 1)]] * 40)[0], want, "float32")


def test_residual_after_every_layer(serve):
    cfg = T.config([(T.attn(), T.moe()), (T.attn(), None)], loop=(0, 2, 2), width=100)
    w = T.weights(cfg, 15)
    t = tokens(cfg, 25, 16)
    eng = serve(cfg, w)
    s = eng.open_seq()
    _, tap = eng.step_taps([(s, t, [0])])
    from oracle import layer_stack as ls
    want = []
    ls.forward(cfg, w, t, taps=want)
    assert tap.shape == (4, 25, 100) and len(want) == 4
    for a, b in zip(tap, want):
        assert np.abs(a - b).max() < 1e-4 * np.abs(b).max()


# ------------------------------------------------------------- whole models
MODELS = {
    "plain": T.config([(T.attn(heads=8, kv_heads=1, vdim=24), T.moe())] * 3, loop=(1, 3, 2)),
    "unlike_layers": T.config(
        [(T.attn(), T.moe(experts=5, top=1, shared=0)),
         (T.attn(heads=6, kv_heads=3, dim=20, vdim=12, rot=20, base=50.0), None),
         (T.attn(heads=2, kv_heads=1, dim=80, vdim=33, rot=0), T.moe(experts=40, top=4, ff=12)),
         (T.attn(), T.moe())],
        width=84, vocab=211, loop=(0, 2, 2)),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
@pytest.mark.parametrize("sizes", [[2], [3, 2, 7], [16], [64], [63, 65], [1]])
def test_portions(serve, name, sizes, dtype):
    cfg = MODELS[name]
    w = model_weights(cfg, 17, dtype)
    t = tokens(cfg, 140, 18)
    eng = serve(cfg, w, dtype)
    got = T.replay(eng, {0: t}, [[(0, n)] for n in T.portions(len(t), sizes)])[0]
    T.check_rows(got, T.logits(cfg, w, t), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_mixed_batches_with_pages_and_slots_used_again(serve, name, dtype):
    """A pool that just holds the live requests: unequal requests, together and
    one after another in the same pages, each as if it were alone."""
    cfg = MODELS[name]
    w = model_weights(cfg, 19, dtype)
    req = {i: tokens(cfg, n, 20 + i) for i, n in
           enumerate([1, 70, 190, 5, 128, 64, 33, 150, 65, 2, 100, 129])}
    steps = T.random_schedule(req, 4, 21)
    most = T.most_pages(req, steps)
    eng = serve(cfg, w, dtype, max_tokens=64 * most, max_seqs=4)
    free = eng.free_tokens
    got = T.replay(eng, req, steps)
    assert eng.free_tokens == free
    for i, t in req.items():
        T.check_rows(got[i], T.logits(cfg, w, t), dtype)


def test_batch_alone_and_step_size_give_the_same(serve):
    """The same request alone, beside others, and with a small step size."""
    cfg = MODELS["plain"]
    w = T.weights(cfg, 23)
    a, b, c = (tokens(cfg, n, n) for n in (130, 77, 20))
    eng = serve(cfg, w, max_seqs=3)
    small = serve(cfg, w, max_seqs=3, max_step_tokens=24, name="small")
    alone = run_whole(eng, a)
    together = T.replay(eng, {0: c, 1: a, 2: b}, [[(0, 20), (1, 130), (2, 77)]])[1]
    cut = T.replay(small, {0: c, 1: a, 2: b}, [[(0, 20), (1, 130), (2, 77)]])[1]
    assert T.row_error(together, alone).max() < T.FP32_TOL
    assert T.row_error(cut, alone).max() < T.FP32_TOL


# --------------------------------------------------------- keys that stand out
def needle_model(seed, heads=4):
    """A model whose token 1 looks for token 0 wherever it is: its query meets
    that key, in dimensions that are not rotated, far above every other score,
    and token 0's value is unlike the others'."""
    a = T.attn(heads=heads, kv_heads=2, dim=32, vdim=16, rot=8)
    cfg = T.config([(a, None)], width=64, vocab=60)
    w = T.weights(cfg, seed)
    W = cfg["width"]
    w["embed"][:, :2] = 0
    w["embed"][0] = 0
    w["embed"][0, 0] = np.sqrt(W)
    w["embed"][1] = 0
    w["embed"][1, 1] = np.sqrt(W)
    w["l0.norm1"][:2] = 1
    for n in ("q", "k", "v"):
        w["l0.mix." + n][:, :2] = 0
    for h in range(2):
        w["l0.mix.k"][32 * h + 20, 0] = 4.0      # key of token 0
        w["l0.mix.v"][16 * h:16 * h + 16, 0] = np.linspace(-1, 1, 16)
    for h in range(heads):
        w["l0.mix.q"][32 * h + 20, 1] = 4.0      # query of token 1: score 16 * 64 / sqrt(32)
        w["l0.mix.q"][32 * h + 20, 2:] = 0
    w["l0.mix.k"][[20, 52], 1:] = 0
    return cfg, {k: T.to_bf16(v) for k, v in w.items()}


NEEDLES = [0, 1, 31, 32, 62, 63, 64, 65, 127, 128, 191, 192, 250]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
def test_one_key_at_page_borders_and_far_away(serve, dtype, decoded):
    cfg, w = needle_model(29)
    n = 260
    eng = serve(cfg, w, dtype, max_tokens=8 * 320, max_seqs=8)
    base = 2 + np.random.default_rng(30).integers(0, cfg["vocab"] - 2, n).astype(np.int32)
    ask = [p for p in (2, 33, 63, 64, 66, 127, 129, 193, 251, 259)]
    for at in NEEDLES:
        t = base.copy()
        t[at] = 0
        asked = [p for p in ask if p > at]
        t[asked] = 1
        cut = min(asked)
        steps = [[(0, cut)]] + [[(0, 1)]] * (n - cut) if decoded else [[(0, n)]]
        got = T.replay(eng, {0: t}, steps)[0][asked]
        want = T.logits(cfg, w, t)
        gone = t.copy()
        gone[at] = base[at]
        shows = T.row_error(T.logits(cfg, w, gone)[asked], want[asked])
        assert shows.min() > 0.3  # the key decides these rows
        e = T.row_error(got, want[asked])
        assert e.max() < (T.FP32_TOL if dtype == "float32" else T.BF16_TOL), (at, e)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("group", [2, 8])
def test_far_keys_in_long_contexts(serve, dtype, group):
    """Contexts long enough that every launch form splits the keys: whole
    prompts, prompts past the step size, short portions and single tokens far
    from the key; a heavy sink that counts once whatever the splits."""
    cfg, w = needle_model(33, heads=2 * group)
    w["l0.mix.sink"] = T.to_bf16(np.linspace(8, 11, 2 * group))
    n = 1200
    base = 2 + np.random.default_rng(34).integers(0, cfg["vocab"] - 2, n).astype(np.int32)
    eng = serve(cfg, w, dtype, max_tokens=2 * 1536, max_seqs=2, max_step_tokens=700)
    for at, asked in ((3, [700, 1199]), (1023, [1024, 1190])):
        t = base.copy()
        t[at], t[asked] = 0, 1
        want = T.logits(cfg, w, t)[asked]
        gone = np.where(np.arange(n) == at, base, t)
        assert T.row_error(T.logits(cfg, w, gone)[asked], want).min() > 0.3
        for steps in ([[(0, n)]],
                      [[(0, 400)], [(0, 300)], [(0, 3)], [(0, 460)]] + [[(0, 2)]] * 10 + [[(0, 1)]] * 17):
            got = T.replay(eng, {0: t}, steps)[0][asked]
            T.check_rows(got, want, dtype)


def test_key_just_ahead_is_not_seen(serve):
    """The standing-out key one place after the query, in one portion and across
    the portion's edge."""
    cfg, w = needle_model(31)
    eng = serve(cfg, w)
    for p in (5, 62, 63, 64, 127):
        t = 2 + np.random.default_rng(p).integers(0, cfg["vocab"] - 2, 140).astype(np.int32)
        t[p], t[p + 1] = 1, 0
        want = T.logits(cfg, w, t)
        for steps in ([[(0, 140)]], [[(0, p + 1)], [(0, 139 - p)]], [[(0, p)]] + [[(0, 1)]] * 5,
                      [[(0, 140 - 2)], [(0, 2)]]):
            got = T.replay(eng, {0: t}, steps)[0]
            T.check_rows(got, want[:len(got)], "float32")


# ------------------------------------------------------------------ decoding
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_of_a_batch(serve, dtype):
    """Hundreds of decode steps (replayed graphs) of three sequences, other work
    in between, every step against the restatement."""
    cfg = MODELS["plain"]
    w = model_weights(cfg, 37, dtype)
    req = {0: tokens(cfg, 300, 1), 1: tokens(cfg, 330, 2), 2: tokens(cfg, 270, 3)}
    steps = [[(0, 20), (1, 50)], [(2, 3)]]
    for k in range(267):
        steps.append([(0, 1), (1, 1), (2, 1)])
        if k % 60 == 30:
            steps.append([(1, 2)])
    at = {0: 20, 1: 50 + 2 * 4, 2: 3}
    at = {i: n + 267 for i, n in at.items()}
    steps.append([(i, len(req[i]) - at[i]) for i in req if at[i] < len(req[i])])
    got = T.replay(serve(cfg, w, dtype, max_seqs=3), req, steps)
    for i, t in req.items():
        T.check_rows(got[i], T.logits(cfg, w, t), dtype)


def test_greedy_generation_through_the_scheduler(serve):
    """More requests than slots and than the pool holds at once."""
    cfg = MODELS["plain"]
    w = T.weights(cfg, 41)
    prompts = [tokens(cfg, n, 50 + n).tolist() for n in (1, 9, 70, 64, 130, 3, 40)]
    eng = serve(cfg, w, max_seqs=3, max_tokens=64 * 6, max_step_tokens=48)
    out = eng.generate_batch(prompts, 12)
    for p, o in zip(prompts, out):
        assert o == T.greedy(cfg, w, p, 12)
    assert eng.free_tokens == 64 * 6
    # the first generated id as the end of the request
    eos = out[1][3]
    cut = eng.generate_batch(prompts, 12, eos_token=eos)
    for o, c in zip(out, cut):
        assert c == (o[:o.index(eos) + 1] if eos in o else o)


def test_sampled_generation_does_not_depend_on_the_batch(serve):
    cfg = MODELS["plain"]
    w = T.weights(cfg, 43)
    prompts = [tokens(cfg, n, 60 + n).tolist() for n in (5, 66, 12)]
    eng = serve(cfg, w, max_seqs=3)
    par = dict(temperature=0.9, top_k=20, top_p=0.95)
    ids = [eng.submit(p, 10, seed=s, **par) for s, p in enumerate(prompts)]
    while eng.run():
        pass
    together = [eng.result(i)[0] for i in ids]
    for s, p in enumerate(prompts):
        assert eng.generate_batch([p], 10, seed=s, **par)[0] == together[s]
    assert eng.generate_batch([prompts[0]], 10, seed=99, **par)[0] != together[0]


def test_refused_requests_leave_the_engine_working(serve):
    import llm_capi
    cfg = MODELS["plain"]
    w = T.weights(cfg, 47)
    eng = serve(cfg, w, max_seqs=2, max_tokens=128)
    a, b = eng.open_seq(), eng.open_seq()
    with pytest.raises(llm_capi.LlmError):
        eng.open_seq()
    for bad in ([(a, [cfg["vocab"]], [])], [(a, [1], [1])], [(a, [1], []), (a, [2], [])],
                [(a, list(range(129)), [])], [(7, [1], [])]):
        with pytest.raises(llm_capi.LlmError):
            eng.step(bad)
    t = tokens(cfg, 100, 1)
    eng.step([(a, t, [])])
    with pytest.raises(llm_capi.LlmError):  # no page left for it
        eng.step([(b, t[:3], [0])])
    eng.close_seq(a)
    T.check_rows(eng.step([(b, t[:3], [0, 1, 2])]), T.logits(cfg, w, t[:3]), "float32")
    eng.close_seq(b)
    with pytest.raises(llm_capi.LlmError):
        eng.submit(t.tolist(), 60)


# --------------------------------------------------------------- front ends
def test_trace_run_replays_steps(gpu, tmp_path):
    cfg = MODELS["plain"]
    w = T.weights(cfg, 53)
    T.save(tmp_path / "m", cfg, w)
    a, b = tokens(cfg, 75, 1), tokens(cfg, 40, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:70].tolist(), "want": [0, 69]},
                                {"id": "b", "tokens": b[:2].tolist(), "want": []}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[2:].tolist(), "want": [37]}], "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": a[70:].tolist(), "want": []}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "c", "tokens": b.tolist(), "want": [39]}], "end": ["c"]}]
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model",
                        str(tmp_path / "m"), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "192"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                       text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not (out / "2.f32").exists()
    la, lb = T.logits(cfg, w, a), T.logits(cfg, w, b)
    got = np.fromfile(out / "0.f32", "<f4").reshape(2, -1)
    T.check_rows(got, la[[0, 69]], "float32")
    for s in (1, 3):
        T.check_rows(np.fromfile(out / f"{s}.f32", "<f4").reshape(1, -1), lb[39:], "float32")


def test_generate_command(gpu, tmp_path):
    cfg = MODELS["plain"]
    w = T.weights(cfg, 59)
    T.save(tmp_path / "m", cfg, w)
    prompts = [tokens(cfg, n, n).tolist() for n in (4, 9)]
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "generate"), "--model",
                        str(tmp_path / "m"), "--dtype", "float32", "--max-new", "6",
                        "--max-tokens", "512"] + [",".join(map(str, p)) for p in prompts],
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    got = [[int(t) for t in x.split(",")] for x in r.stdout.split()]
    assert got == [T.greedy(cfg, w, p, 6) for p in prompts]


# ------------------------------------------- the other models behind the engine
def write_decoder(folder, arch, seed):
    """A small fp32 weight folder of the dense decoders with a config.json."""
    L, H, D, V = 2, 2, 64, 96
    hid, inter = H * D, 4 * H * D
    rng = np.random.default_rng(seed)
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(
        {"architecture": arch, "num_layers": L, "num_heads": H, "head_dim": D, "vocab_size": V,
         "max_seq_len": 256, "attn_scale": 0.125}))

    def put(name, *shape, s=0.05):
        (rng.standard_normal(shape) * s).astype("<f4").tofile(folder / name)
    put("embedding.bin", V, hid, s=1.0)
    for i in range(L):
        (folder / f"layer_{i}").mkdir()
        for ln in ("ln1", "ln2"):
            np.concatenate([np.ones(hid), 0.1 * rng.standard_normal(hid)]).astype("<f4").tofile(
                folder / f"layer_{i}" / f"{ln}.bin")
        for m in ("wq", "wk", "wv", "wo"):
            put(f"layer_{i}/attn_{m}.bin", hid, hid)
        put(f"layer_{i}/mlp_fc1.bin", hid, inter)
        put(f"layer_{i}/mlp_fc2.bin", inter, hid)
        put(f"layer_{i}/mlp_biases.bin", inter + hid)
    return dict(L=L, H=H, D=D, hid=hid, V=V)


@pytest.mark.parametrize("arch", ["CUDADecoder", "INT8Decoder"])
def test_dense_decoders_behind_the_engine(gpu, tmp_path, arch):
    """The registry serves the dense decoders too: portions and mixed batches
    give what their own step function gives."""
    import engine
    import llm_decoder
    import torch
    c = write_decoder(tmp_path / "m", arch, 61)
    toks = {i: np.random.default_rng(i).integers(0, c["V"], n).astype(np.int32)
            for i, n in enumerate((40, 25, 3))}
    dec = getattr(llm_decoder, arch)(c["L"], c["H"], c["D"], c["hid"], c["V"], 256, max_batch=1,
                                     attn_scale=0.125)
    dec.load_weights(str(tmp_path / "m"))
    want = {}
    buf = torch.empty((1, c["V"]), device="cuda")
    for i, t in toks.items():
        dec.begin_synthetic(1, 0, 0, False)
        rows = []
        for x in t:
            dec.step([int(x)], logits_ptr=buf.data_ptr())
            torch.cuda.synchronize()
            rows.append(buf.cpu().numpy()[0].copy())
        want[i] = np.stack(rows)
    eng = engine.Engine(tmp_path / "m", max_seqs=3, max_tokens=192)
    got = T.replay(eng, toks, [[(0, 17)], [(0, 1), (1, 20), (2, 3)], [(1, 1), (0, 1)],
                               [(0, 21), (1, 4)]])
    for i in toks:
        # int8 rounding of activations flips with the order of fp32 sums
        assert T.row_error(got[i], want[i]).max() < (5e-3 if arch == "CUDADecoder" else 5e-2)
    assert eng.generate_batch([t.tolist() for t in toks.values()], 4) is not None
    with pytest.raises(Exception, match="float32"):
        engine.Engine(tmp_path / "m", dtype="float32", max_tokens=192)
    eng.close()
