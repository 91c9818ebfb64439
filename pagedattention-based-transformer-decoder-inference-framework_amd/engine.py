"""Python face of the serving engine (llm_engine_* of include/llm_decoder.h):
models found by their config.json, sequences in cache slots, mixed-batch steps
and the request scheduler."""
from __future__ import annotations

import ctypes
import fcntl
import os
import subprocess
import sys
from contextlib import contextmanager
from pathlib import Path

import numpy as np

import llm_capi
from llm_capi import (LLM_BF16, LLM_F32, EngineConfig, EngineEntry, RequestParams, c_int,
                      c_void_p)

HERE = Path(__file__).resolve().parent
# The engine and its models without the other decoders' kernels (make engine).
ENGINE_LIB_PATH = HERE / "libllm_engine_hip.so"
DTYPES = {"bfloat16": LLM_BF16, "float32": LLM_F32}


@contextmanager
def _build_lock():
    try:
        f = open(HERE / ".build.lock", "w")
    except OSError:  # a read-only checkout: nothing to build there either
        yield
        return
    with f:
        fcntl.flock(f, fcntl.LOCK_EX)
        yield


def build_engine_library() -> Path:
    """Bring libllm_engine_hip.so up to date (compiles in a fresh checkout)."""
    with _build_lock():
        jobs = str(min(16, os.cpu_count() or 4))
        subprocess.run(["make", "-s", "-j", jobs, "-C", str(HERE), "engine"], check=True,
                       stdout=sys.stderr)
    return ENGINE_LIB_PATH


class Engine:
    """One model and its cache.

    max_tokens: the most tokens live sequences hold together, each rounded up to
    whole pages; max_seqs: the most live sequences."""

    def __init__(self, model_dir, *, dtype="bfloat16", max_seqs=4, max_tokens=4096,
                 max_seq_len=0, max_step_tokens=0, lib=None):
        self.lib = lib or llm_capi.load()
        self._h = c_void_p()
        cfg = EngineConfig(DTYPES[dtype], max_seqs, max_tokens, max_seq_len, max_step_tokens)
        self._check(self.lib.llm_engine_create(os.fsencode(str(model_dir)), ctypes.byref(cfg),
                                               ctypes.byref(self._h)))
        self.vocab = self.lib.llm_engine_vocab(self._h)
        self.max_seq_len = self.lib.llm_engine_max_seq_len(self._h)
        self.page_tokens = self.lib.llm_engine_page_tokens(self._h)
        self.layer_runs = self.lib.llm_engine_layer_runs(self._h)
        self.width = self.lib.llm_engine_width(self._h)

    def _check(self, rc):
        llm_capi.check(rc, self.lib)

    def close(self):
        if self._h:
            self.lib.llm_engine_destroy(self._h)
            self._h = c_void_p()

    def __enter__(self):
        return self

    def __exit__(self, *_):
        self.close()

    def __del__(self):
        try:
            self.close()
        except Exception:  # interpreter shutdown
            pass

    @property
    def free_tokens(self) -> int:
        return self.lib.llm_engine_free_tokens(self._h)

    def open_seq(self) -> int:
        s = c_int()
        self._check(self.lib.llm_engine_open(self._h, ctypes.byref(s)))
        return s.value

    def close_seq(self, seq: int) -> None:
        self._check(self.lib.llm_engine_close(self._h, seq))

    def seq_len(self, seq: int) -> int:
        return self.lib.llm_engine_seq_len(self._h, seq)

    def step(self, entries):
        """entries: [(seq, tokens, want)]; one batch.  Returns fp32 logits
        [wanted rows][vocab] in the order of the entries and of `want`."""
        arr = (EngineEntry * max(len(entries), 1))()
        keep, rows = [], 0
        for i, (seq, tokens, want) in enumerate(entries):
            t = np.ascontiguousarray(tokens, dtype=np.int32)
            w = np.ascontiguousarray(want, dtype=np.int32)
            keep.append((t, w))
            arr[i] = EngineEntry(seq, t.ctypes.data, t.size, w.ctypes.data, w.size)
            rows += w.size
        out = np.empty((rows, self.vocab), np.float32)
        self._check(self.lib.llm_engine_step(self._h, arr, len(entries),
                                             out.ctypes.data if rows else None))
        return out

    def step_taps(self, entries):
        """step, and the residual stream after every layer run
        [layer runs][tokens][width]."""
        n = sum(len(t) for _, t, _ in entries)
        tap = np.empty((self.layer_runs, n, self.width), np.float32)
        self._check(self.lib.llm_engine_set_tap(self._h, tap.ctypes.data))
        try:
            return self.step(entries), tap
        finally:
            self._check(self.lib.llm_engine_set_tap(self._h, None))

    def submit(self, prompt, max_new_tokens, *, temperature=0.0, top_k=0, top_p=1.0, seed=0,
               eos_token=-1) -> int:
        p = np.ascontiguousarray(prompt, dtype=np.int32)
        r = c_int()
        par = RequestParams(max_new_tokens, temperature, top_k, top_p, seed, eos_token)
        self._check(self.lib.llm_engine_submit(self._h, p.ctypes.data, p.size, ctypes.byref(par),
                                               ctypes.byref(r)))
        return r.value

    def run(self) -> int:
        """One scheduler pass; returns the requests still waiting or running."""
        a = c_int()
        self._check(self.lib.llm_engine_run(self._h, ctypes.byref(a)))
        return a.value

    def result(self, request: int, cap: int = 1 << 16):
        """(tokens generated so far, finished); a finished request is forgotten."""
        out = np.empty(cap, np.int32)
        n, fin = c_int(), c_int()
        self._check(self.lib.llm_engine_result(self._h, request, out.ctypes.data, cap,
                                               ctypes.byref(n), ctypes.byref(fin)))
        return out[:min(n.value, cap)].tolist(), bool(fin.value)

    def generate_batch(self, prompts, max_new_tokens, **sampling):
        """Submit every prompt, run the scheduler dry; lists of generated ids."""
        ids = [self.submit(p, max_new_tokens, **sampling) for p in prompts]
        while self.run():
            pass
        return [self.result(i, max(max_new_tokens, 1))[0] for i in ids]
