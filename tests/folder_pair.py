"""A folder model on the GPU beside its plain implementation, and the replay of a trace (not collected by pytest)."""
import json
import os
import subprocess

import numpy as np

from conftest import ROOT
from oracle.lokinex_oracle import bfloat16
from wick_amd import model as M
from wick_amd.model import NATIVE, RocmModel

TOL_F32 = 2e-5


def error(got, want):
    """Per row: rms of the difference over the rms of what is expected, the worst row."""
    got, want = np.atleast_2d(got).astype(np.float64), np.atleast_2d(want).astype(np.float64)
    assert got.shape == want.shape and np.isfinite(got).all()
    return float(np.max(np.sqrt(np.mean((got - want) ** 2, -1) / np.mean(want ** 2, -1))))


class Pair:
    """A model on the GPU and its oracle.  `synth` makes the tensors of a configuration, `oracle` is the plain implementation."""

    def __init__(self, ctx, tmp_path, synth, oracle, cfg, dtype, seed=1, context=320, t=None):
        self.cfg, self.dtype = cfg, dtype
        self.t = synth.tensors(cfg, seed) if t is None else t
        self.path = synth.write(tmp_path / f"m{seed}", cfg, self.t)
        self.gpu = RocmModel(ctx, self.path, context, dtype)
        self.oracle = oracle(cfg, self.t)
        self.rounded = oracle(cfg, self.t, r=bfloat16)
        self.tol = TOL_F32

    def tokens(self, n, seed=0):
        return np.random.default_rng(seed).integers(0, self.cfg["vocab"], n)

    def want(self, toks, trace=None):
        """What is expected for toks; sets the tolerance that `check` uses from here on."""
        self.oracle.reset()
        want = self.oracle.forward(toks, trace)
        if self.dtype == NATIVE:
            self.rounded.reset()
            self.tol = 3.0 * error(self.rounded.forward(toks), want)
        return want

    def check(self, got, want):
        e = error(got, want)
        assert e <= self.tol, f"error {e:.2e}, tolerance {self.tol:.2e}"

    def portions(self, toks, cuts):
        got, at = [], 0
        for c in cuts:
            got.append(self.gpu.forward(toks[at:at + c], at, np.arange(c)))
            at += c
        assert at == len(toks)
        return np.concatenate(got)

    def __enter__(self):
        return self

    def __exit__(self, *exc):
        self.gpu.free()


def greedy(p, prompt, n):
    p.oracle.reset()
    logits, out = p.oracle.forward(prompt)[-1], []
    for _ in range(n):
        out.append(M.greedy_pick(logits))
        logits = p.oracle.forward([out[-1]])[-1]
    return out


def run_trace(path, dtype, steps, out, max_tokens):
    proc = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", str(max_tokens)],
                          input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert proc.returncode == 0, proc.stderr[-2000:]
    return [l for l in proc.stdout.splitlines() if l.startswith("done ")]
