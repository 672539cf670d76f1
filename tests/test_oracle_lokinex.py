"""The plain Lokinex implementation against itself: what has to hold whatever the weights are.  These properties are what the GPU
tests rely on when they compare with it."""
import numpy as np
import pytest

import lokinex_synth as S
from oracle import lokinex_oracle as O


@pytest.fixture(scope="module")
def model():
    cfg = S.mixed()
    return cfg, O.LokinexOracle(cfg, S.tensors(cfg, 3))


def test_portions_do_not_change_the_logits(model):
    cfg, o = model
    toks = np.random.default_rng(0).integers(0, cfg["vocab"], 19)
    o.reset()
    whole = o.forward(toks)
    for cuts in ([1] * 19, [2, 2, 3, 1, 5, 6], [17, 2]):
        o.reset()
        got, at = [], 0
        for c in cuts:
            got.append(o.forward(toks[at:at + c]))
            at += c
        assert np.allclose(np.concatenate(got), whole, atol=1e-10)


def test_loop_order_counts_every_pass(model):
    cfg, o = model
    assert [i for i, _ in o.order] == [0, 1, 2, 1, 2, 3]
    assert [s for _, s in o.order] == [None, 0, None, 1, None, None]
    trace = []
    o.reset()
    o.forward([1, 2, 3], trace)
    assert len(trace) == 6 and all(x.shape == (3, cfg["width"]) for x in trace)


def test_rotation_depends_on_the_distance_only():
    rng = np.random.default_rng(1)
    q, k = rng.standard_normal((1, 8)), rng.standard_normal((1, 8))
    dot = lambda a, b: float(np.sum(O.rope_interleaved(q, np.array([a]), 100.0) * O.rope_interleaved(k, np.array([b]), 100.0)))
    assert np.isclose(dot(7.0, 3.0), dot(104.0, 100.0)) and not np.isclose(dot(7.0, 3.0), dot(8.0, 3.0))


def test_recurrence_keeps_its_norm_when_the_gate_is_closed():
    """a^2 + (1 - a^2) = 1: with i u = 1 throughout, S stays between 0 and 1 / sqrt of the step it takes."""
    cfg = S.config([S.layer(S.rglru(width=4, blocks=1, conv=1))], width=4)
    t = S.tensors(cfg, 2)
    t = {k: (v * 0 if k.startswith("l0.mix.") else v) for k, v in t.items()}
    t["l0.mix.lam"] = np.full(4, -30.0)  # log a ~ -4e-13: the state neither decays nor takes anything in
    out, (S1, _) = O.rglru(np.ones((5, 4)), t, "l0.mix.", cfg["layers"][0]["mixer"], (np.full(4, 2.0), np.zeros((0, 4))))
    assert np.allclose(S1, 2.0)


def test_table_decides_the_experts():
    cfg = S.config([S.layer(S.rglru(), S.moe(top=2, shared=None))])
    t = S.tensors(cfg, 5)
    h = np.random.default_rng(2).standard_normal((2, cfg["width"]))
    a = O.table_moe(h, t, "l0.mlp.", cfg["layers"][0]["mlp"], [3, 4])
    e = t["l0.mlp.table"][3]
    want = sum(O.gated_mlp(h[:1], t, f"l0.mlp.e{int(k)}.")[0] for k in e) / 2
    assert np.allclose(a[0], want)
