"""The plain Zirurax implementation against itself and against closed forms: what the GPU tests rely on when they compare with it."""
import numpy as np
import pytest

import zirurax_synth as S
from oracle import zirurax_oracle as O


@pytest.fixture(scope="module")
def model():
    cfg = S.mixed()
    return cfg, O.ZiruraxOracle(cfg, S.tensors(cfg, 3))


def test_portions_do_not_change_the_logits(model):
    cfg, o = model
    toks = np.random.default_rng(0).integers(0, cfg["vocab"], 90)
    o.reset()
    whole = o.forward(toks)
    for cuts in ([1] * 90, [2, 2, 3, 1, 5, 6, 71], [88, 2]):
        o.reset()
        got, at = [], 0
        for c in cuts:
            got.append(o.forward(toks[at:at + c]))
            at += c
        assert np.allclose(np.concatenate(got), whole, atol=1e-9)


def test_window_ends_where_it_says():
    """What lies outside the window does not show, what lies at its edge does (one layer without the recurrence's share)."""
    cfg = S.config([S.layer(S.attention(window=5), ff=None)])
    t = S.tensors(cfg, 2)
    t["l0.mix.right.out"] = t["l0.mix.right.out"] * 0
    toks = np.arange(12)

    def last(change):
        o = O.ZiruraxOracle(cfg, t)
        k = toks.copy()
        k[change] = 99
        return o.forward(k)[-1]

    same = O.ZiruraxOracle(cfg, t).forward(toks)[-1]
    assert np.array_equal(last(11 - 5), same) and not np.allclose(last(11 - 4), same)


def test_frequencies_keep_the_short_and_stretch_the_long_wavelengths():
    r = S.rot(64, 1e6)
    plain, f, sc = O.frequencies({**r, "scaling": None}), O.frequencies(r), r["scaling"]
    wave = 2 * np.pi / plain
    short, long = wave < sc["original"] / sc["high"], wave > sc["original"] / sc["low"]
    assert short.any() and long.any() and (~short & ~long).any()
    assert np.allclose(f[short], plain[short]) and np.allclose(f[long], plain[long] / sc["factor"])
    mid = f[~short & ~long] / plain[~short & ~long]
    assert ((mid > 1 / sc["factor"]) & (mid < 1)).all() and (np.diff(f) < 0).all()


def test_recurrence_is_the_sum_over_the_past():
    """y_t = sum over j <= t of exp(sum of the log decays behind j) dt_j (C_t . B_j) x_j + D x_t."""
    cfg = S.config([S.layer(right=S.ssd(conv=1, parts=1))])
    m, t = cfg["layers"][0]["mixer"]["right"], S.tensors(cfg, 4)
    p, H, P, N, G, n = "l0.mix.right.", m["heads"], m["vdim"], m["state"], m["groups"], 9
    h = np.random.default_rng(1).standard_normal((n, cfg["width"]))
    got, _ = O.ssd(h, t, p, m, 1e-5, (np.zeros((H, N, P)), np.zeros((0, H * P + 2 * G * N))))
    w = h @ t[p + "in"].T
    inner = H * P
    u = O.silu(w[:, inner:2 * inner + 2 * G * N] * t[p + "conv"][:, 0] + t[p + "conv.b"])
    dt = np.log1p(np.exp(w[:, 2 * inner + 2 * G * N:] + t[p + "dt_bias"]))
    y = np.zeros((n, inner))
    for x in range(H):
        b = u[:, inner + x // (H // G) * N:][:, :N]
        c = u[:, inner + G * N + x // (H // G) * N:][:, :N]
        v = u[:, x * P:(x + 1) * P]
        la = np.cumsum(-np.exp(t[p + "A_log"][x]) * dt[:, x])
        k = np.tril(np.exp(np.minimum(la[:, None] - la[None, :], 0.0)) * dt[None, :, x] * (c @ b.T))
        y[:, x * P:(x + 1) * P] = k @ v + t[p + "D"][x] * v
    y = O.rms(y * O.silu(w[:, :inner]), 1e-5) * t[p + "norm"]
    assert np.allclose(got, y @ t[p + "o"].T)
