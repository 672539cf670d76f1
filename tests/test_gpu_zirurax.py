"""Zirurax on the GPU, through the model handle, against the plain implementation (oracle/zirurax_oracle.py).

The f32 model is held to f32 rounding, which shows a wrong key, a lost state or a window that is off by one anywhere; the served
(bfloat16) model to three times what rounding the products' activations does to the plain implementation on the same tokens.  Where
random weights would hide a fault -- one far key among hundreds, the edge of a window -- the weights are made so that the fault would
move the logits by far more than the tolerance, and the test says so first."""
import copy
import subprocess
import sys

import numpy as np
import pytest

import folder_pair
import zirurax_synth as S
from conftest import ROOT
from folder_pair import TOL_F32, error, greedy, run_trace
from oracle import zirurax_oracle as O
from wick_amd import model as M
from wick_amd.checkpoint import from_bf16, to_bf16
from wick_amd.model import F32, NATIVE, RocmModel
from wick_amd.rocm import RocmError

pytestmark = pytest.mark.gpu

BOTH = pytest.mark.parametrize("dtype", [F32, NATIVE], ids=["f32", "bf16"])


def Pair(ctx, tmp_path, cfg, dtype, **kw):
    return folder_pair.Pair(ctx, tmp_path, S, O.ZiruraxOracle, cfg, dtype, **kw)


def only(**kw):
    return S.config([S.layer(**kw)])


# One mechanism at a time, then together; sizes that the kernels have to pad, values of 1, the shapes that take other routes.
ONE = {
    "plain": only(),
    "no_feed_forward": only(ff=None),
    "everything_one": S.config([S.layer(S.attention(1, 1, 2, 1, 1, S.rot(2, 3.0)), S.ssd(1, 1, 1, 1, 1, 1), ff=1)], width=64, vocab=70),
    "window_one": only(left=S.attention(window=1)),
    "window_two": only(left=S.attention(window=2)),
    "no_window": only(left=S.attention(window=None)),
    "window_past_the_context": only(left=S.attention(window=5000)),
    "no_cap": only(left=S.attention(softcap=None)),
    "tight_cap": only(left=S.attention(softcap=0.7, scale=1.0)),
    "no_rotation": only(left=S.attention(turn=None)),
    "plain_frequencies": only(left=S.attention(turn=S.rot(24, 100.0, None))),
    "many_query_heads": only(left=S.attention(heads=7, kv_heads=1, dim=64, vdim=32)),
    "heads_alone": only(left=S.attention(heads=5, kv_heads=5, dim=48, vdim=80)),
    "dim_128": only(left=S.attention(heads=12, kv_heads=4, dim=128, vdim=128, turn=S.rot(64))),
    "dim_90_vdim_200": only(left=S.attention(heads=2, kv_heads=1, dim=90, vdim=200)),
    "dim_256": only(left=S.attention(heads=2, kv_heads=2, dim=256, vdim=256, turn=S.rot(256))),
    "heads_beyond_matrix_cores": only(left=S.attention(heads=4, kv_heads=2, dim=300, vdim=530, turn=S.rot(200), scale=0.06)),
    "state_128": only(right=S.ssd(heads=4, groups=1, state=128, vdim=64, parts=1)),
    "state_200": only(right=S.ssd(heads=3, groups=3, state=200, vdim=16, parts=3)),
    "state_500": only(right=S.ssd(heads=2, groups=1, state=500, vdim=24, parts=2)),
    "many_parts": only(right=S.ssd(heads=6, groups=2, vdim=20, parts=24)),
    "parts_across_heads": only(right=S.ssd(heads=3, groups=1, vdim=20, parts=4)),
    "conv_1": only(right=S.ssd(conv=1)),
    "conv_2": only(right=S.ssd(conv=2)),
    "conv_8": only(right=S.ssd(conv=8)),
    "odd_width": S.config([S.layer(S.attention(dim=10, vdim=7, turn=S.rot(6)), S.ssd(heads=2, groups=2, state=5, vdim=3, parts=1), ff=7)], width=101, vocab=37),
    "width_2000": S.config([S.layer(ff=96), S.layer(ff=None)], width=2000, vocab=60),
    "width_3000": S.config([S.layer(ff=96), S.layer(ff=32)], width=3000, vocab=60),
    "width_4300": S.config([S.layer(ff=40), S.layer(ff=None)], width=4300, vocab=60),
    "mixed": S.mixed(),
}


@BOTH
@pytest.mark.parametrize("name", list(ONE))
def test_each_mechanism(ctx, tmp_path, name, dtype):
    """The residual stream after every layer, the logits of a prompt, the same tokens one by one and as short portions."""
    print(name, dtype, flush=True)
    with Pair(ctx, tmp_path, ONE[name], dtype) as p:
        toks = p.tokens(37)
        trace, rounded = [], []
        want = p.want(toks, trace)
        p.rounded.reset()
        p.rounded.forward(toks, rounded)
        layers = p.gpu.forward_layers(toks, 0)
        assert len(layers) == len(trace)
        for got, ref, r in zip(layers, trace, rounded):  # (the residual has a tolerance of its own)
            assert error(got, ref) <= (TOL_F32 if dtype == F32 else 3.0 * error(r, ref))
        p.check(p.gpu.forward(toks, 0, np.arange(37)), want)
        p.check(p.portions(toks, [1] * 37), want)
        p.check(p.portions(toks, [3, 4, 16, 1, 13]), want)


@BOTH
def test_portions_of_many_sizes(ctx, tmp_path, dtype):
    """Cuts in the middle and at the edges of windows, tiles and chunks, down to two tokens."""
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=2) as p:
        toks = p.tokens(210, 1)
        want = p.want(toks)
        for cuts in ([210], [2] * 105, [3] * 70, [64, 2, 62, 1, 64, 17], [17, 16, 31, 33, 2, 1, 50, 60], [209, 1], [1, 209], [5, 60, 80, 5, 60], [63, 65, 82],
                     [20, 55, 75, 60]):
            p.check(p.portions(toks, cuts), want)


@BOTH
def test_first_tokens(ctx, tmp_path, dtype):
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=3) as p:
        for n in (1, 2, 3, 4, 5, 17):
            toks = p.tokens(n, n)
            p.check(p.gpu.forward(toks, 0, np.arange(n)), p.want(toks))


@BOTH
def test_a_used_state_does_not_leak_into_the_next_sequence(ctx, tmp_path, dtype):
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=4) as p:
        for short in (p.tokens(9, 7), p.tokens(30, 6)):
            n = len(short)
            fresh = p.gpu.forward(short, 0, np.arange(n))
            steps = p.portions(short, [1] * n)
            p.gpu.forward(p.tokens(200, 8), 0, [])
            assert np.array_equal(p.gpu.forward(short, 0, np.arange(n)), fresh)
            p.portions(p.tokens(80, 9), [1] * 80)
            assert np.array_equal(p.portions(short, [1] * n), steps)
            p.check(fresh, p.want(short))


@BOTH
def test_requests_that_take_turns_against_each_alone(ctx, tmp_path, dtype):
    """Unequal requests in interleaved portions, switched by snapshots, give what each gives alone, bit for bit."""
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=5) as p:
        cuts = {"a": [70, 1, 1, 2, 30], "b": [3, 1, 1, 1, 1], "c": [1, 1, 66, 2, 1]}
        toks = {k: p.tokens(sum(c), 20 + i) for i, (k, c) in enumerate(cuts.items())}
        alone = {k: p.portions(toks[k], c) for k, c in cuts.items()}
        state, pos, got = {}, dict.fromkeys(cuts, 0), {k: [] for k in cuts}
        for i in range(5):
            for k, c in cuts.items():
                if k in state:
                    p.gpu.restore_state(state[k], pos[k])
                got[k].append(p.gpu.forward(toks[k][pos[k]:pos[k] + c[i]], pos[k], np.arange(c[i])))
                pos[k] += c[i]
                state[k] = p.gpu.snapshot_state(pos[k])
        for k in cuts:
            assert np.array_equal(np.concatenate(got[k]), alone[k])
            p.check(alone[k], p.want(toks[k]))


def last(p, toks):
    p.oracle.reset()
    return p.oracle.forward(toks)[-1]


@BOTH
@pytest.mark.parametrize("shape", [dict(window=60), dict(window=64), dict(window=129), dict(heads=6, kv_heads=1, dim=70, vdim=66, window=100)],
                         ids=["60", "64", "129", "100_one_kv_head"])
def test_the_edges_of_a_window(ctx, tmp_path, dtype, shape):
    """One key that takes the attention of a query: just inside the window it shows, one further out it does not; in prompts, portions and
    steps, at the borders of the 64-position tiles, and nothing that lies ahead is seen."""
    cfg = S.config([S.layer(S.attention(turn=S.rot(2, 1e6, None), scale=2.0, softcap=40.0, **shape), ff=None)], vocab=64, scale=0.3)
    t = S.tensors(cfg, 6)
    t["l0.mix.right.out"] = t["l0.mix.right.out"] * 0  # the attention alone
    w = shape["window"]
    with Pair(ctx, tmp_path, cfg, dtype, seed=6, t=t) as p:
        n, query, best = 203, 5, (0.0, 0, 0)
        for filler in range(8, 16):  # the filler and the key that differ most for the query
            toks = np.full(n, filler)
            toks[-1] = query
            ref = last(p, toks)
            for key in (18, 24, 30, 36):
                toks[-10] = key
                best = max(best, (error(last(p, toks), ref), filler, key))
                toks[-10] = filler
        assert best[0] > 0.3, "the key does not stand out"
        filler, key = best[1:]
        plain = np.full(n, filler)
        plain[-1] = query
        ref = last(p, plain)
        inside = n - w
        for at in (inside - 2, inside - 1, inside, inside + 1, 127, 128, 191, 192, 201):
            toks = plain.copy()
            toks[at] = key
            want = p.want(toks)
            shows = error(want[-1], ref)
            assert shows > max(0.15, 5 * p.tol) if at >= inside else shows < 1e-9
            p.check(p.gpu.forward(toks, 0, [n - 1]), want[-1])                      # in a prompt
            p.gpu.forward(toks[:-1], 0, [])
            p.check(p.gpu.forward(toks[-1:], n - 1), want[-1])                      # decoded
            p.gpu.forward(toks[:-5], 0, [])
            p.check(p.gpu.forward(toks[-5:], n - 5, [4]), want[-1])                 # in a short portion
            p.gpu.forward(toks[:100], 0, [])
            p.check(p.gpu.forward(toks[100:], 100, [n - 101]), want[-1])            # in a portion that starts inside a tile
        toks = np.full(n, filler)
        toks[64], toks[65] = query, key
        want = p.want(toks)
        p.check(p.gpu.forward(toks, 0, [63, 64, 65]), want[63:66])
        # the key passes out of the window while tokens are decoded
        toks = np.full(n, query)
        toks[90] = key
        want = p.want(toks)
        p.check(p.portions(toks, [91] + [1] * (n - 91)), want)


@BOTH
def test_a_state_that_remembers(ctx, tmp_path, dtype):
    """Slow decays: the first tokens of a sequence still show hundreds of tokens later, in prompts, portions and steps."""
    cfg = S.config([S.layer(right=S.ssd(heads=4, groups=2, state=40, vdim=24, conv=3, parts=2), ff=None)])
    t = S.tensors(cfg, 8)
    filler, n, p0 = 3, 300, "l0.mix.right."
    t["l0.mix.left.out"] = t["l0.mix.left.out"] * 0
    t[p0 + "A_log"] = np.full_like(t[p0 + "A_log"], -3.0)
    # the first tokens take large steps, the filler a small one: it adds next to nothing to the state
    first = np.array([7, 9, 11, 13, 15, 17])
    h = O.rms(t["embed"].astype(np.float64) * cfg["embedding"]["scale"], cfg["norm"]["eps"]) * t["l0.norm1"]
    w = h[first].sum(0) - h[filler] * (h[first].sum(0) @ h[filler]) / (h[filler] @ h[filler])
    t[p0 + "in"][-4:] = from_bf16(to_bf16(9.0 * w / (h[first] @ w).mean()))
    t[p0 + "dt_bias"] = np.full_like(t[p0 + "dt_bias"], -7.0)
    with Pair(ctx, tmp_path, cfg, dtype, seed=8, t=t) as p:
        toks = np.full(n, filler)
        toks[:6] = first
        want = p.want(toks)
        other = toks.copy()
        other[:6] = first[::-1]
        assert error(last(p, other), want[-1]) > 5 * p.tol
        p.check(p.gpu.forward(toks, 0, [n - 1]), want[-1])
        p.check(p.portions(toks, [31, 33, 2, 1, 1, 32, 100, 90, 10])[-1], want[-1])
        p.check(p.portions(toks, [250] + [1] * 50)[200:], want[200:])


@BOTH
def test_long_decoding(ctx, tmp_path, dtype):
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=9, context=400) as p:
        toks = p.tokens(390, 4)
        want = p.want(toks)
        p.check(p.portions(toks, [30] + [1] * 360), want)


@BOTH
def test_the_ring_of_keys_and_values_goes_round(ctx, tmp_path, dtype):
    """More positions than the ring holds: slots that are used again, in prompt passes, portions and steps, and a snapshot behind it."""
    full = 512 if dtype == F32 else 2048  # tokens of a pass
    cfg = S.config([S.layer(S.attention(heads=2, kv_heads=1, dim=16, vdim=16, window=70), S.ssd(heads=2, groups=1, state=8, vdim=8), ff=None)], width=64, vocab=60)
    n = 2 * full + 150
    with Pair(ctx, tmp_path, cfg, dtype, seed=16, context=n + 8) as p:
        toks = p.tokens(n, 3)
        want = p.want(toks)
        places = np.unique(np.r_[np.arange(0, n, 97), full - 1:full + 3, n - 80:n])
        p.check(p.gpu.forward(toks, 0, places), want[places])
        state = p.gpu.snapshot_state(n)
        step = p.gpu.forward([3], n)
        p.gpu.forward(toks[:200], 0, [])
        p.gpu.restore_state(state, n)
        assert np.array_equal(p.gpu.forward([3], n), step)
        got = p.portions(toks, [full - 30, 100, 2, 41, 1, 1, full - 65] + [1] * 70 + [3, 27])
        p.check(got[places], want[places])


@BOTH
def test_one_key_thousands_of_positions_back(ctx, tmp_path, dtype):
    """Without a window: more tiles than a step has workgroups along the sequence, a key that stands out in the first and in the last of
    them, and between; in a step and in prompt passes."""
    cfg = S.config([S.layer(S.attention(heads=2, kv_heads=1, dim=16, vdim=16, window=None, turn=S.rot(2, 1e7, None), scale=3.0, softcap=60.0),
                            S.ssd(heads=1, groups=1, state=4, vdim=4), ff=None)], width=64, vocab=64, scale=0.3)
    t = S.tensors(cfg, 17)
    t["l0.mix.right.out"] = t["l0.mix.right.out"] * 0
    x, eps = t["embed"].astype(np.float64) * 0.3, cfg["norm"]["eps"]
    h = O.rms(x, eps) * t["l0.norm1"]
    q, k = (h @ t["l0.mix.left.q"].T).reshape(64, 2, 16), h @ t["l0.mix.left.k"].T
    score = 60.0 * np.tanh(3.0 * np.einsum("qhd,kd->qhk", q, k) / 60.0)
    gap = (score.max(-1) - np.median(score, -1)).min(-1)  # a query with a key far above most others, for both heads
    query = int(np.argmax(gap))
    key, filler = int(np.argmax(score[query].min(0))), int(np.argmin(score[query].max(0)))
    n = 4200
    with Pair(ctx, tmp_path, cfg, dtype, seed=17, context=n + 4, t=t) as p:
        plain = np.full(n, filler)
        plain[-1] = query
        ref = last(p, plain)
        for at in (0, 63, 64, 2050, 4095, 4096, 4160):
            toks = plain.copy()
            toks[at] = key
            want = last(p, toks)
            p.tol = TOL_F32 if dtype == F32 else 0.03  # (about ten roundings of a bfloat16 activation)
            assert error(want, ref) > max(0.15, 5 * p.tol)
            p.gpu.forward(toks[:-1], 0, [])
            p.check(p.gpu.forward(toks[-1:], n - 1), want)
            if at in (64, 4096):
                p.check(p.gpu.forward(toks, 0, [n - 1]), want)
                p.gpu.forward(toks[:-9], 0, [])
                p.check(p.gpu.forward(toks[-9:], n - 9, [8]), want)


def test_many_wanted_places(ctx, tmp_path):
    """More wanted rows than one product with the head takes, in a step each and in one pass."""
    with Pair(ctx, tmp_path, S.mixed(), NATIVE, seed=10) as p:
        toks = p.tokens(200, 5)
        want = p.want(toks)
        p.check(p.gpu.forward(toks, 0, np.arange(200)), want)
        for places in ([199], [0, 1, 2, 199], [3, 70, 71, 100, 150]):
            p.check(p.gpu.forward(toks, 0, places), want[places])


def test_large_products_and_several_passes(ctx, tmp_path):
    """Shapes that fill the chip (the 128 x 128 tiles) over more tokens than one pass takes, against the f32 model."""
    cfg = S.config([S.layer(S.attention(heads=8, kv_heads=2, dim=64, vdim=64, window=700, turn=S.rot(64), scale=0.125), S.ssd(heads=16, groups=1, state=128, vdim=64, parts=1),
                            ff=1500)] * 2, width=512, vocab=500)
    t = S.tensors(cfg, 11)
    path = S.write(tmp_path / "m", cfg, t)
    toks = np.random.default_rng(6).integers(0, 500, 2150)
    o, rounded = O.ZiruraxOracle(cfg, t), O.ZiruraxOracle(cfg, t, r=O.bfloat16)
    first = o.forward(toks[:150])
    tol = 3.0 * error(rounded.forward(toks[:150]), first)
    places = [0, 511, 512, 1024, 2047, 2048, 2049, 2149]
    with RocmModel(ctx, path, 2200, F32) as exact, RocmModel(ctx, path, 2200, NATIVE) as served:
        want = exact.forward(toks, 0, places)
        assert error(served.forward(toks, 0, places), want) <= tol
        state = served.snapshot_state(2150)
        step, exact_step = served.forward([3], 2150), exact.forward([3], 2150)
        assert error(step, exact_step) <= tol
        served.forward(toks[:300], 0, [])
        served.restore_state(state, 2150)
        assert np.array_equal(served.forward([3], 2150), step)
        assert error(exact.forward(toks[:150], 0, [149]), first[-1]) <= TOL_F32


@BOTH
def test_graph_replay_is_the_same_launches(ctx, tmp_path, dtype):
    """Replays with eager prompt passes and synchronisations between them, against the launches enqueued one by one."""
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=12) as p:
        toks = p.tokens(60, 3)
        cuts = [10] + [1] * 12 + [27] + [1] * 11
        p.gpu.set_graph_replay(False)
        eager = p.portions(toks, cuts)
        p.gpu.set_graph_replay(True)
        for _ in range(3):
            assert np.array_equal(p.portions(toks, cuts), eager)
            ctx.sync()


def test_greedy_generation(ctx, tmp_path):
    """The generation loop over the handle: chunked prompt, picks on the device, stop tokens, a sampler in their place."""
    with Pair(ctx, tmp_path, S.mixed(), F32, seed=13) as p:
        prompt = [int(t) for t in p.tokens(25, 2)]
        want = greedy(p, prompt, 70)
        for ubatch in (0, 1, 2, 7):
            assert M.generate(p.gpu, prompt, 70, ubatch=ubatch) == want
        assert M.generate(p.gpu, prompt, 70, sample=M.greedy_pick) == want
        stop = want[10]
        assert M.generate(p.gpu, prompt, 70, stop=[stop]) == want[:want.index(stop) + 1]
        assert len(M.generate(p.gpu, prompt, 1000)) == p.gpu.max_seq_len - len(prompt) + 1


@pytest.mark.parametrize("dtype, kind", [("float32", F32), ("bfloat16", NATIVE)])
def test_trace_replay(ctx, tmp_path, dtype, kind):
    with Pair(ctx, tmp_path, S.mixed(), kind, seed=14) as p:
        a, b = [int(t) for t in p.tokens(30, 1)], [int(t) for t in p.tokens(12, 2)]
        steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [19, 0]}], "end": []},
                 {"step": 1, "entries": [{"id": "b", "tokens": b[:7], "want": []}], "end": []},
                 {"step": 2, "entries": [{"id": "a", "tokens": a[20:], "want": [0, 9]}], "end": ["a"]},
                 {"step": 3, "entries": [{"id": "b", "tokens": b[7:8], "want": [0]}, {"id": "c", "tokens": a[:3], "want": [2]}], "end": ["c"]},
                 {"step": 4, "entries": [{"id": "b", "tokens": b[8:], "want": [3]}], "end": ["b"]}]
        out = tmp_path / "out"
        out.mkdir()
        assert run_trace(p.path, dtype, steps, out, 64) == [f"done {i}" for i in range(5)]
        wa, wb = p.want(a), p.want(b)
        want = {0: wa[[19, 0]], 2: wa[[20, 29]], 3: np.stack([wb[7], wa[2]]), 4: wb[[11]]}
        for i, w in want.items():
            p.check(np.fromfile(out / f"{i}.f32", "<f4").reshape(w.shape), w)


def test_command_line(ctx, tmp_path):
    with Pair(ctx, tmp_path, S.mixed(), F32, seed=13) as p:
        prompt = [int(t) for t in p.tokens(25, 2)]
        want = greedy(p, prompt, 12)
        proc = subprocess.run([sys.executable, "-m", "wick_amd", "generate", "--model", p.path, "--dtype", "float32", "--tokens", ",".join(map(str, prompt)),
                               "--max-new", "12"], cwd=ROOT, capture_output=True, text=True, timeout=100)
        assert proc.returncode == 0, proc.stderr[-2000:]
        assert [int(t) for t in proc.stdout.split()] == want


def test_what_does_not_fit_is_an_error(ctx, tmp_path):
    cfg = S.mixed()
    t = S.tensors(cfg, 1)
    with RocmModel(ctx, S.write(tmp_path / "ok", cfg, t), 16) as m:
        for toks, pos in (([cfg["vocab"]], 0), ([1], 16), ([1] * 17, 0), ([1, 2, 3], 14)):
            with pytest.raises(RocmError):
                m.forward(toks, pos)
        with pytest.raises(RocmError):
            m.restore_state(np.zeros(8, np.uint8), 3)

    def bad(change_cfg=None, change_t=None):
        c, tt = copy.deepcopy(cfg), dict(t)
        if change_cfg:
            change_cfg(c)
        if change_t:
            change_t(tt)
        with pytest.raises(RocmError):
            RocmModel(ctx, S.write(tmp_path / "bad", c, tt), 16).free()

    left, right = lambda c: c["layers"][0]["mixer"]["left"], lambda c: c["layers"][0]["mixer"]["right"]
    bad(lambda c: c.pop("embedding"))
    bad(lambda c: c["layers"][0].update(type="serial"))
    bad(lambda c: c["layers"][0]["mixer"].pop("right"))
    bad(lambda c: c["layers"][0]["mlp"].update(kind="moe"))
    bad(lambda c: left(c).update(kv_heads=3))
    bad(lambda c: left(c)["rot"].update(dims=26))
    bad(lambda c: left(c)["rot"]["scaling"].pop("low"))
    bad(lambda c: left(c)["mask"].update(size=0))
    bad(lambda c: right(c).update(groups=3))
    bad(lambda c: right(c).update(norm_groups=7))
    bad(lambda c: right(c).update(state=600))
    bad(lambda c: right(c).update(conv=5))
    bad(None, lambda tt: tt.pop("l1.mix.right.conv.b"))
    bad(None, lambda tt: tt.update({"l0.norm1": tt["l0.norm1"][:-1]}))
