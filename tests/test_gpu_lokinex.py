"""Lokinex on the GPU, through the model handle, against the plain implementation (oracle/lokinex_oracle.py).

The f32 model is held to f32 rounding, which shows a wrong key, a lost state or a tap that is off by one anywhere; the served
(bfloat16) model to three times what rounding the products' activations does to the plain implementation on the same tokens.  Where random weights would hide a fault -- one far key among hundreds -- the
weights are made so that the fault would move the logits by far more than the tolerance, and the test says so first."""
import subprocess
import sys

import numpy as np
import pytest

import folder_pair
import lokinex_synth as S
from conftest import ROOT
from folder_pair import TOL_F32, error, greedy, run_trace
from oracle import lokinex_oracle as O
from wick_amd import model as M
from wick_amd.checkpoint import from_bf16, to_bf16
from wick_amd.model import F32, NATIVE, RocmModel
from wick_amd.rocm import RocmError

pytestmark = pytest.mark.gpu

BOTH = pytest.mark.parametrize("dtype", [F32, NATIVE], ids=["f32", "bf16"])


def Pair(ctx, tmp_path, cfg, dtype, **kw):
    return folder_pair.Pair(ctx, tmp_path, S, O.LokinexOracle, cfg, dtype, **kw)


# One mechanism at a time, then together; sizes that the kernels have to pad, values of 1, the shapes that take other routes.
ONE = {
    "recurrent": S.config([S.layer(S.rglru())]),
    "recurrent_one_block": S.config([S.layer(S.rglru(width=70, blocks=1, conv=1))], taps=1),
    "recurrent_wide_blocks": S.config([S.layer(S.rglru(width=600, blocks=2, conv=3))], width=200, taps=2),
    "latent": S.config([S.layer(S.latent())]),
    "latent_one_head": S.config([S.layer(S.latent(heads=1, dim=1, rot=2, vdim=1, rank=1, base=3.0))], taps=2),
    "latent_many_heads": S.config([S.layer(S.latent(heads=19, dim=32, rot=32, vdim=32, rank=96))], width=256),
    "latent_wide": S.config([S.layer(S.latent(heads=2, dim=128, rot=64, vdim=128, rank=544))], width=192),
    "latent_beyond_matrix_cores": S.config([S.layer(S.latent(heads=2, dim=232, rot=40, vdim=150, rank=1056))], width=192),
    "dense": S.config([S.layer(S.rglru(), S.dense(300))]),
    "moe": S.config([S.layer(S.rglru(), S.moe())]),
    "moe_one_expert": S.config([S.layer(S.rglru(), S.moe(ff=64, experts=1, top=1, shared=64))]),
    "moe_no_shared": S.config([S.layer(S.rglru(), S.moe(ff=24, experts=9, top=3, shared=None))]),
    "moe_many": S.config([S.layer(S.latent(), S.moe(ff=16, experts=300, top=4, shared=8))], vocab=400),
    "loop_all": S.config([S.layer(S.rglru(), S.dense())], loop=(0, 1, 3)),
    "loop_once": S.config([S.layer(S.rglru()), S.layer(S.latent())], loop=(1, 2, 1)),
    "long_convolutions": S.config([S.layer(S.rglru(width=48, blocks=2, conv=7), S.dense(32)), S.layer(S.latent())], width=72, taps=6),
    "long_and_wide": S.config([S.layer(S.rglru(width=64, blocks=1, conv=8))], width=1500, taps=6, vocab=60),
    "width_2000": S.config([S.layer(S.rglru(width=64, blocks=1), S.moe(ff=24)), S.layer(S.latent(), S.dense(96))], width=2000, vocab=60),
    "width_3000": S.config([S.layer(S.rglru(width=64, blocks=1), S.moe(ff=24))], width=3000, vocab=60, loop=(0, 1, 2)),
    "width_4200": S.config([S.layer(S.rglru(width=64, blocks=1), S.dense(24))], width=4200, vocab=60, loop=(0, 1, 2)),
    "odd_width": S.config([S.layer(S.rglru(width=33, blocks=3, conv=3), S.dense(7)), S.layer(S.latent(), S.moe(ff=5, shared=3))], width=101, vocab=37, taps=3),
    "mixed": S.mixed(),
    "mixed_loop_to_the_end": S.mixed(loop=(2, 4, 2)),
}


@BOTH
@pytest.mark.parametrize("name", list(ONE))
def test_each_mechanism(ctx, tmp_path, name, dtype):
    """The residual stream after every layer run, the logits of a prompt, and the same tokens one by one."""
    print(name, dtype, flush=True)
    with Pair(ctx, tmp_path, ONE[name], dtype) as p:
        toks = p.tokens(37)
        trace = []
        want = p.want(toks, trace)
        layers = p.gpu.forward_layers(toks, 0)
        assert len(layers) == len(trace)
        for got, ref in zip(layers, trace):
            p.check(got, ref)
        p.check(p.gpu.forward(toks, 0, np.arange(37)), want)
        p.check(p.portions(toks, [1] * 37), want)


@BOTH
def test_portions_of_many_sizes(ctx, tmp_path, dtype):
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=2) as p:
        toks = p.tokens(150, 1)
        want = p.want(toks)
        for cuts in ([150], [2] * 75, [3] * 50, [64, 2, 62, 1, 21], [17, 16, 31, 33, 2, 1, 50], [149, 1], [1, 149], [5, 60, 80, 5]):
            p.check(p.portions(toks, cuts), want)


@BOTH
def test_first_tokens(ctx, tmp_path, dtype):
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=3) as p:
        for n in (1, 2, 3, 4, 5):
            toks = p.tokens(n, n)
            p.check(p.gpu.forward(toks, 0, np.arange(n)), p.want(toks))


@BOTH
def test_a_used_state_does_not_leak_into_the_next_sequence(ctx, tmp_path, dtype):
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=4) as p:
        short = p.tokens(9, 7)
        fresh = p.gpu.forward(short, 0, np.arange(9))
        steps = p.portions(short, [1] * 9)
        p.gpu.forward(p.tokens(200, 8), 0, [])
        assert np.array_equal(p.gpu.forward(short, 0, np.arange(9)), fresh)
        p.portions(p.tokens(80, 9), [1] * 80)
        assert np.array_equal(p.portions(short, [1] * 9), steps)
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


def peaked(seed, **shape):
    """A latent layer whose attention falls on one key: large scores, so that a key missed or seen too much moves the output."""
    cfg = S.config([S.layer(S.latent(scale=1.0, **shape))], vocab=64, taps=1)
    t = S.tensors(cfg, seed)
    t["l0.canon1"] = t["l0.canon1"] * 0  # what a position reads is its own token: keys are the tokens'
    return cfg, t


def last(p, toks):
    p.oracle.reset()
    return p.oracle.forward(toks)[-1]


@BOTH
@pytest.mark.parametrize("shape", [dict(), dict(heads=2, dim=70, rot=26, vdim=66, rank=100), dict(heads=5, dim=16, rot=8, vdim=16, rank=24)],
                         ids=["plain", "padded", "small"])
def test_one_far_key(ctx, tmp_path, dtype, shape):
    """A key that stands out, at the first positions and around the borders of the 64-position tiles, asked for from far behind."""
    cfg, t = peaked(6, **shape)
    with Pair(ctx, tmp_path, cfg, dtype, seed=6, t=t) as p:
        n = 203
        # the filler and the key that differ most for the query
        query, best = 5, (0.0, 0, 0)
        for filler in range(8, 16):
            toks = np.full(n, filler)
            toks[-1] = query
            ref = last(p, toks)
            for key in (18, 24, 30, 36):
                toks[70] = key
                best = max(best, (error(last(p, toks), ref), filler, key))
        assert best[0] > 0.3, "the key does not stand out"
        for at in (0, 1, 62, 63, 64, 65, 127, 128, 191, 192, 201):
            toks = np.full(n, best[1])
            toks[at], toks[-1] = best[2], query
            want = p.want(toks)
            assert p.tol < best[0] / 5
            p.check(p.gpu.forward(toks, 0, [n - 1]), want[-1])                      # in a prompt
            p.gpu.forward(toks[:-1], 0, [])
            p.check(p.gpu.forward(toks[-1:], n - 1), want[-1])                      # decoded
            p.gpu.forward(toks[:-5], 0, [])
            p.check(p.gpu.forward(toks[-5:], n - 5, [4]), want[-1])                 # in a short portion
        # and nothing is seen that lies ahead: the query in front of the key
        toks = np.full(n, best[1])
        toks[64], toks[65] = query, best[2]
        want = p.want(toks)
        p.check(p.gpu.forward(toks, 0, [63, 64, 65]), want[63:66])


@BOTH
def test_a_state_that_remembers(ctx, tmp_path, dtype):
    """Slow decays: the first token of a sequence still shows hundreds of tokens later, in prompts, portions and steps."""
    cfg = S.config([S.layer(S.rglru(width=96, blocks=3, conv=4))])
    t = S.tensors(cfg, 8)
    filler, n = 3, 300
    t["l0.mix.lam"] = np.full_like(t["l0.mix.lam"], -9.0)
    # the filler token adds next to nothing to the state: its input is taken out of what W_x sees
    h = O.rms(t["embed"][filler].astype(np.float64), cfg["norm"]["eps"]) * (1.0 + t["l0.canon1"].sum(-1))
    for name in ("x.b", "conv.b"):
        t["l0.mix." + name] = t["l0.mix." + name] * 0
    wx = t["l0.mix.x"].astype(np.float64)
    t["l0.mix.x"] = from_bf16(to_bf16(wx - np.outer(wx @ h, h) / (h @ h))).reshape(wx.shape)
    with Pair(ctx, tmp_path, cfg, dtype, seed=8, t=t) as p:
        toks = np.full(n, filler)
        toks[:6] = [7, 9, 11, 13, 15, 17]
        want = p.want(toks)
        other = toks.copy()
        other[:6] = filler
        p.oracle.reset()
        assert error(p.oracle.forward(other)[-1], want[-1]) > 3 * p.tol
        p.check(p.gpu.forward(toks, 0, [n - 1]), want[-1])
        p.check(p.portions(toks, [31, 33, 2, 1, 1, 32, 100, 90, 10])[-1], want[-1])
        got = p.portions(toks, [250] + [1] * 50)
        p.check(got, want)


@BOTH
def test_long_decoding(ctx, tmp_path, dtype):
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=9, context=400) as p:
        toks = p.tokens(390, 4)
        want = p.want(toks)
        p.check(p.portions(toks, [30] + [1] * 360), want)


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
    cfg = S.config([S.layer(S.rglru(width=768, blocks=4, conv=4), S.moe(ff=192, experts=8, top=2, shared=320)),
                    S.layer(S.latent(heads=12, dim=64, rot=32, vdim=64, rank=192, scale=0.1), S.dense(2048))], width=512, vocab=500, loop=(1, 2, 2))
    t = S.tensors(cfg, 11)
    path = S.write(tmp_path / "m", cfg, t)
    toks = np.random.default_rng(6).integers(0, 500, 2150)
    o, rounded = O.LokinexOracle(cfg, t), O.LokinexOracle(cfg, t, r=O.bfloat16)
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
def test_portions_with_long_convolutions(ctx, tmp_path, dtype):
    with Pair(ctx, tmp_path, ONE["long_convolutions"], dtype, seed=15) as p:
        toks = p.tokens(60, 1)
        want = p.want(toks)
        for cuts in ([60], [3] * 20, [4, 2, 1, 3, 5, 6, 7, 32], [1, 59]):
            p.check(p.portions(toks, cuts), want)


@BOTH
def test_graph_replay_is_the_same_launches(ctx, tmp_path, dtype):
    """Replays with eager prompt passes and synchronisations between them, against the launches enqueued one by one."""
    with Pair(ctx, tmp_path, S.mixed(), dtype, seed=12) as p:
        toks = p.tokens(40, 3)
        p.gpu.set_graph_replay(False)
        eager = p.portions(toks, [10] + [1] * 12 + [7] + [1] * 11)
        p.gpu.set_graph_replay(True)
        for _ in range(3):
            assert np.array_equal(p.portions(toks, [10] + [1] * 12 + [7] + [1] * 11), eager)
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
        assert M.generate(p.gpu, prompt, 1) == want[:1] and M.generate(p.gpu, prompt, 0) == []
        assert len(M.generate(p.gpu, prompt, 1000)) == p.gpu.max_seq_len - len(prompt) + 1


def test_cancel_between_chunks(ctx, tmp_path):
    import ctypes

    with Pair(ctx, tmp_path, S.mixed(), F32, seed=13) as p:
        toks = p.tokens(20, 1)
        flag = ctypes.c_int32(1)
        done, logits = p.gpu.prefill_chunked(toks, 0, 6, flag)
        assert done == 6
        p.check(logits, p.want(toks[:6])[-1])
        done, logits = p.gpu.prefill_chunked(toks[6:], 6, 6)
        assert done == 14
        p.check(logits, p.want(toks)[-1])


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
        assert sorted(f.name for f in out.iterdir()) == sorted(f"{i}.f32" for i in want)
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


def test_gguf_behind_the_same_handle(ctx, oracle):
    """The model that was there before, through the registry: the logits of its own handle."""
    import lfm2_synth as L
    from wick_amd import gguf as G
    from wick_amd.lfm2 import RocmLfm2Model

    img, cfg, _ = L.build(oracle, seed=3)
    toks = np.random.default_rng(1).integers(0, cfg["vocab_size"], 30)
    with G.GgufFile.from_bytes(img) as g:
        own, same = RocmLfm2Model(ctx, g, 64), RocmModel(ctx, g, 64)
    assert same.architecture == "lfm2" and same.layer_runs == cfg["n_layers"]
    own.reset()
    want = [own.forward_prefill(toks[:11], 0), own.forward_prefill(toks[11:], 11)]
    got = same.forward(toks, 0, [10, 29])
    assert np.array_equal(got[0], want[0]) and np.array_equal(got[1], want[1])
    assert np.array_equal(same.generate_greedy(3, 30, 8), own.generate_greedy(3, 30, 8))
    own.free(), same.free()


def test_what_does_not_fit_is_an_error(ctx, tmp_path):
    cfg = S.mixed()
    t = S.tensors(cfg, 1)
    path = S.write(tmp_path / "ok", cfg, t)
    with RocmModel(ctx, path, 16) as m:
        for toks, pos in (([cfg["vocab"]], 0), ([1], 16), ([1] * 17, 0), ([1, 2, 3], 14)):
            with pytest.raises(RocmError):
                m.forward(toks, pos)
        with pytest.raises(RocmError):
            m.forward([1, 2], 0, [2])
        with pytest.raises(RocmError):
            m.restore_state(np.zeros(8, np.uint8), 3)
    import copy

    def bad(change_cfg=None, change_t=None):
        c, tt = copy.deepcopy(cfg), dict(t)
        if change_cfg:
            change_cfg(c)
        if change_t:
            change_t(tt)
        with pytest.raises(RocmError):
            RocmModel(ctx, S.write(tmp_path / "bad", c, tt), 16).free()

    bad(lambda c: c.update(architecture="Other"))
    bad(lambda c: c.pop("canon"))
    bad(lambda c: c["layers"][0].update(type="convolution"))
    bad(lambda c: c["layers"][0]["mixer"].update(blocks=7))
    bad(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=8))
    bad(lambda c: c["layers"][1]["mixer"].update(heads=2))
    bad(lambda c: c["loop"].update(stop=9))
    bad(lambda c: c["loop"].update(times=1.5))
    bad(lambda c: c["layers"][0]["mlp"]["router"].update(experts=5))
    bad(None, lambda tt: tt.pop("l1.mix.uk"))
    bad(None, lambda tt: tt.update({"l0.mlp.table": tt["l0.mlp.table"] + 3}))
    bad(None, lambda tt: tt.update({"l0.norm1": tt["l0.norm1"].reshape(1)}))
