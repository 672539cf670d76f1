"""Small seeded Lokinex models for the tests (not collected by pytest): a configuration, its tensors (bfloat16-exact floats, int32
tables) and the folder they are loaded from."""
import numpy as np

from wick_amd.checkpoint import from_bf16, to_bf16, write_folder


def latent(heads=3, dim=24, rot=16, vdim=40, rank=56, base=10000.0, scale=0.17):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale,
                                                  "rot": {"base": base, "dims": rot}}}


def rglru(width=96, blocks=3, conv=4):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def dense(ff=144):
    return {"kind": "dense", "ff": ff}


def moe(ff=40, experts=6, top=2, shared=72):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp=None):
    return {**mixer, "mlp": mlp}


def config(layers, width=136, vocab=150, taps=4, eps=1e-5, loop=None):
    c = {"architecture": "Lokinex", "vocab": vocab, "width": width, "canon": {"taps": taps}, "norm": {"eps": eps}, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def tensors(cfg, seed=1):
    rng = np.random.default_rng(seed)
    D, V, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    t = {}

    def put(name, shape, sigma, center=0.0):
        t[name] = from_bf16(to_bf16(center + sigma * rng.standard_normal(shape))).reshape(shape)

    def mat(name, m, k, gain=1.0):
        put(name, (m, k), gain / np.sqrt(k))

    put("embed", (V, D), 1.0)
    mat("head", V, D)
    put("final.norm", (), 0.1, 1.0)
    if cfg.get("loop"):
        mat("loop.in", D, 2 * D)
        put("loop.step", (cfg["loop"]["times"], D), 0.3)
    for i, l in enumerate(cfg["layers"]):
        p, x = f"l{i}.", f"l{i}.mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] else ()):
            put(p + n, (), 0.2, 1.0)
        put(p + "canon1", (D, taps), 0.3)
        m = l["mixer"]
        if l["type"] == "rglru":
            W, b = m["width"], m["blocks"]
            for n in ("y", "x"):
                mat(x + n, W, D)
                put(x + n + ".b", (W,), 0.3)
            put(x + "conv", (W, m["conv"]), 0.5)
            put(x + "conv.b", (W,), 0.2)
            for n in ("ra", "ri"):
                put(x + n, (b, W // b, W // b), 1.0 / np.sqrt(W // b))
                put(x + n + ".b", (b, W // b), 0.5)
            put(x + "lam", (W,), 1.5, -4.0)  # decays from fast to a memory of thousands of tokens
            mat(x + "o", D, W)
        else:
            H = m["heads"]
            mat(x + "q", H * (m["dim"] + m["rot_dim"]), D, 2.0)
            mat(x + "dkv", m["kv_rank"] + m["rot_dim"], D, 2.0)
            put(x + "dkv.norm", (m["kv_rank"],), 0.3, 1.0)
            mat(x + "uk", H * m["dim"], m["kv_rank"])
            mat(x + "uv", H * m["vdim"], m["kv_rank"])
            mat(x + "o", D, H * m["vdim"])
        c, f = l["mlp"], p + "mlp."
        if not c:
            continue
        if c["kind"] == "dense":
            mat(f + "up", c["ff"], D)
            mat(f + "down", D, c["ff"])
            continue
        E, top = c["router"]["experts"], c["router"]["top"]
        for name, ff in [(f"e{e}", c["expert"]["ff"]) for e in range(E)] + ([("shared", c["shared"]["ff"])] if c.get("shared") else []):
            mat(f + name + ".gate", ff, D)
            mat(f + name + ".up", ff, D)
            mat(f + name + ".down", D, ff)
        if c.get("shared"):
            mat(f + "shared.sg", 1, D)
        t[f + "table"] = np.stack([rng.permutation(E)[:top] for _ in range(V)]).astype(np.int32)
    return t


def write(path, cfg, t):
    write_folder(str(path), cfg, t)
    return str(path)


# Every mechanism at sizes that are no multiples of anything convenient, and one that takes the matrix-core attention's other shapes.
def mixed(loop=(1, 3, 2)):
    return config([layer(rglru(), moe()), layer(latent(), dense()), layer(rglru(width=60, blocks=5, conv=2), moe(top=1, experts=5, shared=None)),
                   layer(latent(heads=2, dim=70, rot=26, vdim=66, rank=100, base=500.0, scale=0.1))], loop=loop)
