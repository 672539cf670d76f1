"""Small seeded Zirurax models for the tests (not collected by pytest): a configuration, its tensors (bfloat16-exact floats) and the folder
they are loaded from."""
import numpy as np

from lokinex_synth import write  # noqa: F401  (the same folders)
from wick_amd.checkpoint import from_bf16, to_bf16

SCALING = {"factor": 6.0, "low": 1.5, "high": 3.0, "original": 300}


def rot(dims=16, base=20000.0, scaling=SCALING):
    return {"base": base, "dims": dims, **({"scaling": scaling} if scaling else {})}


def attention(heads=4, kv_heads=2, dim=24, vdim=40, window=20, turn=rot(), scale=0.23, softcap=9.0):
    a = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        a["mask"] = {"size": window}
    if turn:
        a["rot"] = turn
    if softcap:
        a["softcap"] = softcap
    return a


def ssd(heads=4, groups=2, state=24, vdim=20, conv=4, parts=2):
    return {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv, "norm_groups": parts}


def layer(left=None, right=None, ff=144):
    return {"type": "parallel", "mixer": {"left": left or attention(), "right": right or ssd()}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, width=136, vocab=150, eps=1e-5, scale=3.0):
    return {"architecture": "Zirurax", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


def tensors(cfg, seed=1):
    rng = np.random.default_rng(seed)
    D, V = cfg["width"], cfg["vocab"]
    t = {}

    def put(name, shape, sigma, center=0.0):
        t[name] = from_bf16(to_bf16(center + sigma * rng.standard_normal(shape))).reshape(shape)

    def mat(name, m, k, gain=1.0):
        put(name, (m, k), gain / np.sqrt(k))

    put("embed", (V, D), 0.4)
    put("final.norm", (D,), 0.3, 1.0)
    for i, l in enumerate(cfg["layers"]):
        p, a, s = f"l{i}.", l["mixer"]["left"], l["mixer"]["right"]
        x, y = p + "mix.left.", p + "mix.right."
        put(p + "norm1", (D,), 0.3, 1.0)
        H, G = a["heads"], a["kv_heads"]
        mat(x + "q", H * a["dim"], D, 1.5)
        mat(x + "k", G * a["dim"], D, 1.5)
        mat(x + "v", G * a["vdim"], D)
        mat(x + "g", H * a["vdim"], D)
        mat(x + "o", D, H * a["vdim"])
        put(x + "out", (D,), 0.3, 1.0)
        h, inner, bc = s["heads"], s["heads"] * s["vdim"], 2 * s["groups"] * s["state"]
        mat(y + "in", 2 * inner + bc + h, D)
        put(y + "conv", (inner + bc, s["conv"]), 0.5)
        put(y + "conv.b", (inner + bc,), 0.3)
        put(y + "dt_bias", (h,), 1.0, -2.0)
        put(y + "A_log", (h,), 1.0, 0.0)
        put(y + "D", (h,), 0.5, 0.5)
        put(y + "norm", (inner,), 0.3, 1.0)
        mat(y + "o", D, inner)
        put(y + "out", (D,), 0.3, 1.0)
        if l["mlp"]:
            f, ff = p + "mlp.", l["mlp"]["ff"]
            mat(f + "gate", ff, D)
            mat(f + "up", ff, D)
            mat(f + "down", D, ff)
    return t


# Layers that differ in everything, at sizes that are no multiples of anything convenient.
def mixed(**kw):
    return config([layer(), layer(attention(heads=6, kv_heads=1, dim=70, vdim=66, window=75, turn=rot(26, 500.0, None), scale=0.11, softcap=30.0),
                                  ssd(heads=6, groups=3, state=40, vdim=33, conv=2, parts=3), ff=None),
                   layer(attention(heads=3, kv_heads=3, dim=30, vdim=18, window=130, turn=rot(30, 1e6)), ssd(heads=2, groups=1, state=9, vdim=48, conv=3, parts=4), ff=70)], **kw)
