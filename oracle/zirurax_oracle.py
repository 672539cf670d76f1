"""Plain, slow numpy implementation of the Zirurax design: what the GPU model is compared with (test infrastructure only).

One function per mechanism, each over a whole sequence [T, ...] with an explicit state for what came before it, everything in
float64 unless a test asks for another type.  No code is shared with the product path.

A model is a config dictionary (the keys of config.json) and a dictionary of tensors by name.  `r` arguments: how a matrix product's
activations are rounded (see lokinex_oracle)."""
from __future__ import annotations

import numpy as np

from .lokinex_oracle import bfloat16, causal_conv, exact, gelu_tanh, rms, sigmoid, silu, softplus

__all__ = ["ZiruraxOracle", "bfloat16", "exact", "frequencies", "rope_partial", "windowed_attention", "ssd", "parallel_mixer", "dense_mlp"]


def frequencies(rot):
    """Angle per position of pair i: base^(-2i / dims), long wavelengths stretched by `factor` with a ramp in between."""
    f = rot["base"] ** (-2.0 * np.arange(rot["dims"] // 2) / rot["dims"])
    sc = rot.get("scaling")
    if not sc:
        return f
    out = []
    for v in f:
        waves = sc["original"] * v / (2.0 * np.pi)  # periods that fit the original length
        if waves > sc["high"]:
            out.append(v)
        elif waves < sc["low"]:
            out.append(v / sc["factor"])
        else:
            s = (waves - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1.0 - s) * v / sc["factor"] + s * v)
    return np.array(out)


def rope_partial(v, pos, rot):
    """Turns the pairs (2i, 2i + 1) of the first rot.dims coordinates of v [T, heads, dim]; the others pass."""
    if not rot:
        return v
    out = v.copy()
    a = pos[:, None, None] * frequencies(rot)
    u, w = v[..., 0:rot["dims"]:2], v[..., 1:rot["dims"]:2]
    out[..., 0:rot["dims"]:2] = u * np.cos(a) - w * np.sin(a)
    out[..., 1:rot["dims"]:2] = w * np.cos(a) + u * np.sin(a)
    return out


def windowed_attention(h, t, p, m, pos, cache, r=exact):
    """Grouped-query attention over the last mask.size positions, capped scores, gated output.  cache: (keys, values) of every position
    before h[0]."""
    n, H, G, dim, vdim = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rope_partial((r(h) @ t[p + "q"].T).reshape(n, H, dim), pos, m.get("rot"))
    k = rope_partial((r(h) @ t[p + "k"].T).reshape(n, G, dim), pos, m.get("rot"))
    v = (r(h) @ t[p + "v"].T).reshape(n, G, vdim)
    gate = sigmoid(r(h) @ t[p + "g"].T)
    k, v = np.concatenate([cache[0], r(k)]), np.concatenate([cache[1], r(v)])
    q = r(q)
    window = (m.get("mask") or {}).get("size")
    cap = m.get("softcap")
    out = np.empty((n, H, vdim), h.dtype)
    for i in range(n):
        at = int(pos[i])
        first = 0 if window is None else max(0, at - window + 1)
        for x in range(H):
            g = x // (H // G)
            s = (k[first:at + 1, g] @ q[i, x]) * m["scale"]
            if cap:
                s = cap * np.tanh(s / cap)
            e = np.exp(s - s.max())
            out[i, x] = (e / e.sum()) @ v[first:at + 1, g]
    return r(out.reshape(n, H * vdim) * gate) @ t[p + "o"].T, (k, v)


def ssd(h, t, p, m, eps, state, r=exact):
    """State-space duality block.  state: (S [heads, N, P], past inputs of the convolution [taps - 1, channels])."""
    n, H, G, N, P, parts = len(h), m["heads"], m["groups"], m["state"], m["vdim"], m["norm_groups"]
    inner = H * P
    w = r(h) @ t[p + "in"].T
    z, xbc, dt = w[:, :inner], w[:, inner:2 * inner + 2 * G * N], w[:, 2 * inner + 2 * G * N:]
    u, past = causal_conv(xbc, t[p + "conv"], state[1])
    u = r(silu(u + t[p + "conv.b"]))
    x, B, C = u[:, :inner].reshape(n, H, P), u[:, inner:inner + G * N].reshape(n, G, N), u[:, inner + G * N:].reshape(n, G, N)
    dt = softplus(dt + t[p + "dt_bias"])
    rate = -np.exp(t[p + "A_log"])
    S, y = state[0], np.empty((n, H, P), h.dtype)
    for i in range(n):
        b, c = np.repeat(B[i], H // G, axis=0), np.repeat(C[i], H // G, axis=0)  # a head's group
        S = np.exp(rate * dt[i])[:, None, None] * S + dt[i][:, None, None] * b[:, :, None] * x[i][:, None, :]
        y[i] = np.einsum("hn,hnp->hp", c, S) + t[p + "D"][:, None] * x[i]
    y = (y.reshape(n, inner) * silu(z)).reshape(n, parts, inner // parts)
    y = rms(y, eps).reshape(n, inner) * t[p + "norm"]
    return r(y) @ t[p + "o"].T, (S, past)


def parallel_mixer(h, t, p, m, eps, pos, state, r=exact):
    """Half the sum of the two mixers' outputs, each normed over the width.  state: (attention's, recurrence's)."""
    a, sa = windowed_attention(h, t, p + "left.", m["left"], pos, state[0], r)
    b, sb = ssd(h, t, p + "right.", m["right"], eps, state[1], r)
    return 0.5 * (rms(a, eps) * t[p + "left.out"] + rms(b, eps) * t[p + "right.out"]), (sa, sb)


def dense_mlp(h, t, p, r=exact):
    return r(gelu_tanh(r(h) @ t[p + "gate"].T) * (r(h) @ t[p + "up"].T)) @ t[p + "down"].T


class ZiruraxOracle:
    """The whole model over one sequence; `forward` continues from where the previous call stopped."""

    def __init__(self, cfg, tensors, dtype=np.float64, r=exact):
        self.cfg, self.dtype, self.r = cfg, dtype, r
        self.t = {k: np.asarray(v, dtype) for k, v in tensors.items()}
        self.reset()

    def reset(self):
        self.pos, self.states = 0, [self._fresh(l["mixer"]) for l in self.cfg["layers"]]

    def _fresh(self, m):
        a, b, z = m["left"], m["right"], lambda *s: np.zeros(s, self.dtype)
        channels = b["heads"] * b["vdim"] + 2 * b["groups"] * b["state"]
        return (z(0, a["kv_heads"], a["dim"]), z(0, a["kv_heads"], a["vdim"])), (z(b["heads"], b["state"], b["vdim"]), z(b["conv"] - 1, channels))

    def forward(self, tokens, trace=None):
        """Logits [T, vocab]; trace (a list) receives the residual stream after every layer."""
        t, r, eps = self.t, self.r, self.cfg["norm"]["eps"]
        x = t["embed"][np.asarray(tokens)] * self.cfg["embedding"]["scale"]
        pos = (self.pos + np.arange(len(x))).astype(self.dtype)
        for i, layer in enumerate(self.cfg["layers"]):
            p = f"l{i}."
            h = rms(x, eps) * t[p + "norm1"]
            y, self.states[i] = parallel_mixer(h, t, p + "mix.", layer["mixer"], eps, pos, self.states[i], r)
            if layer["mlp"]:
                y = y + dense_mlp(h, t, p + "mlp.", r)
            x = x + y
            if trace is not None:
                trace.append(x.copy())
        self.pos += len(x)
        return r(rms(x, eps) * t["final.norm"]) @ t["embed"].T
