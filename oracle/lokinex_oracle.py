"""Plain, slow numpy implementation of the Lokinex design: what the GPU model is compared with (test infrastructure
only).

One function per mechanism, each over a whole sequence [T, ...] with an explicit state for what came before it, everything in
float64 unless a test asks for another type.  No code is shared with the product path.

A model is a config dictionary (the keys of config.json) and a dictionary of tensors by name.

`r` arguments: how a matrix product's activations are rounded.  Exact by default; bfloat16 gives what the products' rounding alone
does to a result, which is what a bfloat16 model is measured against."""
from __future__ import annotations

import numpy as np


def exact(x):
    return x


def bfloat16(x):
    """Round to nearest even at 8 significant bits."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    u = (u + np.uint32(0x7FFF) + ((u >> np.uint32(16)) & np.uint32(1))) & np.uint32(0xFFFF0000)
    return u.view(np.float32).astype(x.dtype).reshape(x.shape)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.logaddexp(0.0, z)


def rms(x, eps):
    """x over its root mean square, along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def causal_conv(h, w, past):
    """Depthwise causal convolution over time: out[t] = sum_j w[:, j] * in[t - taps + 1 + j].  past: [taps - 1, C], the inputs
    before h[0] (zeros at a sequence's start).  Returns (out, the new past)."""
    taps, n = w.shape[1], h.shape[0]
    seq = np.concatenate([past, h], axis=0)
    out = np.zeros_like(h)
    for j in range(taps):
        out += w[:, j] * seq[j:j + n]
    return out, seq[len(seq) - (taps - 1):]


def input_conv(h, w, past):
    """What a mixer reads: the normed input plus its causal convolution."""
    c, past = causal_conv(h, w, past)
    return h + c, past


def rope_interleaved(v, pos, base):
    """Rotates the pairs (2i, 2i + 1) of the last axis of v [T, ..., dims] by pos[t] * base^(-2i / dims)."""
    dims = v.shape[-1]
    f = base ** (-2.0 * np.arange(dims // 2) / dims)
    a = pos.reshape((-1,) + (1,) * (v.ndim - 1)) * f
    c, s = np.cos(a), np.sin(a)
    out = np.empty_like(v)
    u, w = v[..., 0::2], v[..., 1::2]
    out[..., 0::2], out[..., 1::2] = u * c - w * s, w * c + u * s
    return out


def latent_attention(h, t, p, m, eps, pos, cache, r=exact):
    """Multi-head attention over a cached latent.  cache: (latents [P, rank], rotated key parts [P, rot]) of the positions before
    h[0].  Keys and values are expanded per head."""
    H, dim, rot, vdim, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    n = h.shape[0]
    q = (r(h) @ t[p + "q"].T).reshape(n, H, dim + rot)
    d = r(h) @ t[p + "dkv"].T
    c = r(rms(d[:, :rank], eps) * t[p + "dkv.norm"])
    qr = r(rope_interleaved(q[..., dim:], pos, m["rot"]["base"]))
    kr = r(rope_interleaved(d[:, rank:], pos, m["rot"]["base"]))
    c, kr = np.concatenate([cache[0], c]), np.concatenate([cache[1], kr])
    k = r(c @ t[p + "uk"].T).reshape(-1, H, dim)
    v = r(c @ t[p + "uv"].T).reshape(-1, H, vdim)
    q = r(q)
    out = np.empty((n, H, vdim), h.dtype)
    for i in range(n):
        see = int(pos[i]) + 1
        s = (np.einsum("hd,khd->hk", q[i, :, :dim], k[:see]) + qr[i] @ kr[:see].T) * m["scale"]
        e = np.exp(s - s.max(axis=-1, keepdims=True))
        out[i] = np.einsum("hk,khv->hv", e / e.sum(axis=-1, keepdims=True), v[:see])
    return r(out.reshape(n, H * vdim)) @ t[p + "o"].T, (c, kr)


def rglru(h, t, p, m, state, r=exact):
    """Recurrent block with a real-gated linear recurrent unit.  state: (S [W], past inputs of the convolution [taps - 1, W])."""
    W, blocks = m["width"], m["blocks"]
    bs = W // blocks
    y = gelu_tanh(r(h) @ t[p + "y"].T + t[p + "y.b"])
    u, past = causal_conv(r(h) @ t[p + "x"].T + t[p + "x.b"], t[p + "conv"], state[1])
    u = u + t[p + "conv.b"]
    ub = u.reshape(-1, blocks, bs)
    gate = sigmoid(np.einsum("boi,tbi->tbo", t[p + "ra"], ub) + t[p + "ra.b"]).reshape(-1, W)
    i = sigmoid(np.einsum("boi,tbi->tbo", t[p + "ri"], ub) + t[p + "ri.b"]).reshape(-1, W)
    log_a = -8.0 * gate * softplus(t[p + "lam"])
    a, gain = np.exp(log_a), np.sqrt(-np.expm1(2.0 * log_a))
    S, out = state[0], np.empty_like(u)
    for k in range(h.shape[0]):
        S = a[k] * S + gain[k] * i[k] * u[k]
        out[k] = S
    return r(out * y) @ t[p + "o"].T, (S, past)


def dense_mlp(h, t, p, r=exact):
    return r(np.maximum(r(h) @ t[p + "up"].T, 0.0) ** 2) @ t[p + "down"].T


def gated_mlp(h, t, p, r=exact):
    return r(silu(r(h) @ t[p + "gate"].T) * (r(h) @ t[p + "up"].T)) @ t[p + "down"].T


def table_moe(h, t, p, m, tokens, r=exact):
    """Experts chosen by token id through a table, each weighted 1 / top, plus a gated shared expert."""
    top = m["router"]["top"]
    out = np.zeros_like(h)
    for k, tok in enumerate(tokens):
        for e in t[p + "table"][tok]:
            out[k] += gated_mlp(h[k:k + 1], t, f"{p}e{int(e)}.", r)[0] / top
    if m.get("shared"):
        out += sigmoid(h @ t[p + "shared.sg"].T) * gated_mlp(h, t, p + "shared.", r)
    return out


class LokinexOracle:
    """The whole model over one sequence; `forward` continues from where the previous call stopped."""

    def __init__(self, cfg, tensors, dtype=np.float64, r=exact):
        self.cfg, self.dtype, self.r = cfg, dtype, r
        self.t = {k: (v if v.dtype.kind == "i" else np.asarray(v, dtype)) for k, v in tensors.items()}
        n, loop = len(cfg["layers"]), cfg.get("loop")
        if loop:
            a, b, times = loop["start"], loop["stop"], loop["times"]
            self.order = [(i, None) for i in range(a)]
            for k in range(times):
                self.order += [(i, k if i == a else None) for i in range(a, b)]
            self.order += [(i, None) for i in range(b, n)]
        else:
            self.order = [(i, None) for i in range(n)]
        self.reset()

    def reset(self):
        self.pos, self.states = 0, [None] * len(self.order)

    def _fresh(self, layer):
        m, z = layer["mixer"], lambda *s: np.zeros(s, self.dtype)
        canon = z(self.cfg["canon"]["taps"] - 1, self.cfg["width"])
        if layer["type"] == "rglru":
            return canon, (z(m["width"]), z(m["conv"] - 1, m["width"]))
        return canon, (z(0, m["kv_rank"]), z(0, m["rot_dim"]))

    def forward(self, tokens, trace=None):
        """Logits [T, vocab]; trace (a list) receives the residual stream after every layer run."""
        t, r, eps = self.t, self.r, self.cfg["norm"]["eps"]
        tokens = np.asarray(tokens)
        x0 = t["embed"][tokens]
        x, pos = x0.copy(), (self.pos + np.arange(len(tokens))).astype(self.dtype)
        for run, (i, step) in enumerate(self.order):
            layer, p = self.cfg["layers"][i], f"l{i}."
            if step is not None:
                x = np.concatenate([x, x0], axis=-1) @ t["loop.in"].T + t["loop.step"][step]
            canon, state = self.states[run] or self._fresh(layer)
            h, canon = input_conv(rms(x, eps) * t[p + "norm1"], t[p + "canon1"], canon)
            if layer["type"] == "rglru":
                y, state = rglru(h, t, p + "mix.", layer["mixer"], state, r)
            else:
                y, state = latent_attention(h, t, p + "mix.", layer["mixer"], eps, pos, state, r)
            self.states[run] = (canon, state)
            x = x + rms(y, eps) * t[p + "norm1b"]
            if layer["mlp"]:
                h = rms(x, eps) * t[p + "norm2"]
                if layer["mlp"]["kind"] == "dense":
                    y = dense_mlp(h, t, p + "mlp.", r)
                else:
                    y = table_moe(h, t, p + "mlp.", layer["mlp"], tokens, r)
                x = x + rms(y, eps) * t[p + "norm2b"]
            if trace is not None:
                trace.append(x.copy())
        self.pos += len(tokens)
        return r(rms(x, eps) * t["final.norm"]) @ t["head"].T
