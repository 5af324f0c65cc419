"""Plain, slow restatement of the Lirulix design in float64 numpy: one function per
mechanism, whole sequences only, no cache.  The tests compare the library with it; it
shares no code with the product."""
from __future__ import annotations

import math

import numpy as np

from nukopel_oracle import (bf16, from_bf16_bits, read_model, rms, sigmoid, silu,  # noqa: F401
                            to_bf16_bits, write_model)


def centred_norm(x, w, eps):
    """RMS norm with one gain per channel, stored as its distance from 1."""
    return rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def plain_frequencies(dims, base):
    return np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])


def yarn(dims, base, s):
    """-> (frequencies, factor on cos and sin)."""
    def turn_dim(t):
        return dims * math.log(s["original"] / (2 * math.pi * t)) / (2 * math.log(base))
    lo = max(math.floor(turn_dim(s["fast"])), 0)
    hi = min(math.ceil(turn_dim(s["slow"])), dims - 1)
    f = plain_frequencies(dims, base)
    out = np.empty_like(f)
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out[i] = fi / s["factor"] * ramp + fi * (1.0 - ramp)
    return out, 0.1 * math.log(s["factor"]) + 1.0


def banded(dims, base, s):
    """Long wavelengths slowed down by `factor`, short ones kept, a linear passage
    between the two bands."""
    out = []
    for f in plain_frequencies(dims, base):
        wave = 2 * math.pi / f
        if wave < s["original"] / s["high"]:
            out.append(f)
        elif wave > s["original"] / s["low"]:
            out.append(f / s["factor"])
        else:
            t = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
            out.append((1 - t) * f / s["factor"] + t * f)
    return np.array(out)


def rotate(x, pos, freq, factor=1.0):
    """x [..., tokens, dim]: of the first 2 * len(freq) coordinates, i turns with
    i + len(freq)."""
    half = len(freq)
    a = pos[:, None] * freq[None, :]
    c, s = np.cos(a) * factor, np.sin(a) * factor
    u, v, rest = x[..., :half], x[..., half:2 * half], x[..., 2 * half:]
    return np.concatenate([u * c - v * s, v * c + u * s, rest], -1)


def scores(q, k, scale, window=None):
    """q, k [tokens, dim] of one head -> masked scores [tokens, tokens]."""
    n = q.shape[0]
    gap = np.arange(n)[:, None] - np.arange(n)[None, :]
    seen = gap >= 0
    if window is not None:
        seen &= gap < window
    return np.where(seen, (q @ k.T) * scale, -np.inf)


def softmax(s):
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def sink_softmax(s, sink):
    """The denominator also counts exp(sink)."""
    m = np.maximum(s.max(-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - m))


def attention(h, w, c, eps):
    """w: tensors by their name behind '.mix.'; c: the mixer's sizes."""
    n, H, G, D, VD = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    pos = np.arange(n, dtype=np.float64)
    freq, factor = yarn(c["rot"]["dims"], c["rot"]["base"], c["rot"]["scaling"])
    q = rotate((h @ w["q"].T).reshape(n, H, D).transpose(1, 0, 2), pos, freq, factor)
    k = rotate((h @ w["k"].T).reshape(n, G, D).transpose(1, 0, 2), pos, freq, factor)
    v = (h @ w["v"].T).reshape(n, G, VD).transpose(1, 0, 2)
    out = np.empty((n, H, VD))
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = sink_softmax(scores(q[hd], k[g], c["scale"]), w["sink"][hd]) @ v[g]
    return out.reshape(n, H * VD) @ w["o"].T


def differential_attention(h, w, c, eps):
    n, H, G, D, VD = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    pos = np.arange(n, dtype=np.float64)
    freq = banded(c["rot"]["dims"], c["rot"]["base"], c["rot"]["scaling"])
    q = rotate((h @ w["q"].T).reshape(n, H, 2, D).transpose(1, 2, 0, 3), pos, freq)
    k = rotate((h @ w["k"].T).reshape(n, G, 2, D).transpose(1, 2, 0, 3), pos, freq)
    v = (h @ w["v"].T).reshape(n, G, VD).transpose(1, 0, 2)
    lam = math.exp(w["lq1"] @ w["lk1"]) - math.exp(w["lq2"] @ w["lk2"]) + c["diff"]
    out = np.empty((n, H, VD))
    for hd in range(H):
        g = hd // (H // G)
        a = [softmax(scores(q[hd, m], k[g, m], c["scale"], c["mask"]["size"])) @ v[g] for m in (0, 1)]
        out[:, hd] = rms(a[0] - lam * a[1], eps) * (1.0 - c["diff"])
    return (out.reshape(n, H * VD) * sigmoid(h @ w["g"].T)) @ w["o"].T


def short_conv(x, taps_w):
    """Causal depth-wise convolution; taps_w [channels, taps], last tap = now."""
    n, taps = x.shape[0], taps_w.shape[1]
    out = np.zeros_like(x)
    for back in range(min(taps, n)):
        out[back:] += taps_w[:, taps - 1 - back] * x[:n - back]
    return out


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def softplus(z):
    return np.logaddexp(0.0, z)


def delta_inputs(h, w, c):
    """-> q, k [n, kv_heads, dim], v [n, heads, vdim], beta [n, heads], log decay
    [n, heads, dim]."""
    n, H, G, D, VD = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (silu(short_conv(h @ w[x].T, w[x + ".conv"])) for x in "qkv")
    q = unit(q.reshape(n, G, D)) * D ** -0.5
    k = unit(k.reshape(n, G, D))
    beta = sigmoid(h @ w["b"].T)
    dt = softplus((h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]).reshape(n, H, D)
    return q, k, v.reshape(n, H, VD), beta, -np.exp(w["A_log"])[:, None] * dt


def delta_rule(q, k, v, beta, log_decay):
    """One head, token by token: q, k, log_decay [n, dim], v [n, vdim], beta [n]."""
    S = np.zeros((q.shape[1], v.shape[1]))
    out = np.empty_like(v)
    for t in range(q.shape[0]):
        S = np.exp(log_decay[t])[:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out


def channel_delta(h, w, c, eps):
    n, H, G, VD = h.shape[0], c["heads"], c["kv_heads"], c["vdim"]
    q, k, v, beta, ld = delta_inputs(h, w, c)
    o = np.empty((n, H, VD))
    for hd in range(H):
        g = hd // (H // G)
        o[:, hd] = delta_rule(q[:, g], k[:, g], v[:, hd], beta[:, hd], ld[:, hd])
    o = rms(o, eps) * w["norm"]
    gate = sigmoid((h @ w["g1"].T) @ w["g2"].T)
    return (o.reshape(n, H * VD) * gate) @ w["o"].T


def dense(h, w):
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


MIXERS = {"attention": attention, "attention_2": differential_attention,
          "channel_delta": channel_delta}


def order(cfg):
    """(layer, pass to announce before it or None) in the order in which they run."""
    n, loop = len(cfg["layers"]), cfg["loop"]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, tensors, tokens, layers_out=None):
    """Logits [tokens, vocab] of one sequence."""
    eps = cfg["norm"]["eps"]
    x = centred_norm(tensors["embed"][np.asarray(tokens)], tensors["embed.norm"], eps)
    for i, announced in order(cfg):
        if announced is not None:
            x = x + tensors["loop.step"][announced]
        layer, p = cfg["layers"][i], f"l{i}."
        w = {k[len(p):]: v for k, v in tensors.items() if k.startswith(p)}
        mix = {k[4:]: v for k, v in w.items() if k.startswith("mix.")}
        x = x + MIXERS[layer["type"]](centred_norm(x, w["norm1"], eps), mix, layer["mixer"], eps)
        if layer["mlp"] is not None:
            ff = {k[4:]: v for k, v in w.items() if k.startswith("mlp.")}
            x = x + dense(centred_norm(x, w["norm2"], eps), ff)
        if layers_out is not None:
            layers_out.append(x.copy())
    return centred_norm(x, tensors["final.norm"], eps) @ tensors["head"].T


# ---- models ----------------------------------------------------------------------

def tensor_shapes(cfg, rank=None):
    """rank: of the decay's and the gate's inner projections."""
    W, V, loop = cfg["width"], cfg["vocab"], cfg["loop"]
    out = {"embed": (V, W), "embed.norm": (W,), "loop.step": (loop["times"], W),
           "final.norm": (W,), "head": (V, W)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, G, D, VD = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        mats = {}
        if layer["type"] == "attention":
            mats = {"q": (H * D, W), "k": (G * D, W), "v": (G * VD, W), "sink": (H,),
                    "o": (W, H * VD)}
        elif layer["type"] == "attention_2":
            mats = {"q": (H * 2 * D, W), "k": (G * 2 * D, W), "v": (G * VD, W),
                    "lq1": (D,), "lk1": (D,), "lq2": (D,), "lk2": (D,),
                    "g": (H * VD, W), "o": (W, H * VD)}
        else:
            T, (ra, rg) = m["conv"], rank or (7, 5)
            mats = {"q": (G * D, W), "q.conv": (G * D, T), "k": (G * D, W), "k.conv": (G * D, T),
                    "v": (H * VD, W), "v.conv": (H * VD, T), "b": (H, W), "A_log": (H,),
                    "norm": (VD,), "a1": (ra, W), "a2": (H * D, ra), "dt_bias": (H * D,),
                    "g1": (rg, W), "g2": (H * VD, rg), "o": (W, H * VD)}
        out[p + "norm1"] = (W,)
        out.update({p + "mix." + k: s for k, s in mats.items()})
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W),
                        p + "mlp.down": (W, ff)})
    return out


def random_tensors(cfg, seed, rank=None):
    """Weights that keep every mechanism visible: projections at unit gain (queries and
    keys a little above it), gains away from 1, sinks as large as scores, decays from
    fast to slow, lambda away from its constant."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, rank).items():
        last = name.rsplit(".", 1)[-1]
        z = rng.standard_normal(shape)
        if name == "embed":
            a = z
        elif name == "loop.step":
            a = 0.7 * z
        elif last in ("norm1", "norm2") or name in ("embed.norm", "final.norm"):
            a = 0.3 * z
        elif last == "norm":
            a = 1.0 + 0.3 * z
        elif last == "conv":
            a = 0.6 * z
        elif last == "sink":
            a = 1.5 + z
        elif last == "A_log":
            a = 1.5 * z - 1.0
        elif last == "dt_bias":
            a = 2.0 * z - 1.5
        elif last[:2] in ("lq", "lk"):
            a = z / shape[0] ** 0.5 * 0.8
        else:
            a = (1.6 if last in ("q", "k", "a2", "b") else 1.0) * z / np.sqrt(shape[-1])
        out[name] = bf16(a)
    return out
