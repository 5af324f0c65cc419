"""Plain, slow restatement of the Nukopel design in float64 numpy: one function
per mechanism, whole sequences only, no cache.  The tests compare the library
with it; it shares no code with the product.

Also here: random models of any size (bfloat16-valued weights) and a writer for
the safetensors container, so that the tests can hand the library a model folder.
"""
from __future__ import annotations

import json
import struct
from pathlib import Path

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def scalar_norm(x, g, eps):
    """RMS norm whose gain is one number."""
    return rms(x, eps) * float(g)


def input_conv(h, taps_w):
    """h + a causal depth-wise convolution of h; taps_w [width, taps], last tap = now."""
    n, taps = h.shape[0], taps_w.shape[1]
    out = h.copy()
    for back in range(taps):
        if back < n:
            out[back:] += taps_w[:, taps - 1 - back] * h[:n - back]
    return out


def rotate(x, pos, base):
    """x [..., tokens, dims]: coordinate i turns with i + dims/2."""
    d = x.shape[-1]
    half = d // 2
    f = base ** (-2.0 * np.arange(half) / d)
    a = pos[:, None] * f[None, :]
    u, v = x[..., :half], x[..., half:]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)], -1)


def latent_attention(h, w, c, eps):
    """w: tensors by their name behind '.mix.'; c: the mixer's sizes."""
    n = h.shape[0]
    H, D, R, VD, L = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    pos = np.arange(n, dtype=np.float64)
    q = (h @ w["q"].T).reshape(n, H, D + R).transpose(1, 0, 2)
    down = h @ w["dkv"].T
    lat = rms(down[:, :L], eps) * w["dkv.norm"]
    k_rot = rotate(down[:, L:], pos, c["rot"]["base"])
    q_rot = rotate(q[..., D:], pos, c["rot"]["base"])
    k = (lat @ w["uk"].T).reshape(n, H, D).transpose(1, 0, 2)
    v = (lat @ w["uv"].T).reshape(n, H, VD).transpose(1, 0, 2)
    s = (q[..., :D] @ k.transpose(0, 2, 1) + q_rot @ k_rot.T) * c["scale"]
    gap = pos[:, None] - pos[None, :]
    s = np.where((gap >= 0) & (gap < c["mask"]["size"]), s, -np.inf)
    p = np.exp(s - s.max(-1, keepdims=True))
    p /= p.sum(-1, keepdims=True)
    o = (p @ v).transpose(1, 0, 2)
    o = o * sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(n, H * VD) @ w["o"].T


def lightning(h, w, c, eps):
    n = h.shape[0]
    H, D, VD = c["heads"], c["dim"], c["vdim"]
    q = silu(h @ w["q"].T).reshape(n, H, D)
    k = silu(h @ w["k"].T).reshape(n, H, D)
    v = silu(h @ w["v"].T).reshape(n, H, VD)
    S = np.zeros((H, D, VD))
    decay = np.asarray(c["decay"], np.float64)[:, None, None]
    o = np.empty((n, H, VD))
    for t in range(n):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    o = rms(o.reshape(n, H * VD), eps) * w["norm"]
    return (o * sigmoid(h @ w["g"].T)) @ w["o"].T


def expert(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def route(h, router, top):
    """-> chosen experts [n, top] and their weights."""
    z = h @ router.T
    idx = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    zc = np.take_along_axis(z, idx, -1)
    e = np.exp(zc - zc.max(-1, keepdims=True))
    return idx, e / e.sum(-1, keepdims=True)


def moe(h, w, c):
    idx, wt = route(h, w["router"], c["router"]["top"])
    y = np.zeros_like(h)
    for e in range(c["router"]["experts"]):
        t, slot = np.nonzero(idx == e)
        if t.size:
            y[t] += wt[t, slot][:, None] * expert(
                h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], c["expert"]["limit"])
    if c.get("shared"):
        y = y + expert(h, w["shared.gate"], w["shared.up"], w["shared.down"],
                       c["shared"]["limit"])
    return y


MIXERS = {"latent_attention": latent_attention, "lightning": lightning}


def forward(cfg, tensors, tokens, layers_out=None):
    """Logits [tokens, vocab] of one sequence."""
    eps = cfg["norm"]["eps"]
    x = tensors["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        w = {k[len(p):]: v for k, v in tensors.items() if k.startswith(p)}
        mix = {k[4:]: v for k, v in w.items() if k.startswith("mix.")}
        h = input_conv(scalar_norm(x, w["norm1"], eps), w["canon1"])
        x = x + scalar_norm(MIXERS[layer["type"]](h, mix, layer["mixer"], eps), w["norm1b"], eps)
        if layer["mlp"] is not None:
            ff = {k[4:]: v for k, v in w.items() if k.startswith("mlp.")}
            h = scalar_norm(x, w["norm2"], eps)
            x = x + scalar_norm(moe(h, ff, layer["mlp"]), w["norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return scalar_norm(x, tensors["final.norm"], eps) @ tensors["head"].T


# ---- models ------------------------------------------------------------------

def to_bf16_bits(a):
    """float -> bfloat16 bit patterns, round to nearest even."""
    u = np.array(a, np.float32, order="C").view(np.uint32)
    return np.asarray((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16_bits(b):
    return np.asarray(np.asarray(b).astype(np.uint32) << 16).view(np.float32).astype(np.float64)


def bf16(a):
    return from_bf16_bits(to_bf16_bits(a))


def tensor_shapes(cfg):
    W, V, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": ()}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, D, VD = m["heads"], m["dim"], m["vdim"]
        out[p + "canon1"] = (W, taps)
        out[p + "norm1"] = out[p + "norm1b"] = ()
        if layer["type"] == "latent_attention":
            R, L = m["rot_dim"], m["kv_rank"]
            out.update({p + "mix.q": (H * (D + R), W), p + "mix.dkv": (L + R, W),
                        p + "mix.dkv.norm": (L,), p + "mix.uk": (H * D, L),
                        p + "mix.uv": (H * VD, L), p + "mix.g": (H, W), p + "mix.o": (W, H * VD)})
        else:
            out.update({p + "mix.q": (H * D, W), p + "mix.k": (H * D, W), p + "mix.v": (H * VD, W),
                        p + "mix.g": (H * VD, W), p + "mix.norm": (H * VD,),
                        p + "mix.o": (W, H * VD)})
        f = layer["mlp"]
        if f is not None:
            out[p + "norm2"] = out[p + "norm2b"] = ()
            out[p + "mlp.router"] = (f["router"]["experts"], W)
            names = [(f"e{e}", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
            if f.get("shared"):
                names.append(("shared", f["shared"]["ff"]))
            for name, ff in names:
                out[f"{p}mlp.{name}.gate"] = out[f"{p}mlp.{name}.up"] = (ff, W)
                out[f"{p}mlp.{name}.down"] = (W, ff)
    return out


def random_tensors(cfg, seed):
    """Weights that keep every mechanism visible: projections at unit gain (keys and
    queries a little above it), gains away from 1, convolution taps of size ~0.4."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm", "norm1", "norm2", "norm1b", "norm2b"):
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif last == "canon1":
            a = 0.4 * rng.standard_normal(shape)
        elif name == "embed":
            a = rng.standard_normal(shape) / cfg["embedding"]["scale"]
        else:
            gain = 1.6 if last in ("q", "k", "uk", "dkv") else 2.0 if last == "router" else 1.0
            a = gain * rng.standard_normal(shape) / np.sqrt(shape[-1])
        out[name] = bf16(a)
    return out


def write_model(folder, cfg, tensors):
    """config.json + model.safetensors (bfloat16; integer arrays as int32)."""
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    header, blobs, at = {}, [], 0
    for name, a in tensors.items():
        a = np.asarray(a)
        if a.dtype.kind in "iu":
            raw, dtype = np.ascontiguousarray(a, "<i4").tobytes(), "I32"
        else:
            raw, dtype = to_bf16_bits(a).tobytes(), "BF16"
        header[name] = {"dtype": dtype, "shape": list(a.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(folder / "model.safetensors", "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for b in blobs:
            f.write(b)
    return folder


def read_model(folder):
    folder = Path(folder)
    cfg = json.loads((folder / "config.json").read_text())
    raw = (folder / "model.safetensors").read_bytes()
    n = struct.unpack("<Q", raw[:8])[0]
    head = json.loads(raw[8:8 + n])
    out = {}
    for name, e in head.items():
        if name == "__metadata__":
            continue
        lo, hi = e["data_offsets"]
        b = raw[8 + n + lo:8 + n + hi]
        a = from_bf16_bits(np.frombuffer(b, "<u2")) if e["dtype"] == "BF16" else np.frombuffer(b, "<i4")
        out[name] = a.reshape(e["shape"])
    return cfg, out
