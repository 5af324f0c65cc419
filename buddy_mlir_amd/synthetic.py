"""Seeded synthetic Qwen2-shaped int8 decoder for tests and the benchmark.

Random-init weights ~ N(0, 0.02) generated on the device with torch's seeded
generator, quantized per output channel by libbuddy_hip's own quantizer (the
reference recipe, tools/buddy-codegen/import_model.py:837-848); norm weights
are ones; the KV cache is filled with N(0,1) for the first `context` rows.
Weights are kept in the importer's orientation: W[K, N] = [in, out].
"""
from __future__ import annotations

import numpy as np
import torch

from . import ops
from .session import DecoderSession, Shape

SEED = 0x5EED


def _gen(seed):
    return torch.Generator(device="cuda").manual_seed(seed)


def quantized_linear(K: int, N: int, seed: int, std: float = 0.02):
    W = torch.randn((K, N), generator=_gen(seed), device="cuda") * std
    q, s = ops.quantize_w8(W)
    del W
    return q, s


def inv_freq(head_dim: int, theta: float = 1e6) -> torch.Tensor:
    i = torch.arange(0, head_dim, 2, dtype=torch.int64).float()
    return (1.0 / (theta ** (i / head_dim))).cuda()


def make_layer(shape: Shape, layer: int, ln_jitter: float = 0.0):
    H, QN, KVN, I = (shape.hidden, shape.heads * shape.head_dim,
                     shape.kv_heads * shape.head_dim, shape.inter)
    base = SEED + 100 * layer
    w = {}
    w["wq"], w["sq"] = quantized_linear(H, QN, base + 1)
    w["wk"], w["sk"] = quantized_linear(H, KVN, base + 2)
    w["wv"], w["sv"] = quantized_linear(H, KVN, base + 3)
    w["wo"], w["so"] = quantized_linear(QN, H, base + 4)
    w["wg"], w["sg"] = quantized_linear(H, I, base + 5)
    w["wu"], w["su"] = quantized_linear(H, I, base + 6)
    w["wd"], w["sd"] = quantized_linear(I, H, base + 7)
    ones = torch.ones(H, device="cuda")
    if ln_jitter:
        w["ln1"] = ones + ln_jitter * torch.randn(H, generator=_gen(base + 8), device="cuda")
        w["ln2"] = ones + ln_jitter * torch.randn(H, generator=_gen(base + 9), device="cuda")
    else:
        w["ln1"], w["ln2"] = ones.clone(), ones.clone()
    return w


def make_globals(shape: Shape):
    g = {}
    g["embed"] = torch.randn((shape.vocab, shape.hidden), generator=_gen(SEED - 1),
                             device="cuda") * 0.02
    g["inv_freq"] = inv_freq(shape.head_dim)
    g["ln_f"] = torch.ones(shape.hidden, device="cuda")
    g["w_lm"], g["s_lm"] = quantized_linear(shape.hidden, shape.vocab, SEED - 2)
    return g


def make_kv(shape: Shape, kv_index: int, context: int) -> torch.Tensor:
    t = torch.zeros((shape.kv_heads, shape.max_len, shape.head_dim), device="cuda")
    if context:
        t[:, :context, :] = torch.randn((shape.kv_heads, context, shape.head_dim),
                                        generator=_gen(SEED + 7000 + kv_index),
                                        device="cuda")
    return t


def build_session(shape: Shape, context: int, keep_host: bool = False,
                  ln_jitter: float = 0.0):
    """Returns (session, host) where host holds numpy copies of every tensor
    when keep_host is set (for the CPU oracle), else None."""
    sess = DecoderSession(shape)
    host = {"layers": [], "kv": []} if keep_host else None
    g = make_globals(shape)
    sess.set_globals(g["embed"], g["inv_freq"], g["ln_f"], g["w_lm"], g["s_lm"])
    if keep_host:
        host["globals"] = {k: v.cpu().numpy() for k, v in g.items()}
    sess._globals = g
    for i in range(shape.layers):
        w = make_layer(shape, i, ln_jitter)
        sess.set_layer(i, w)
        if keep_host:
            host["layers"].append({k: v.cpu().numpy() for k, v in w.items()})
        del w
    for j in range(2 * shape.layers):
        kv = make_kv(shape, j, context)
        sess.set_kv(j, kv)
        if keep_host:
            host["kv"].append(kv.cpu().numpy())
        del kv
    torch.cuda.synchronize()
    return sess, host


def first_tokens(shape: Shape, n: int, seed: int = SEED + 9999) -> np.ndarray:
    rng = np.random.default_rng(seed)
    return rng.integers(0, shape.vocab, n).astype(np.int64)


# ---- Nukopel ---------------------------------------------------------------------

def nukopel_config(width: int, layers: str, heads: int, *, dim: int = 128, rot_dim: int = 64,
                   kv_rank: int = 512, window: int = 1024, experts: int = 16, top: int = 4,
                   ff: int = 1792, vocab: int = 32768, taps: int = 4) -> dict:
    """A configuration of the layers of a real model; `layers`: a letter per layer, a =
    latent attention, l = lightning."""
    mlp = {"kind": "moe", "router": {"experts": experts, "top": top},
           "expert": {"ff": ff, "limit": 7.0}, "shared": {"ff": ff, "limit": 7.0}}
    latent = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": dim, "kv_rank": kv_rank,
              "mask": {"size": window}, "rot": {"base": 1e6, "dims": rot_dim},
              "scale": (dim + rot_dim) ** -0.5}
    linear = {"heads": heads, "dim": dim, "vdim": dim,
              "decay": [1.0 - 2.0 ** -(3 + 5.0 * h / heads) for h in range(heads)]}
    return {"architecture": "Nukopel", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
            "embedding": {"scale": width ** 0.5}, "canon": {"taps": taps},
            "layers": [{"type": "latent_attention" if c == "a" else "lightning",
                        "mixer": latent if c == "a" else linear, "mlp": mlp} for c in layers]}


def nukopel_shapes(cfg: dict):
    """(name, shape, standard deviation) of every tensor; None: a gain of one."""
    W, V = cfg["width"], cfg["vocab"]
    yield "embed", (V, W), W ** -0.5
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        H, D, VD = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b", "norm2", "norm2b"):
            yield p + n, (), None
        yield p + "canon1", (W, cfg["canon"]["taps"]), 0.3
        if layer["type"] == "latent_attention":
            R, L = m["rot_dim"], m["kv_rank"]
            mats = {"q": (H * (D + R), W), "dkv": (L + R, W), "uk": (H * D, L), "uv": (H * VD, L),
                    "g": (H, W), "o": (W, H * VD)}
            yield p + "mix.dkv.norm", (L,), None
        else:
            mats = {"q": (H * D, W), "k": (H * D, W), "v": (H * VD, W), "g": (H * VD, W),
                    "o": (W, H * VD)}
            yield p + "mix.norm", (H * VD,), None
        for n, s in mats.items():
            yield p + "mix." + n, s, s[1] ** -0.5
        yield p + "mlp.router", (f["router"]["experts"], W), W ** -0.5
        names = [(f"e{e}", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
        for n, ff in names + [("shared", f["shared"]["ff"])]:
            yield f"{p}mlp.{n}.gate", (ff, W), W ** -0.5
            yield f"{p}mlp.{n}.up", (ff, W), W ** -0.5
            yield f"{p}mlp.{n}.down", (W, ff), ff ** -0.5
    yield "final.norm", (), None
    yield "head", (V, W), W ** -0.5


def write_nukopel_folder(folder, cfg: dict, seed: int = SEED):
    return write_folder(folder, cfg, nukopel_shapes(cfg), seed)


# ---- Lirulix ---------------------------------------------------------------------

def lirulix_config(width: int, layers: str, heads: int, *, kv_heads: int = 2, dim: int = 128,
                   window: int = 1024, ff: int = 8960, vocab: int = 32768, taps: int = 4,
                   loop: tuple = (0, 1, 1)) -> dict:
    """A configuration of the layers of a real model; `layers`: a letter per layer, f =
    attention over everything, s = differential attention through a window, d = gated
    delta rule."""
    kinds = {
        "f": ("attention",
              {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5,
               "rot": {"base": 1e6, "dims": dim,
                       "scaling": {"factor": 4.0, "original": 8192, "fast": 32.0, "slow": 1.0}}}),
        "s": ("attention_2",
              {"heads": heads, "kv_heads": kv_heads, "dim": dim // 2, "vdim": dim, "diff": 0.5,
               "scale": (dim // 2) ** -0.5, "mask": {"size": window},
               "rot": {"base": 1e5, "dims": dim // 2,
                       "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}),
        "d": ("channel_delta",
              {"heads": heads, "kv_heads": heads, "dim": dim, "vdim": dim, "conv": taps}),
    }
    return {"architecture": "Lirulix", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
            "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]},
            "layers": [{"type": kinds[c][0], "mixer": kinds[c][1], "mlp": {"kind": "dense", "ff": ff}}
                       for c in layers]}


def lirulix_shapes(cfg: dict, rank: int = 128):
    """(name, shape, standard deviation) of every tensor; `rank`: of the decay's and the
    gate's inner projections."""
    W, V = cfg["width"], cfg["vocab"]
    yield "embed", (V, W), 1.0
    yield "embed.norm", (W,), 0.1
    yield "loop.step", (cfg["loop"]["times"], W), 0.1
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", layer["mixer"], layer["mlp"]["ff"]
        H, G, D, VD = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        yield p + "norm1", (W,), 0.1
        yield p + "norm2", (W,), 0.1
        if layer["type"] == "attention":
            mats = {"q": (H * D, W), "k": (G * D, W), "v": (G * VD, W)}
            yield p + "mix.sink", (H,), 1.0
        elif layer["type"] == "attention_2":
            mats = {"q": (H * 2 * D, W), "k": (G * 2 * D, W), "v": (G * VD, W), "g": (H * VD, W)}
            for n in ("lq1", "lk1", "lq2", "lk2"):
                yield p + "mix." + n, (D,), 0.1
        else:
            mats = {"q": (G * D, W), "k": (G * D, W), "v": (H * VD, W), "b": (H, W),
                    "a1": (rank, W), "a2": (H * D, rank), "g1": (rank, W), "g2": (H * VD, rank)}
            for n, c in (("q", G * D), ("k", G * D), ("v", H * VD)):
                yield f"{p}mix.{n}.conv", (c, m["conv"]), 0.5
            yield p + "mix.A_log", (H,), 1.0
            yield p + "mix.dt_bias", (H * D,), 1.0
            yield p + "mix.norm", (VD,), 1.0
        for n, s in mats.items():
            yield p + "mix." + n, s, s[1] ** -0.5
        yield p + "mix.o", (W, H * VD), (H * VD) ** -0.5
        yield p + "mlp.gate", (ff, W), W ** -0.5
        yield p + "mlp.up", (ff, W), W ** -0.5
        yield p + "mlp.down", (W, ff), ff ** -0.5
    yield "final.norm", (W,), 0.1
    yield "head", (V, W), W ** -0.5


def write_lirulix_folder(folder, cfg: dict, seed: int = SEED):
    return write_folder(folder, cfg, lirulix_shapes(cfg), seed)


# ---- model folders ---------------------------------------------------------------

def write_folder(folder, cfg: dict, shapes, seed: int = SEED):
    """config.json and model.safetensors with random weights in bfloat16; shapes: (name,
    shape, standard deviation or None for ones) of every tensor."""
    import json
    import struct
    from math import prod
    from pathlib import Path

    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    tensors, head, at = list(shapes), {}, 0
    for name, shape, _ in tensors:
        size = 2 * prod(shape)
        head[name] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [at, at + size]}
        at += size
    text = json.dumps(head).encode()
    text += b" " * (-len(text) % 8)
    g = _gen(seed)
    with open(folder / "model.safetensors", "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for _, shape, std in tensors:
            if std is None:
                t = torch.ones(shape, dtype=torch.bfloat16)
            else:
                t = (torch.randn(shape, generator=g, device="cuda") * std).bfloat16().cpu()
            f.write(t.reshape(-1).view(torch.int16).numpy().tobytes())
    return folder
