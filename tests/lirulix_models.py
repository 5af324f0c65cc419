"""Small Lirulix models for the tests: configurations of many sizes, and models whose
weights are placed by hand so that one key, a sink or one loud token decides the
logits."""
from __future__ import annotations

import numpy as np

import lirulix_oracle as L
from nukopel_models import row_errors  # noqa: F401


def yarn(factor=3.0, original=64, fast=8.0, slow=0.5):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def banded(factor=5.0, low=0.5, high=3.0, original=96):
    return {"factor": factor, "low": low, "high": high, "original": original}


def full(heads=3, kv=1, dim=20, rot=12, vdim=14, base=5000.0, scale=None, scaling=None, ff=40):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                      "rot": {"base": base, "dims": rot, "scaling": scaling or yarn()},
                      "scale": dim ** -0.5 if scale is None else scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def diff(heads=4, kv=2, dim=10, rot=6, vdim=18, window=19, lam=0.4, base=900.0, scale=None,
         scaling=None, ff=40):
    return {"type": "attention_2",
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "diff": lam,
                      "mask": {"size": window},
                      "rot": {"base": base, "dims": rot, "scaling": scaling or banded()},
                      "scale": dim ** -0.5 if scale is None else scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def delta(heads=4, kv=2, dim=12, vdim=10, taps=4, ff=None):
    return {"type": "channel_delta",
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": taps},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, loop=(0, 1, 1), width=48, vocab=75, eps=1e-5):
    return {"architecture": "Lirulix", "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
            "width": width, "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]}}


# several sizes, orders of layers and loops; none a multiple of what the kernels like
# unless it says so
SIZES = {
    "mixed": config([delta(ff=24), full(), diff(), delta()], loop=(1, 3, 2)),
    "whole_loop": config([diff(window=7), delta(heads=2, kv=2), full(heads=2, kv=2)], loop=(0, 3, 3)),
    "no_feed_forward": config([full(ff=None), diff(ff=None)], loop=(1, 2, 1)),
    "ones": config([full(heads=1, dim=2, rot=2, vdim=1, ff=1),
                    diff(heads=1, kv=1, dim=2, rot=2, vdim=3, window=1, ff=1),
                    delta(heads=1, kv=1, dim=1, vdim=1, taps=1)], loop=(2, 3, 1), width=16, vocab=16),
    "odd": config([diff(heads=6, kv=2, dim=11, rot=4, vdim=7, window=33, ff=9),
                   full(heads=5, kv=5, dim=9, rot=8, vdim=21, ff=13),
                   delta(heads=6, kv=2, dim=9, vdim=5, taps=7, ff=17)],
                  loop=(1, 2, 4), width=44, vocab=37, eps=1e-3),
    "even": config([full(heads=4, kv=2, dim=64, rot=64, vdim=64, ff=128),
                    diff(heads=4, kv=2, dim=32, rot=32, vdim=64, window=64, ff=128),
                    delta(heads=2, kv=1, dim=64, vdim=64, ff=64)], loop=(0, 2, 2), width=128, vocab=256),
    "many_heads": config([full(heads=34, kv=2, dim=4, rot=2, vdim=6),
                          diff(heads=20, kv=1, dim=6, rot=6, vdim=4, window=12),
                          delta(heads=21, kv=3, dim=4, vdim=6, taps=2)], width=72),
    "wide_heads": config([full(heads=2, dim=160, rot=64, vdim=136, ff=None),
                          diff(heads=1, kv=1, dim=72, rot=72, vdim=270, window=25, ff=None),
                          full(heads=1, dim=300, rot=8, vdim=40, ff=None),
                          delta(heads=2, kv=1, dim=130, vdim=140), delta(heads=1, kv=1, dim=40, vdim=270)],
                         width=96),
    # rows of other lengths than multiples of four, and of thousands of values
    "width_46": config([full(ff=11), diff(), delta()], loop=(0, 3, 2), width=46),
    "width_2600": config([full(heads=1, ff=2100), delta(heads=1, kv=1)], loop=(0, 2, 2), width=2600),
    "width_8300": config([diff(heads=1, kv=1, ff=None), delta(heads=1, kv=1)], loop=(0, 2, 2),
                         width=8300, vocab=33),
}
# sizes at which the prompt kernels take their large tiles; for a long prompt
LARGE = config([diff(heads=8, kv=2, dim=64, rot=64, vdim=128, window=300, ff=2100),
                full(heads=8, kv=2, dim=128, rot=128, vdim=128, ff=512),
                delta(heads=4, kv=2, dim=128, vdim=128)], loop=(1, 3, 2), width=256, vocab=300)


def build(tmp_path, cfg, seed=0, edit=None, rank=None):
    """-> (folder, tensors)."""
    t = L.random_tensors(cfg, seed, rank)
    if edit:
        edit(t)
        t = {k: L.bf16(v) for k, v in t.items()}
    return L.write_model(tmp_path, cfg, t), t


ASK, NEEDLE, FOUND = 1, 2, 5


def needle_model(kind, window=24, heads=2, kv=1, width=32, vocab=24, sink=-30.0):
    """One layer of attention ("full" or "diff") in which token ASK attends to token
    NEEDLE and to nothing else it can see: their score stands out whatever the gap, and
    what is found turns up in logit FOUND.  Weights everywhere else are small noise."""
    dim, rot, vdim = 8, 4, 8
    layer = full(heads=heads, kv=kv, dim=dim, rot=rot, vdim=vdim, scale=1.0, ff=None) if kind == "full" \
        else diff(heads=heads, kv=kv, dim=dim, rot=rot, vdim=vdim, window=window, scale=1.0, lam=0.2, ff=None)
    cfg = config([layer], width=width, vocab=vocab)
    t = L.random_tensors(cfg, 5)
    rng = np.random.default_rng(9)
    emb = np.zeros((vocab, width))
    emb[:, 6:] = 0.3 * rng.standard_normal((vocab, width - 6))
    emb[:, 3] = 1.5                             # what every token carries
    emb[ASK, 1] = 4.0
    emb[NEEDLE, 2] = 4.0
    t["embed"] = emb
    for n in ("q", "k", "v", "o", "g"):
        if "l0.mix." + n in t:
            t["l0.mix." + n] = 0.02 * rng.standard_normal(t["l0.mix." + n].shape)
    for n in ("embed.norm", "l0.norm1", "final.norm", "loop.step"):
        t[n] = np.zeros_like(t[n])
    maps = 1 if kind == "full" else 2
    for h in range(heads):
        t["l0.mix.q"][h * maps * dim + rot, 1] = 2.0   # an unrotated coordinate, first map
        t["l0.mix.o"][FOUND, h * vdim] = 2.0           # value 0 -> residual FOUND
        t["l0.mix.o"][4, h * vdim + 1] = 0.5           # the common part -> residual 4
    for g in range(kv):
        t["l0.mix.k"][g * maps * dim + rot, 2] = 2.0
        t["l0.mix.v"][g * vdim, 2] = 1.0               # value 0 <- NEEDLE
        t["l0.mix.v"][g * vdim + 1, 3] = 1.0           # value 1 <- the common part
    if kind == "full":
        t["l0.mix.sink"] = np.full(heads, sink)
    head = np.zeros((vocab, width))
    np.fill_diagonal(head, 1.0)
    t["head"] = head
    return cfg, {k: L.bf16(v) for k, v in t.items()}
