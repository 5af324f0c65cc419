"""Small Nukopel models for the tests: configurations of many sizes, and models whose
weights are placed by hand so that one key, one gate or one expert decides the
logits."""
from __future__ import annotations

import numpy as np

import nukopel_oracle as N


def latent(heads=3, dim=20, rot=8, vdim=12, rank=28, window=19, base=10000.0, scale=None, mlp="moe"):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
                      "mask": {"size": window}, "rot": {"base": base, "dims": rot},
                      "scale": (dim + rot) ** -0.5 if scale is None else scale},
            "mlp": moe() if mlp == "moe" else mlp}


def linear(decay=(0.5, 0.93, 0.998), dim=18, vdim=14, mlp="moe"):
    return {"type": "lightning",
            "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)},
            "mlp": moe() if mlp == "moe" else mlp}


def moe(experts=5, top=2, ff=24, limit=1.2, shared_ff=40, shared_limit=0.9):
    m = {"kind": "moe", "router": {"experts": experts, "top": top},
         "expert": {"ff": ff, "limit": limit}}
    if shared_ff:
        m["shared"] = {"ff": shared_ff, "limit": shared_limit}
    return m


def config(layers, width=48, vocab=75, taps=3, eps=1e-5, embed=3.0):
    return {"architecture": "Nukopel", "canon": {"taps": taps}, "embedding": {"scale": embed},
            "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


# several sizes and orders of layers; none a multiple of what the kernels like unless
# it says so
SIZES = {
    "mixed": config([latent(), linear(), latent(window=7, heads=2), linear(decay=(0.8,))]),
    "no_feed_forward": config([linear(mlp=None), latent(mlp=None)]),
    "one_of_each": config([latent(heads=1, dim=1, rot=2, vdim=1, rank=1, window=1),
                           linear(decay=(1.0,), dim=1, vdim=1)], width=16, vocab=16, taps=1),
    "odd": config([latent(heads=5, dim=11, rot=6, vdim=7, rank=21, window=33,
                          mlp=moe(experts=7, top=3, ff=9, shared_ff=13)),
                   linear(decay=(0.0, 0.3, 1.0, 0.999, 0.7), dim=9, vdim=5,
                          mlp=moe(experts=3, top=3, ff=17, shared_ff=0))],
                  width=44, vocab=37, taps=6, embed=1.0),
    "even": config([latent(heads=4, dim=64, rot=32, vdim=64, rank=128, window=64,
                            mlp=moe(experts=8, top=2, ff=64, shared_ff=128)),
                     linear(decay=(0.9, 0.99), dim=64, vdim=64,
                            mlp=moe(experts=8, top=1, ff=128, shared_ff=64))],
                    width=128, vocab=256, taps=4),
    "many_heads": config([latent(heads=19, dim=8, rot=4, vdim=6, rank=40, window=50),
                          latent(heads=33, dim=4, rot=2, vdim=4, rank=16, window=12)], width=72),
    "wide_heads": config([latent(heads=2, dim=96, rot=64, vdim=136, rank=150, window=40),
                          latent(heads=1, dim=40, rot=16, vdim=270, rank=64, window=25),
                          linear(decay=(0.97, 0.4), dim=130, vdim=140)], width=96),
    # rows of other lengths than multiples of four, and of thousands of values
    "width_46": config([latent(mlp=moe(experts=3, top=2, ff=11, shared_ff=6)), linear()], width=46),
    "width_2600": config([latent(heads=1), linear(decay=(0.9,))], width=2600),
    "width_4400": config([latent(heads=1, mlp=moe(experts=2, top=1, ff=2100, shared_ff=70))], width=4400),
    "width_8300": config([linear(decay=(0.9,), mlp=None)], width=8300, vocab=33),
    "many_experts": config([linear(mlp=moe(experts=70, top=6, ff=8, shared_ff=8)),
                            latent(mlp=moe(experts=130, top=9, ff=4, shared_ff=20))], width=64),
}
# sizes at which the prompt kernels take their large tiles; for a long prompt
LARGE = config([latent(heads=24, dim=128, rot=64, vdim=128, rank=160, window=300,
                       mlp=moe(experts=4, top=2, ff=2100, shared_ff=2100)),
                linear(decay=(0.9, 0.99, 0.999), dim=128, vdim=128, mlp=None)], width=256, vocab=300)

# every expert is chosen, so no rounding can choose another one
_all = moe(experts=3, top=3)
STEADY = config([latent(mlp=_all), linear(mlp=_all), latent(window=7, heads=2, mlp=_all),
                 linear(decay=(0.8,), mlp=_all)])


def build(tmp_path, cfg, seed=0, edit=None):
    """-> (folder, tensors)."""
    t = N.random_tensors(cfg, seed)
    if edit:
        edit(t)
        t = {k: N.bf16(v) for k, v in t.items()}
    return N.write_model(tmp_path, cfg, t), t


def needle_model(window, heads=2, width=32, vocab=24, rank=16, extra_layer=None, taps=2):
    """One latent layer in which token ASK attends to token NEEDLE and to nothing else
    it can see: their score is ~14 above all others, whatever the gap, and what is
    found turns up in logit FOUND.  Weights everywhere else are small noise."""
    ask, needle, found = 1, 2, 5
    layer = latent(heads=heads, dim=8, rot=4, vdim=8, rank=rank, window=window, scale=1.0, mlp=None)
    cfg = config([layer] + ([extra_layer] if extra_layer else []), width=width, vocab=vocab, taps=taps,
                 embed=1.0)
    t = N.random_tensors(cfg, 5)
    rng = np.random.default_rng(9)
    emb = np.zeros((vocab, width))
    emb[:, 4:] = 0.3 * rng.standard_normal((vocab, width - 4))
    emb[:, 3] = 1.5                             # what every token carries
    emb[ask, 1] = 4.0
    emb[needle, 2] = 4.0
    t["embed"] = emb
    for n in ("q", "dkv", "uk", "uv", "o"):
        t["l0.mix." + n] = 0.02 * rng.standard_normal(t["l0.mix." + n].shape)
    for n in ("norm1", "norm1b"):
        t["l0." + n] = np.array(1.0)
    t["l0.canon1"] = np.zeros_like(t["l0.canon1"])
    t["l0.mix.dkv.norm"] = np.ones(rank)
    for h in range(heads):
        t["l0.mix.q"][h * 12, 1] = 1.0          # unrotated query dimension 0 <- ASK
        t["l0.mix.uk"][h * 8, 0] = 1.0          # unrotated key dimension 0 <- latent 0
        t["l0.mix.uv"][h * 8, 0] = 1.0
        t["l0.mix.o"][found, h * 8] = 1.0       # value dimension 0 -> residual FOUND
        t["l0.mix.uv"][h * 8 + 1, 1] = 1.0      # the common part -> residual 6: without the
        t["l0.mix.o"][6, h * 8 + 1] = 1.0       # needle it is what the output norm scales up
    t["l0.mix.dkv"][0, 2] = 1.0                 # latent 0 <- NEEDLE
    t["l0.mix.dkv"][1, 3] = 1.0                 # latent 1 <- the common part
    head = np.zeros((vocab, width))
    np.fill_diagonal(head, 1.0)
    t["head"] = head
    t["final.norm"] = np.array(1.0)
    return cfg, {k: N.bf16(v) for k, v in t.items()}, ask, needle, found


def row_errors(got, want):
    """Per row: root mean square of the difference over that of the wanted logits,
    both without their mean."""
    d = got.astype(np.float64) - want
    d -= d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1) / np.maximum((w * w).mean(-1), 1e-12))
