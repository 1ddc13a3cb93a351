"""Small random Nogitar models for the tests: configurations and weights (folders, engines, comparisons:
stack_models.py)."""
from __future__ import annotations

import numpy as np

from stack_models import to_bf16


def attn(heads, kv_heads, dim, vdim, coef=0.4, every=16, scale=None, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, q_temp=dict(coef=coef, every=every),
             scale=dim ** -0.5 if scale is None else scale)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "attention", m


def mamba2(heads, vdim, state, groups=1, norm_groups=1, conv=4):
    return "mamba2", dict(heads=heads, vdim=vdim, state=state, groups=groups, norm_groups=norm_groups, conv=conv)


def rglru(width, blocks, conv=4):
    return "rglru", dict(width=width, blocks=blocks, conv=conv)


def config(vocab, width, layers, eps=1e-5, emb_scale=1.0, bigram=(101, 7, 3)):
    """layers: (type, mixer, feed-forward size or None)."""
    return dict(architecture="Nogitar", vocab=vocab, width=width, norm=dict(eps=eps),
                embedding=dict(scale=emb_scale, bigram=dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))),
                layers=[dict(type=t, mixer=m, mlp=None if f is None else dict(kind="dense", ff=f)) for (t, m), f in layers])


# every kind of layer, with and without a feed-forward, sizes all different; keys and values shared twice
# (other scale and temperature), groups and norm groups above one
MIXED = config(211, 84, [
    (rglru(60, 3, 4), 52),
    (attn(6, 2, 20, 28, 0.7, 7), None),
    (mamba2(6, 12, 20, 2, 3, 3), 100),
    (attn(6, 2, 20, 28, 0.2, 33, 0.4, kv_from=1), 36),
    (mamba2(4, 24, 36, 4, 1, 2), None),
    (attn(4, 4, 24, 16), 44),
    (attn(6, 2, 20, 28, 1.1, 5, kv_from=1), None),
    (rglru(72, 1, 2), None),
], eps=1e-3, emb_scale=1.7, bigram=(89, 1013, 77))
# nothing a multiple of four; one kernel tap, one block per few channels, products of multipliers past 32 bits
ODD = config(97, 50, [
    (mamba2(3, 7, 5, 3, 3, 1), 13),
    (rglru(33, 3, 3), None),
    (attn(5, 1, 7, 9, 2.0, 3), 21),
    (rglru(35, 7, 1), 9),
    (mamba2(1, 17, 13, 1, 1, 6), None),
    (attn(3, 3, 33, 18, 0.0, 1), None),
], emb_scale=0.6, bigram=(31, 2000000011, 1999999943))
# more query heads per key/value head than one tile, long states and heads, wide values
WIDE = config(130, 96, [
    (attn(34, 2, 40, 72, 0.3, 64), None),
    (mamba2(2, 40, 132, 2, 2, 4), None),
    (attn(4, 2, 136, 200, 0.3, 100), 64),
    (mamba2(2, 16, 256, 1, 2, 4), 40),
    (mamba2(5, 64, 64, 1, 5, 4), None),
    (rglru(320, 2, 4), None),
])
# one layer of each kind
ONE_ATTN = config(60, 32, [(attn(4, 2, 16, 24, 0.5, 4), None)])
ONE_SSD = config(60, 32, [(mamba2(4, 16, 16, 2, 2, 4), None)])
ONE_LRU = config(60, 32, [(rglru(48, 4, 4), None)])
ONE_MLP = config(60, 32, [(attn(1, 1, 8, 8), 70)])
CONFIGS = dict(mixed=MIXED, odd=ODD, wide=WIDE, one_attn=ONE_ATTN, one_ssd=ONE_SSD, one_lru=ONE_LRU, one_mlp=ONE_MLP)


def shapes(cfg):
    """name -> shape of every tensor the checkpoint of `cfg` holds."""
    V, W = cfg["vocab"], cfg["width"]
    s = {"embed": (V, W), "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, W), "final.norm": (W,), "head": (V, W)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}."
        s[p + "norm1"] = (W,)
        if L["mlp"]:
            s[p + "norm2"], s[p + "mlp.up"], s[p + "mlp.down"] = (W,), (L["mlp"]["ff"], W), (W, L["mlp"]["ff"])
        if L["type"] == "attention":
            q, k, v, o = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"], m["heads"] * m["vdim"]
            s.update({p + "mix.q": (q, W), p + "mix.q.norm": (q,), p + "mix.g": (o, W), p + "mix.o": (W, o)})
            if "kv_from" not in m:
                s.update({p + "mix.k": (k, W), p + "mix.k.norm": (k,), p + "mix.v": (v, W)})
        elif L["type"] == "mamba2":
            inner, bc, H = m["heads"] * m["vdim"], 2 * m["groups"] * m["state"], m["heads"]
            s.update({p + "mix.in": (2 * inner + bc + H, W), p + "mix.conv": (inner + bc, m["conv"]), p + "mix.conv.b": (inner + bc,),
                      p + "mix.dt_bias": (H,), p + "mix.A_log": (H,), p + "mix.D": (H,), p + "mix.norm": (inner,),
                      p + "mix.o": (W, inner)})
        else:
            w, b = m["width"], m["blocks"]
            s.update({p + "mix.y": (w, W), p + "mix.y.b": (w,), p + "mix.x": (w, W), p + "mix.x.b": (w,),
                      p + "mix.conv": (w, m["conv"]), p + "mix.conv.b": (w,), p + "mix.ra": (b, w // b, w // b),
                      p + "mix.ra.b": (b, w // b), p + "mix.ri": (b, w // b, w // b), p + "mix.ri.b": (b, w // b),
                      p + "mix.lam": (w,), p + "mix.o": (W, w)})
    return s


def random_weights(cfg, seed, peak=2.0):
    """bf16-exact random weights.  Query norms are scaled by `peak`, so that attention singles out keys;
    decays reach from a few tokens to thousands."""
    rng, w = np.random.default_rng(seed), {}
    for n, sh in shapes(cfg).items():
        if n.endswith(".A_log"):
            a = rng.uniform(-4.0, 2.0, sh)
        elif n.endswith(".dt_bias"):
            a = rng.normal(-2.0, 1.5, sh)
        elif n.endswith(".lam"):
            a = rng.uniform(-9.0, 1.0, sh)
        elif n.endswith(".b"):
            a = rng.normal(0, 0.3, sh)
        elif n.endswith("q.norm"):
            a = peak * rng.uniform(0.5, 1.5, sh)
        elif len(sh) == 1:
            a = rng.uniform(0.5, 1.5, sh)
        elif n in ("embed", "bigram"):
            a = rng.normal(0, 1, sh)
        else:
            a = rng.normal(0, sh[-1] ** -0.5, sh) * (2.0 if ".mix.ra" in n or ".mix.ri" in n else 1.0)
        w[n] = to_bf16(a.astype(np.float32))
    return w
