"""Small random layer-stack models for the tests: configurations, weights, model folders."""
from __future__ import annotations

import json
import os
import struct

import numpy as np


def mixer(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=10000.0, scale=None):
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
                rot=dict(base=base, dims=rot_dim), scale=(dim + rot_dim) ** -0.5 if scale is None else scale)


def moe(experts, top, ff):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))


def config(vocab, width, layers, loop=None, eps=1e-5, emb_scale=1.0):
    c = dict(architecture="Gegepel", vocab=vocab, width=width, embedding=dict(scale=emb_scale), norm=dict(eps=eps),
             layers=[dict(type="latent_attention", mixer=m, mlp=f) for m, f in layers])
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


# every size different from layer to layer, odd ones included; one layer without a feed-forward; more than
# 16 heads; a latent of more than one 128-wide group
MIXED = config(211, 84, [
    (mixer(3, 20, 12, 28, 36, 40, base=500.0), moe(5, 2, 24)),
    (mixer(17, 36, 8, 12, 20, 136, scale=0.3), None),
    (mixer(2, 7, 4, 70, 65, 33, base=3e4), moe(9, 3, 44)),
], loop=(1, 3, 2), eps=1e-3, emb_scale=1.7)
# loop from the first layer to the last, three passes, all experts used
LOOP_ALL = config(97, 64, [
    (mixer(4, 16, 16, 16, 32, 32), moe(4, 4, 32)),
    (mixer(5, 24, 6, 20, 24, 48), moe(6, 1, 16)),
], loop=(0, 2, 3), emb_scale=0.75)
# no loop; a single pass is the loop's other degenerate form
PLAIN = config(130, 48, [(mixer(1, 8, 8, 8, 16, 16), moe(3, 2, 8)), (mixer(6, 12, 10, 9, 18, 22), moe(7, 2, 30))])
ONCE = config(130, 48, [(mixer(2, 8, 8, 8, 16, 16), moe(1, 1, 40)), (mixer(6, 12, 10, 9, 18, 22), None)], loop=(1, 2, 1))
# every token uses every expert: no discontinuous choice (bf16 comparisons of every row)
ALL_EXPERTS = config(150, 72, [(mixer(5, 18, 14, 22, 30, 130), moe(3, 3, 28)), (mixer(3, 40, 4, 34, 40, 20), moe(2, 2, 36))],
                     loop=(1, 2, 2))
CONFIGS = dict(all_experts=ALL_EXPERTS, mixed=MIXED, loop_all=LOOP_ALL, plain=PLAIN, once=ONCE)


def shapes(cfg):
    """name -> shape of every tensor the checkpoint of `cfg` holds."""
    V, W = cfg["vocab"], cfg["width"]
    s = {"embed": (V, W), "head": (V, W), "final.norm": (W,), "final.norm.b": (W,)}
    if cfg.get("loop"):
        s["loop.in"], s["loop.step"] = (W, 2 * W), (cfg["loop"]["times"], W)
    for i, L in enumerate(cfg["layers"]):
        m, f, p = L["mixer"], L["mlp"], f"l{i}."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            s[p + n], s[p + n + ".b"] = (W,), (W,)
        H, q, kv = m["heads"], m["q_rank"], m["kv_rank"]
        s.update({p + "mix.dq": (q, W), p + "mix.dq.norm": (q,), p + "mix.uq": (H * (m["dim"] + m["rot_dim"]), q),
                  p + "mix.dkv": (kv + m["rot_dim"], W), p + "mix.dkv.norm": (kv,), p + "mix.uk": (H * m["dim"], kv),
                  p + "mix.uv": (H * m["vdim"], kv), p + "mix.sink": (H,), p + "mix.g": (H, W),
                  p + "mix.o": (W, H * m["vdim"])})
        if f:
            ff = f["expert"]["ff"]
            s[p + "mlp.router"] = (f["router"]["experts"], W)
            for e in range(f["router"]["experts"]):
                s[f"{p}mlp.e{e}.gate"], s[f"{p}mlp.e{e}.up"], s[f"{p}mlp.e{e}.down"] = (ff, W), (ff, W), (W, ff)
    return s


def to_bf16(a):
    """fp32 rounded to the nearest bf16 (ties to even), as fp32."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32)


def random_weights(cfg, seed, peak=2.5):
    """bf16-exact random weights.  Queries are scaled by `peak`, so that attention singles out keys."""
    rng, w = np.random.default_rng(seed), {}
    for n, sh in shapes(cfg).items():
        if n.endswith(".b"):
            a = rng.normal(0, 0.2, sh)
        elif n.endswith(".sink"):
            a = rng.normal(1.0, 1.5, sh)
        elif len(sh) == 1:
            a = rng.uniform(0.5, 1.5, sh)
        elif n == "embed":
            a = rng.normal(0, 1, sh)
        elif n == "loop.step":
            a = rng.normal(0, 0.5, sh)
        else:
            a = rng.normal(0, sh[1] ** -0.5, sh) * (peak if n.endswith("uq") else 3.0 if n.endswith("router") else 1.0)
        w[n] = to_bf16(a.astype(np.float32))
    return w


def f64(w):
    return {k: v.astype(np.float64) for k, v in w.items()}


def write_model(folder, cfg, w):
    """config.json + model.safetensors (bf16)."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    head, at, blobs = {"__metadata__": {"format": "pt"}}, 0, []
    for n, a in w.items():
        b = (np.ascontiguousarray(a, np.float32).view(np.uint32) >> 16).astype(np.uint16).tobytes()
        head[n] = dict(dtype="BF16", shape=list(a.shape), data_offsets=[at, at + len(b)])
        blobs.append(b)
        at += len(b)
    h = json.dumps(head).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))


def engine(ti, cfg, w, dtype="float32", max_seq=256, max_batch=4):
    e = ti.Engine.stack(cfg, dtype, max_seq=max_seq, max_batch=max_batch)
    for n, a in w.items():
        e.set_weight(n, a)
    return e


def tokens(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def row_error(got, ref):
    """Per row: rms of the difference (mean taken off) over the rms of the reference rows."""
    d = np.asarray(got, np.float64) - ref
    d -= d.mean(-1, keepdims=True)
    return np.sqrt(np.mean(d * d, -1)) / np.sqrt(np.mean((ref - ref.mean(-1, keepdims=True)) ** 2))
