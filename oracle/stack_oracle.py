"""Plain fp64 / fp32 restatement of the layer-stack models (architecture "Gegepel").

One function per mechanism, whole-sequence, no cache, no batching, numpy only: the checker the
engine's layer-stack path (ti_engine_create_stack) is compared with.  It shares no code with the
product.  A model is a (config, weights) pair: config the parsed config.json dictionary, weights a
name -> float array dictionary with the checkpoint's tensor names.
"""
from __future__ import annotations

import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def layer_norm(x, w, b, eps):
    mu = np.mean(x, axis=-1, keepdims=True)
    d = x - mu
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w + b


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rotate_half(v, pos, dims, base):
    """v [..., n, d]: dimensions i and i + dims/2 of every row rotated by pos * base^(-2i/dims)."""
    half = dims // 2
    f = np.power(float(base), -2.0 * np.arange(half) / dims)
    a = np.asarray(pos, np.float64)[:, None] * f[None, :]
    c, s = np.cos(a).astype(v.dtype), np.sin(a).astype(v.dtype)
    u, w = v[..., :half].copy(), v[..., half:dims].copy()
    out = v.copy()
    out[..., :half] = u * c - w * s
    out[..., half:dims] = w * c + u * s
    return out


def softmax_with_sink(scores, sink):
    """Rows of `scores` (-inf = masked); the denominator also counts exp(sink)."""
    m = np.maximum(np.max(scores, axis=-1, keepdims=True), sink)
    e = np.exp(scores - m)
    return e / (np.sum(e, axis=-1, keepdims=True) + np.exp(sink - m))


def latent_attention(h, w, pre, mx, eps):
    """h [T, width] -> [T, width]: low-rank queries, one shared latent for keys and values, a rotated
    key part shared by the heads, causal softmax with a per-head sink, a sigmoid gate per head."""
    T = h.shape[0]
    H, d, r, dv, kr = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    pos = np.arange(T)
    cq = rms_norm(h @ w[pre + "dq"].T, w[pre + "dq.norm"], eps)
    q = (cq @ w[pre + "uq"].T).reshape(T, H, d + r).transpose(1, 0, 2)
    kv = h @ w[pre + "dkv"].T
    c = rms_norm(kv[:, :kr], w[pre + "dkv.norm"], eps)
    qr = rotate_half(q[:, :, d:], pos, mx["rot"]["dims"], mx["rot"]["base"])
    kr_ = rotate_half(kv[None, :, kr:], pos, mx["rot"]["dims"], mx["rot"]["base"])[0]
    k = (c @ w[pre + "uk"].T).reshape(T, H, d).transpose(1, 0, 2)
    v = (c @ w[pre + "uv"].T).reshape(T, H, dv).transpose(1, 0, 2)
    s = (q[:, :, :d] @ k.transpose(0, 2, 1) + qr @ kr_.T[None]) * h.dtype.type(mx["scale"])
    s = np.where(np.tril(np.ones((T, T), bool))[None], s, -np.inf)
    p = softmax_with_sink(s, w[pre + "sink"][:, None, None])
    o = p @ v                                                       # [H, T, dv]
    g = sigmoid(h @ w[pre + "g"].T)                                 # [T, H]
    o = (o * g.T[:, :, None]).transpose(1, 0, 2).reshape(T, H * dv)
    return o @ w[pre + "o"].T


def router(h, wr, top):
    """(chosen experts [T, top], their softmax scores over all experts, not renormalised)."""
    z = h @ wr.T
    e = np.exp(z - np.max(z, axis=-1, keepdims=True))
    s = e / np.sum(e, axis=-1, keepdims=True)
    idx = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return idx, np.take_along_axis(s, idx, axis=-1)


def expert(h, w, pre):
    return (silu(h @ w[pre + ".gate"].T) * (h @ w[pre + ".up"].T)) @ w[pre + ".down"].T


def moe(h, w, pre, ml):
    idx, sc = router(h, w[pre + "router"], ml["router"]["top"])
    out = np.zeros_like(h)
    for e in range(ml["router"]["experts"]):
        t, k = np.nonzero(idx == e)
        if t.size:
            out[t] += sc[t, k][:, None] * expert(h[t], w, f"{pre}e{e}")
    return out


def layer(x, w, i, cfg):
    L, eps = cfg["layers"][i], cfg["norm"]["eps"]
    p = f"l{i}."

    def norm(v, n):
        return layer_norm(v, w[p + n], w[p + n + ".b"], eps)

    x = x + norm(latent_attention(norm(x, "norm1"), w, p + "mix.", L["mixer"], eps), "norm1b")
    if L.get("mlp"):
        x = x + norm(moe(norm(x, "norm2"), w, p + "mlp.", L["mlp"]), "norm2b")
    return x


def schedule(cfg):
    """[(layer, pass or None)] in running order; pass t >= 0 on the first layer of loop pass t."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        runs += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, None) for i in range(lp["stop"], n)]


def forward(tokens, w, cfg, layers_out=None):
    """Logits [T, vocab] of every position; layers_out (a list) receives the residual after each run."""
    x0 = w["embed"][np.asarray(tokens)] * w["embed"].dtype.type(cfg["embedding"]["scale"])
    x = x0
    for i, t in schedule(cfg):
        if t is not None:
            x = np.concatenate([x, x0], axis=-1) @ w["loop.in"].T + w["loop.step"][t]
        x = layer(x, w, i, cfg)
        if layers_out is not None:
            layers_out.append(x)
    x = layer_norm(x, w["final.norm"], w["final.norm.b"], cfg["norm"]["eps"])
    return x @ w["head"].T


def greedy(prompt, n_new, w, cfg):
    """Greedy continuation, the whole sequence recomputed per token: (tokens, each step's logits)."""
    seq, out, lg = list(prompt), [], []
    for _ in range(n_new):
        l = forward(seq, w, cfg)[-1]
        out.append(int(np.argmax(l)))
        lg.append(l)
        seq.append(out[-1])
    return out, lg
