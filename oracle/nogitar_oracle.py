"""Plain restatement of the recurrent layer-stack models (architecture "Nogitar").

One function per mechanism, whole-sequence, token by token where the mechanism is a recurrence, no
cache, no batching, numpy only; what the engine's recurrent and grouped-query layers are compared with.
It shares no code with the product.  A model is a (config, weights) pair: config the parsed config.json
dictionary, weights a name -> float array dictionary with the checkpoint's tensor names.
"""
from __future__ import annotations

import math

import numpy as np

_erf = np.vectorize(math.erf, otypes=[np.float64])


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_erf(z):
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------------ embedding
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the bigram table per token; a sequence's first token has the row behind the buckets."""
    t = [int(v) for v in tokens]
    return [buckets if i == 0 else (t[i - 1] * mul_prev + t[i] * mul_cur) % buckets for i in range(len(t))]


def sinusoid(n, width):
    """[n, width]: sine at even, cosine at odd entries of position / 10000^(2i / width)."""
    out = np.zeros((n, width))
    for e in range(width):
        a = np.arange(n) * 10000.0 ** (-2.0 * (e // 2) / width)
        out[:, e] = np.cos(a) if e % 2 else np.sin(a)
    return out


def embed(tokens, w, cfg):
    e = cfg["embedding"]
    b = e["bigram"]
    x = w["embed"][np.asarray(tokens)] * e["scale"]
    x = x + w["bigram"][bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])]
    return x + sinusoid(len(tokens), cfg["width"])


# ------------------------------------------------------------------ attention
def query_temperature(n, coef, every):
    return 1.0 + coef * np.log(np.floor((np.arange(n) + 1) / every) + 1.0)


def softmax_plus_one(s):
    """Rows of s (-inf: masked): exp(s) / (1 + sum exp(s))."""
    m = np.maximum(np.max(s, axis=-1, keepdims=True), 0.0)
    e = np.exp(s - m)
    return e / (np.exp(-m) + np.sum(e, axis=-1, keepdims=True))


def keys_values(h, w, pre, mx, eps):
    """Keys (normalised over the whole projection) and values [kv head, T, size]."""
    T, G = h.shape[0], mx["kv_heads"]
    k = rms(h @ w[pre + "k"].T, eps) * w[pre + "k.norm"]
    v = h @ w[pre + "v"].T
    return k.reshape(T, G, mx["dim"]).transpose(1, 0, 2), v.reshape(T, G, mx["vdim"]).transpose(1, 0, 2)


def attention(h, w, pre, mx, eps, kv):
    T, H = h.shape[0], mx["heads"]
    q = rms(h @ w[pre + "q"].T, eps) * w[pre + "q.norm"]
    q = q * query_temperature(T, mx["q_temp"]["coef"], mx["q_temp"]["every"])[:, None]
    q = q.reshape(T, H, mx["dim"])
    out = np.zeros((T, H, mx["vdim"]))
    causal = np.tril(np.ones((T, T), bool))
    for hd in range(H):
        g = hd // (H // mx["kv_heads"])
        s = np.where(causal, (q[:, hd] @ kv[0][g].T) * mx["scale"], -np.inf)
        out[:, hd] = softmax_plus_one(s) @ kv[1][g]
    o = out.reshape(T, H * mx["vdim"]) * sigmoid(h @ w[pre + "g"].T)
    return o @ w[pre + "o"].T


# ------------------------------------------------------------------ recurrences
def causal_conv(x, wc, b):
    """Per channel: the last tap belongs to the current token, zeros before the start."""
    taps = wc.shape[1]
    out = np.zeros_like(x)
    for t in range(x.shape[0]):
        acc = b.copy()
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                acc = acc + wc[:, j] * x[s]
        out[t] = acc
    return out


def ssd_recurrence(x, dt, a_log, B, C, D):
    """x [T, heads, P], dt [T, heads] (after softplus), B / C [T, heads, N] -> y [T, heads, P]."""
    T, H, P = x.shape
    S = np.zeros((H, B.shape[2], P))
    y = np.zeros_like(x)
    for t in range(T):
        S = np.exp(-np.exp(a_log) * dt[t])[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        y[t] = np.sum(S * C[t][:, :, None], axis=1) + D[:, None] * x[t]
    return y


def grouped_rms(y, groups, eps):
    T, n = y.shape
    return rms(y.reshape(T, groups, n // groups), eps).reshape(T, n)


def mamba2(h, w, pre, mx, eps):
    T, H, P, N, G = h.shape[0], mx["heads"], mx["vdim"], mx["state"], mx["groups"]
    inner = H * P
    a = h @ w[pre + "in"].T
    z, xbc, dt = a[:, :inner], a[:, inner : 2 * inner + 2 * G * N], a[:, 2 * inner + 2 * G * N :]
    xbc = silu(causal_conv(xbc, w[pre + "conv"], w[pre + "conv.b"]))
    x = xbc[:, :inner].reshape(T, H, P)
    head_group = np.arange(H) // (H // G)
    B = xbc[:, inner : inner + G * N].reshape(T, G, N)[:, head_group]
    C = xbc[:, inner + G * N :].reshape(T, G, N)[:, head_group]
    y = ssd_recurrence(x, softplus(dt + w[pre + "dt_bias"]), w[pre + "A_log"], B, C, w[pre + "D"])
    y = grouped_rms(y.reshape(T, inner) * silu(z), mx["norm_groups"], eps) * w[pre + "norm"]
    return y @ w[pre + "o"].T


def lru_recurrence(u, r, i, lam):
    S, out = np.zeros(u.shape[1]), np.zeros_like(u)
    for t in range(u.shape[0]):
        la = -8.0 * r[t] * softplus(lam)
        S = np.exp(la) * S + np.sqrt(-np.expm1(2.0 * la)) * i[t] * u[t]
        out[t] = S
    return out


def block_gates(u, wr, b):
    """sigmoid of a block-diagonal product: wr [blocks, n, n] (out, in), b [blocks, n]."""
    n = wr.shape[1]
    return np.concatenate([sigmoid(u[:, k * n : (k + 1) * n] @ wr[k].T + b[k]) for k in range(wr.shape[0])], axis=1)


def rglru(h, w, pre, mx, eps):
    y = gelu_tanh(h @ w[pre + "y"].T + w[pre + "y.b"])
    u = causal_conv(h @ w[pre + "x"].T + w[pre + "x.b"], w[pre + "conv"], w[pre + "conv.b"])
    s = lru_recurrence(u, block_gates(u, w[pre + "ra"], w[pre + "ra.b"]), block_gates(u, w[pre + "ri"], w[pre + "ri.b"]),
                       w[pre + "lam"])
    return (s * y) @ w[pre + "o"].T


# ------------------------------------------------------------------ model
def mlp(h, w, pre):
    return gelu_erf(h @ w[pre + "up"].T) @ w[pre + "down"].T


def forward(tokens, w, cfg, layers_out=None):
    """Logits [T, vocab] of every position; layers_out (a list) receives the residual after each layer."""
    x, eps, kvs = embed(tokens, w, cfg), cfg["norm"]["eps"], {}
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        if L["type"] == "attention":
            src = mx.get("kv_from")
            if src is None:
                kvs[i] = keys_values(x, w, p + "mix.", mx, eps)
            m = attention(x, w, p + "mix.", mx, eps, kvs[i if src is None else src])
        else:
            m = dict(mamba2=mamba2, rglru=rglru)[L["type"]](x, w, p + "mix.", mx, eps)
        x = x + rms(m, eps) * w[p + "norm1"]
        if L.get("mlp"):
            x = x + rms(mlp(x, w, p + "mlp."), eps) * w[p + "norm2"]
        if layers_out is not None:
            layers_out.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T


def greedy(prompt, n_new, w, cfg):
    """Greedy continuation, the whole sequence recomputed per token: (tokens, each step's logits)."""
    seq, out, lg = list(prompt), [], []
    for _ in range(n_new):
        l = forward(seq, w, cfg)[-1]
        out.append(int(np.argmax(l)))
        lg.append(l)
        seq.append(out[-1])
    return out, lg
