"""Plain float64 restatement of the Nadozen decoder (test infrastructure): whole sequences, token by token where there is a
recurrence, no cache, one function per mechanism, numpy only.  Nothing here is shared with the product path.

A model is (cfg, w): cfg the dictionary config.json holds, w a mapping from tensor name to array."""
from __future__ import annotations

import math

import numpy as np


# ---- norms and activations ---------------------------------------------------------------------
def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, weight, bias, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * weight + bias


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


# ---- embedding ---------------------------------------------------------------------------------
def sinusoid(positions, width):
    """[positions, width]: pairs (sin, cos) of position times a frequency that falls from 1 to about 1 / 10000."""
    c = np.arange(width)
    angle = np.asarray(positions, np.float64)[:, None] * 10000.0 ** (-(c - c % 2) / width)
    return np.where(c % 2 == 0, np.sin(angle), np.cos(angle))


# ---- mixers ------------------------------------------------------------------------------------
def wkv(h, w, name, m, eps):
    """Time mixing: a matrix state per head, decayed per key channel."""
    n, H, d = h.shape[0], m["heads"], m["dim"]
    before = np.vstack([np.zeros_like(h[:1]), h[:-1]])
    mixed = {s: h + (before - h) * w[name + "mu." + s] for s in "rkvgw"}
    r, k, v = ((mixed[s] @ w[name + s].T).reshape(n, H, d) for s in "rkv")
    gate = silu(mixed["g"] @ w[name + "g"].T)
    decay = np.exp(-np.exp(np.tanh(mixed["w"] @ w[name + "w1"].T) @ w[name + "w2"].T + w[name + "w0"])).reshape(n, H, d)
    o = np.zeros((n, H, d))
    for a in range(H):
        state = np.zeros((d, d))                      # [key channel, value channel]
        for t in range(n):
            outer = np.outer(k[t, a], v[t, a])
            o[t, a] = (state + w[name + "u"][a][:, None] * outer).T @ r[t, a]
            state = decay[t, a][:, None] * state + outer
    return (rms(o, eps).reshape(n, H * d) * w[name + "norm"] * gate) @ w[name + "o"].T


def visible(n, mask):
    """[n, n] boolean: which keys j each position i sees."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    see = j <= i
    return see & (i - j < mask["size"]) if mask else see


def sink_softmax(s, sink):
    """Rows of scores to weights; exp(sink) is one more term of the denominator."""
    top = np.maximum(s.max(axis=1, keepdims=True), sink)
    p = np.exp(s - top)
    return p / (p.sum(axis=1, keepdims=True) + np.exp(sink - top))


def gated_attention(h, w, name, m, eps):
    """Grouped-query attention whose values are the projected keys, with a sink per head and an output gate."""
    n, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = rms((h @ w[name + "q"].T).reshape(n, H, d), eps) * w[name + "q.norm"]
    raw = (h @ w[name + "k"].T).reshape(n, G, d)
    k = rms(raw, eps) * w[name + "k.norm"]
    see = visible(n, m.get("mask"))
    o = np.zeros((n, H, d))
    for a in range(H):
        g = a // (H // G)
        s = np.where(see, (q[:, a] @ k[:, g].T) * m["scale"], -np.inf)
        o[:, a] = sink_softmax(s, w[name + "sink"][a]) @ raw[:, g]
    return (o.reshape(n, H * d) * sigmoid(h @ w[name + "g"].T)) @ w[name + "o"].T


def causal_conv(x, taps, bias):
    """x [tokens, channels], taps [channels, n], the last one for the token itself."""
    n = taps.shape[1]
    padded = np.vstack([np.zeros((n - 1, x.shape[1])), x])
    return sum(padded[i:i + len(x)] * taps[:, i] for i in range(n)) + bias


def ssm(h, w, name, m, eps):
    """State-space mixer: one decay per head, keys and queries shared by the heads of a group."""
    n, H, v, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * v
    z, xbc, dt = np.split(h @ w[name + "in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    x, B, C = np.split(silu(causal_conv(xbc, w[name + "conv"], w[name + "conv.b"])), [inner, inner + G * N], axis=1)
    x, B, C = x.reshape(n, H, v), B.reshape(n, G, N), C.reshape(n, G, N)
    dt = softplus(dt + w[name + "dt_bias"])
    y = np.zeros((n, H, v))
    for a in range(H):
        g = a // (H // G)
        state = np.zeros((N, v))
        for t in range(n):
            state = np.exp(-np.exp(w[name + "A_log"][a]) * dt[t, a]) * state + dt[t, a] * np.outer(B[t, g], x[t, a])
            y[t, a] = state.T @ C[t, g] + w[name + "D"][a] * x[t, a]
    y = y.reshape(n, inner) * silu(z)
    return (rms(y.reshape(n, m["norm_groups"], -1), eps).reshape(n, inner) * w[name + "norm"]) @ w[name + "o"].T


def parallel(h, w, name, m, eps):
    return (m["left_scale"] * gated_attention(h, w, name + "left.", m["left"], eps) +
            m["right_scale"] * ssm(h, w, name + "right.", m["right"], eps))


MIXERS = {"wkv": wkv, "parallel": parallel}


def swiglu(h, w, name):
    return (silu(h @ w[name + "gate"].T) * (h @ w[name + "up"].T)) @ w[name + "down"].T


# ---- streams -----------------------------------------------------------------------------------
def hyper_connect(x, w, name, sublayer):
    """x [streams, tokens, width]: the sublayer reads a blend of the streams and adds to blends of them."""
    y = sublayer(np.einsum("s,snw->nw", w[name + "in"], x))
    return np.einsum("st,snw->tnw", w[name + "mix"], x) + w[name + "out"][:, None, None] * y


# ---- the model ---------------------------------------------------------------------------------
def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def residuals(tokens, w, cfg):
    """Sum of the streams after every layer: [layers, tokens, width]."""
    tokens, eps = np.asarray(tokens), cfg["norm"]["eps"]
    w = {k: np.asarray(v, np.float64) for k, v in w.items()}
    emb = w["embed"][tokens] + sinusoid(np.arange(len(tokens)), cfg["width"])
    x = np.repeat(emb[None], cfg["streams"], axis=0)
    out = []
    for i in range(len(cfg["layers"])):
        j = owner(cfg, i)
        L, p = cfg["layers"][j], "l%d." % j
        x = hyper_connect(x, w, p + "hc1.", lambda u: MIXERS[L["type"]](
            layer_norm(u, w[p + "norm1"], w[p + "norm1.b"], eps), w, p + "mix.", L["mixer"], eps))
        if L.get("mlp"):
            x = hyper_connect(x, w, p + "hc2.", lambda u: swiglu(layer_norm(u, w[p + "norm2"], w[p + "norm2.b"], eps), w, p + "mlp."))
        out.append(x.sum(axis=0))
    return np.stack(out)


def head(x, w, cfg):
    """Logits of residual rows."""
    return layer_norm(x, w["final.norm"], w["final.norm.b"], cfg["norm"]["eps"]) @ np.asarray(w["head"], np.float64).T * cfg["logit_scale"]


def logits(tokens, w, cfg):
    return head(residuals(tokens, w, cfg)[-1], w, cfg)
