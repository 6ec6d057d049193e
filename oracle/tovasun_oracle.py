"""Plain float64 restatement of the Tovasun decoder (test infrastructure): whole sequences, no cache, one function per
mechanism, numpy only.  Nothing here is shared with the product path.

A model is (cfg, w): cfg the dictionary config.json holds, w a mapping from tensor name to array."""
from __future__ import annotations

import math

import numpy as np


# ---- norms and activations ---------------------------------------------------------------------
def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, weight, eps):
    return rms(x, eps) * weight


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return np.square(np.maximum(z, 0.0))


# ---- rotation ----------------------------------------------------------------------------------
def yarn_frequencies(freq, dims, base, scaling):
    """Blend of f_i and f_i / factor along the ramp between the two correction dimensions; also the amplitude of cos, sin."""
    def corr(turns):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(corr(scaling["fast"])), 0)
    hi = min(math.ceil(corr(scaling["slow"])), dims - 1)
    ramp = np.clip((np.arange(len(freq)) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    out = freq / scaling["factor"] * ramp + freq * (1.0 - ramp)
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [tokens, heads, n]: pairs (2i, 2i + 1) of the first rot['dims'] values turn by position * f_i."""
    dims = rot["dims"]
    freq = float(rot["base"]) ** (-np.arange(0, dims, 2, dtype=np.float64) / dims)
    amp = 1.0
    if rot.get("scaling"):
        freq, amp = yarn_frequencies(freq, dims, float(rot["base"]), rot["scaling"])
    a = np.asarray(positions, np.float64)[:, None] * freq[None, :]
    c, s = (np.cos(a) * amp)[:, None, :], (np.sin(a) * amp)[:, None, :]
    out = np.array(x, np.float64)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


# ---- attention ---------------------------------------------------------------------------------
def visible(n, mask):
    """[n, n] boolean: which keys j each position i sees.  No size: everything up to itself."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    see = j <= i
    if mask and mask.get("size"):
        see = see & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    return see


def softmax_attend(q, k, v, scale, see, softcap=None):
    """q [n, H, d], k [n, G, d], v [n, G, dv]; query head h uses key/value head h // (H / G)."""
    n, H, _ = q.shape
    per = H // k.shape[1]
    out = np.zeros((n, H, v.shape[-1]))
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        if softcap:
            s = softcap * np.tanh(s / softcap)
        s = np.where(see, s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, h // per]
    return out


def attention(h, w, name, m, eps):
    n = h.shape[0]
    pos = np.arange(n)
    q = rms_norm(h @ w[name + "q"].T, w[name + "q.norm"], eps).reshape(n, m["heads"], m["dim"])
    k = rms_norm(h @ w[name + "k"].T, w[name + "k.norm"], eps).reshape(n, m["kv_heads"], m["dim"])
    v = (h @ w[name + "v"].T).reshape(n, m["kv_heads"], m["vdim"])
    q, k = rotate(q, pos, m["rot"]), rotate(k, pos, m["rot"])
    o = softmax_attend(q, k, v, m["scale"], visible(n, m.get("mask")), m.get("softcap"))
    return o.reshape(n, -1) @ w[name + "o"].T


def latent_attention(h, w, name, m, eps):
    n, H, d, rd, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    pos = np.arange(n)
    q = (h @ w[name + "q"].T).reshape(n, H, d + rd)
    down = h @ w[name + "dkv"].T
    c = rms_norm(down[:, :rank], w[name + "dkv.norm"], eps)
    k_rot = rotate(down[:, None, rank:], pos, m["rot"])
    q_rot = rotate(q[:, :, d:], pos, m["rot"])
    k = (c @ w[name + "uk"].T).reshape(n, H, d)
    v = (c @ w[name + "uv"].T).reshape(n, H, m["vdim"])
    full_q = np.concatenate([q[:, :, :d], q_rot], axis=2)
    full_k = np.concatenate([k, np.broadcast_to(k_rot, (n, H, rd))], axis=2)
    o = softmax_attend(full_q, full_k, v, m["scale"], visible(n, m.get("mask")), m.get("softcap"))
    return o.reshape(n, -1) @ w[name + "o"].T


MIXERS = {"attention": attention, "latent_attention": latent_attention}


# ---- feed-forward and the per-layer token input -------------------------------------------------
def dense_ff(h, w, name):
    return relu_squared(h @ w[name + "up"].T) @ w[name + "down"].T


def token_side(x, tokens, w, name, layer, dim, eps):
    e = w["side.embed"][tokens][:, layer * dim:(layer + 1) * dim]
    g = gelu_tanh(x @ w[name + "side.gate"].T) * e
    return rms_norm(g @ w[name + "side.proj"].T, w[name + "side.norm"], eps)


# ---- the model ---------------------------------------------------------------------------------
def layer(x, tokens, w, cfg, i):
    L, name, eps = cfg["layers"][i], "l%d." % i, cfg["norm"]["eps"]
    mixed = MIXERS[L["type"]](rms_norm(x, w[name + "norm1"], eps), w, name + "mix.", L["mixer"], eps)
    x = x + rms_norm(mixed, w[name + "norm1b"], eps)
    if L.get("mlp"):
        ff = dense_ff(rms_norm(x, w[name + "norm2"], eps), w, name + "mlp.")
        x = x + rms_norm(ff, w[name + "norm2b"], eps)
    if cfg.get("token_side"):
        x = x + token_side(x, tokens, w, name, i, cfg["token_side"]["dim"], eps)
    return x


def layer_runs(cfg):
    """(layer, pass) in running order; pass is None outside the loop."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    inner = list(range(loop["start"], loop["stop"]))
    return ([(i, None) for i in range(loop["start"])] + [(i, t) for t in range(loop["times"]) for i in inner] +
            [(i, None) for i in range(loop["stop"], n)])


def residuals(tokens, w, cfg):
    """Residual stream after every layer run: [layer runs, tokens, width]."""
    tokens = np.asarray(tokens)
    emb = w["embed"][tokens].astype(np.float64)
    x = emb
    out = []
    for i, t in layer_runs(cfg):
        if t is not None and i == cfg["loop"]["start"]:
            if t > 0:
                x = x + emb
            x = x + w["loop.step"][t]
        x = layer(x, tokens, w, cfg, i)
        out.append(x)
    return np.stack(out)


def logits(tokens, w, cfg):
    x = residuals(tokens, w, cfg)[-1]
    return rms_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T
