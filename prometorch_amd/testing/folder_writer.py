"""Random models in folder form (config.json + model.safetensors) for tests and benchmarks."""
from __future__ import annotations

import json
import os
import struct

import numpy as np


def to_bf16(a: np.ndarray) -> np.ndarray:
    """Nearest-even bfloat16 bits of fp32 values."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16(b: np.ndarray) -> np.ndarray:
    return (b.astype(np.uint32) << 16).view(np.float32)


def write_safetensors(path: str, tensors: dict) -> None:
    """tensors: name -> array; uint16 arrays are written as BF16, fp32 as F32, int32 as I32."""
    names = {np.dtype(np.uint16): "BF16", np.dtype(np.float32): "F32", np.dtype(np.int32): "I32"}
    head, off = {}, 0
    for n, a in tensors.items():
        head[n] = {"dtype": names[a.dtype], "shape": list(a.shape), "data_offsets": [off, off + a.nbytes]}
        off += a.nbytes
    text = json.dumps(head).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for a in tensors.values():
            f.write(np.ascontiguousarray(a).tobytes())


def tovasun_shapes(cfg: dict) -> dict:
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], W)
    side = cfg.get("token_side")
    if side:
        out["side.embed"] = (V, len(cfg["layers"]) * side["dim"])
    for i, layer in enumerate(cfg["layers"]):
        p, m = "l%d." % i, layer["mixer"]
        x = p + "mix."
        out[p + "norm1"] = out[p + "norm1b"] = (W,)
        H, d, v = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "attention":
            G = m["kv_heads"]
            out.update({x + "q": (H * d, W), x + "k": (G * d, W), x + "v": (G * v, W), x + "q.norm": (H * d,), x + "k.norm": (G * d,)})
        else:
            r, k = m["rot_dim"], m["kv_rank"]
            out.update({x + "q": (H * (d + r), W), x + "dkv": (k + r, W), x + "dkv.norm": (k,), x + "uk": (H * d, k), x + "uv": (H * v, k)})
        out[x + "o"] = (W, H * v)
        if layer.get("mlp"):
            ff = layer["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "norm2b": (W,), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff)})
        if side:
            out.update({p + "side.gate": (side["dim"], W), p + "side.proj": (W, side["dim"]), p + "side.norm": (W,)})
    return out


def nadozen_shapes(cfg: dict) -> dict:
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,), "final.norm.b": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = "l%d." % i, layer["mixer"]
        x = p + "mix."
        out.update({p + "norm1": (W,), p + "norm1.b": (W,)})
        if layer["type"] == "wkv":
            hd, rank = m["heads"] * m["dim"], layer["rank"]
            out.update({x + "mu." + s: (W,) for s in "rkvgw"})
            out.update({x + s: (hd, W) for s in "rkvg"})
            out.update({x + "w1": (rank, W), x + "w2": (hd, rank), x + "w0": (hd,), x + "u": (m["heads"], m["dim"]), x + "norm": (hd,),
                        x + "o": (W, hd)})
        else:
            l, r = m["left"], m["right"]
            q, inner = l["heads"] * l["dim"], r["heads"] * r["vdim"]
            ch = inner + 2 * r["groups"] * r["state"]
            x, y = x + "left.", x + "right."
            out.update({x + "q": (q, W), x + "k": (l["kv_heads"] * l["dim"], W), x + "q.norm": (l["dim"],), x + "k.norm": (l["dim"],),
                        x + "sink": (l["heads"],), x + "g": (q, W), x + "o": (W, q)})
            out.update({y + "in": (inner + ch + r["heads"], W), y + "conv": (ch, r["conv"]), y + "conv.b": (ch,), y + "dt_bias": (r["heads"],),
                        y + "A_log": (r["heads"],), y + "D": (r["heads"],), y + "norm": (inner,), y + "o": (W, inner)})
        branches = 1
        if layer.get("mlp"):
            ff = layer["mlp"]["ff"]
            branches = 2
            out.update({p + "norm2": (W,), p + "norm2.b": (W,), p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff)})
        for q in range(1, branches + 1):
            out.update({p + "hc%d.in" % q: (S,), p + "hc%d.out" % q: (S,), p + "hc%d.mix" % q: (S, S)})
    return out


def tensor_shapes(cfg: dict) -> dict:
    """Name -> shape of every tensor a config asks for.  The rank of a wkv layer's decay product, which is only in the tensors, is the
    layer's entry "rank" here (readers of config.json ignore it)."""
    return {"Tovasun": tovasun_shapes, "Nadozen": nadozen_shapes}[cfg["architecture"]](cfg)


# vectors and small matrices that are no norms, by the last part of their names
NADOZEN_SPREAD = {
    "b": lambda a: 0.3 * a,
    "w0": lambda a: 1.5 * a - 2.5,
    "u": lambda a: 0.7 * a,
    "sink": lambda a: 1.0 + a,
    "conv": lambda a: a * a.shape[1] ** -0.5,
    "dt_bias": lambda a: a - 2.0,
    "A_log": lambda a: 0.8 * a,
    "D": lambda a: a,
}


def random_weights(cfg: dict, seed: int) -> dict:
    """Name -> fp32 array of bfloat16 values.  Matrices keep the scale of their input; norms scatter around 1,
    decays reach from a few tokens to a few hundred."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        a = rng.standard_normal(shape, np.float32)
        last = name.rsplit(".", 1)[-1]
        if last in NADOZEN_SPREAD:
            a = NADOZEN_SPREAD[last](a)
        elif ".hc" in name and last == "mix":
            a = np.eye(shape[0], dtype=np.float32) * 0.9 + 0.3 / shape[0] * a
        elif ".hc" in name:  # in and out: one unit over all streams, some of them against it
            a = (1.0 + 0.8 * a) / (shape[0] if last == "in" else 1.0)
        elif ".mu." in name:
            a = 0.5 + 0.3 * a
        elif len(shape) == 1:
            a = 1.0 + 0.25 * a
        elif name not in ("embed", "side.embed"):
            a *= 0.5 if name == "loop.step" else shape[1] ** -0.5
        out[name] = from_bf16(to_bf16(a))
    return out


def write_model_folder(path: str, cfg: dict, weights: dict) -> str:
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(path, "model.safetensors"), {n: to_bf16(a) for n, a in weights.items()})
    return path
