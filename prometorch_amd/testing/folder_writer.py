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


def tensor_shapes(cfg: dict) -> dict:
    """Name -> shape of every tensor a Tovasun config asks for."""
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


def random_weights(cfg: dict, seed: int) -> dict:
    """Name -> fp32 array of bfloat16 values.  Matrices keep the scale of their input; norms scatter around 1."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        a = rng.standard_normal(shape, np.float32)
        if len(shape) == 1:
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
