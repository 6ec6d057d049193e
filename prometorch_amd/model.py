"""The stepping interface every decoder has, and the model registry: load() opens a .gguf file or a model folder
(config.json + model.safetensors, the architecture named by config.json) and returns an object with that interface."""
from __future__ import annotations

import ctypes as C
import os

import numpy as np

from . import _lib
from ._lib import DecodeConfig, check

PRECISIONS = {"bfloat16": 0, "float32": 1}


class Stepper:
    """Calls on a ptm_decoder: subclasses set L (the library), h (the decoder handle) and cfg (with 'vocab', 'hidden')."""

    def set_past_len(self, n: int) -> None:
        check(self.L.ptm_decode_set_past_len(self.h, n), "decode_set_past_len")

    def step(self, token: int) -> int:
        out = C.c_int64()
        check(self.L.ptm_decode_step(self.h, token, C.byref(out)), "decode_step")
        return out.value

    def prefill(self, tokens, chunk_rows: int = 0) -> int:
        """Run the prompt through the model in row batches, appending its K/V rows; returns the greedy next token
        (GGUFModel::forward with use_cache, gguf_model.h:2510-2571)."""
        n = len(tokens)
        buf = (C.c_int32 * n)(*[int(t) for t in tokens])
        out = C.c_int64()
        check(self.L.ptm_decode_prefill(self.h, buf, n, chunk_rows, C.byref(out)), "decode_prefill")
        return out.value

    def prefill_logits(self, tokens, want, chunk_rows: int = 0) -> np.ndarray:
        """prefill() that returns the logits of the ascending places `want` among these tokens: [len(want), vocab]."""
        n, w = len(tokens), len(want)
        buf = (C.c_int32 * n)(*[int(t) for t in tokens])
        wa = (C.c_int32 * max(1, w))(*[int(p) for p in want])
        out = np.empty((w, self.cfg["vocab"]), np.float32)
        nxt = C.c_int64()
        check(self.L.ptm_decode_prefill_logits(self.h, buf, n, chunk_rows, wa, w, out.ctypes.data, C.byref(nxt)),
              "decode_prefill_logits")
        return out

    def generate(self, prompt, uniforms, temperature: float, top_k: int, top_p: float, repeat_penalty: float = 1.0,
                 stop_ids=()) -> list:
        """Prompt, then up to len(uniforms) sampled tokens, ending before the first stop token (the serving loop of
        promeserve/api_handlers.h:848-923 with everything but the token ids kept on the device)."""
        from ._lib import Sampling
        n, m, ns = len(prompt), len(uniforms), len(stop_ids)
        pa = (C.c_int32 * n)(*[int(t) for t in prompt])
        ua = (C.c_float * m)(*[float(u) for u in uniforms])
        sa = (C.c_int32 * max(1, ns))(*[int(t) for t in stop_ids])
        out = (C.c_int64 * m)()
        n_out = C.c_int()
        check(self.L.ptm_decode_generate(self.h, pa, n, Sampling(temperature, top_k, top_p, repeat_penalty), ua, m, sa, ns, out,
                                         C.byref(n_out)), "decode_generate")
        return list(out[:n_out.value])

    def sampling_begin(self, temperature: float, top_k: int, top_p: float, repeat_penalty: float = 1.0) -> None:
        """Start a sampled generation: store the parameters, forget previously generated tokens."""
        from ._lib import Sampling
        check(self.L.ptm_decode_sampling_begin(self.h, Sampling(temperature, top_k, top_p, repeat_penalty)),
              "decode_sampling_begin")

    def sample(self, token: int, uniforms) -> list:
        """len(uniforms) chained sampled steps from `token`, one uniform draw per step."""
        n = len(uniforms)
        u = (C.c_float * n)(*[float(x) for x in uniforms])
        buf = (C.c_int64 * n)()
        check(self.L.ptm_decode_sample(self.h, token, n, u, buf), "decode_sample")
        return list(buf)

    def greedy(self, first_token: int, n: int) -> list:
        buf = (C.c_int64 * n)()
        check(self.L.ptm_decode_greedy(self.h, first_token, n, buf), "decode_greedy")
        return list(buf)

    def logits(self) -> np.ndarray:
        """Logits of the last step or of the last prompt token."""
        out = np.empty(self.cfg["vocab"], np.float32)
        check(self.L.ptm_decode_read_logits(self.h, out.ctypes.data), "decode_read_logits")
        return out

    @property
    def layer_runs(self) -> int:
        return self.L.ptm_decode_layer_runs(self.h)


class LoadedModel(Stepper):
    """A model opened by ptm_model_load* (self.m owns the decoder)."""

    def _adopt(self, m, path: str) -> DecodeConfig:
        self.m = m
        self._path = path
        self.h = self.L.ptm_model_decoder(m)
        c = DecodeConfig()
        check(self.L.ptm_model_config(m, C.byref(c)), "model_config")
        return c

    def close(self) -> None:
        if getattr(self, "m", None):
            self.L.ptm_model_free(self.m)
            self.m = None
            self.h = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass


class FolderModel(LoadedModel):
    """A model folder: bfloat16 weights, layers described one by one by config.json."""

    def __init__(self, path: str, max_seq: int, precision: str = "bfloat16", use_graph: bool = True):
        self.L = _lib.load()
        m = C.c_void_p()
        check(self.L.ptm_model_load(path.encode(), max_seq, PRECISIONS[precision], int(use_graph), C.byref(m)),
              f"model_load({path})")
        c = self._adopt(m, path)
        self.cfg = {"vocab": c.vocab, "hidden": c.hidden, "n_layers": c.n_layers, "max_seq": c.max_seq, "eps": c.rms_eps,
                    "precision": precision}

    def prefill_trace(self, tokens) -> np.ndarray:
        """prefill() in one chunk; returns the residual rows after every layer run: [layer runs, tokens, hidden]."""
        n = len(tokens)
        buf = (C.c_int32 * n)(*[int(t) for t in tokens])
        trace = np.empty((self.layer_runs, n, self.cfg["hidden"]), np.float32)
        nxt = C.c_int64()
        check(self.L.ptm_decode_prefill_trace(self.h, buf, n, C.byref(nxt), trace.ctypes.data), "decode_prefill_trace")
        return trace

    def step_trace(self, token: int):
        """One step as plain launches: (next token, residual after every layer run's mixer branch and at its end
        [layer runs, 2, hidden])."""
        import torch
        trace = torch.empty(self.layer_runs, 2, self.cfg["hidden"], dtype=torch.float32, device="cuda")
        torch.cuda.synchronize()
        out = C.c_int64()
        check(self.L.ptm_decode_step_trace(self.h, token, C.byref(out), trace.data_ptr()), "decode_step_trace")
        return out.value, trace.cpu().numpy()


def load(path: str, max_seq: int, precision: str = "bfloat16", use_graph: bool = True):
    """Open any model: a folder by its config.json, or a .gguf file (precision then chooses the fp16 or the fp32 cache)."""
    if precision not in PRECISIONS:
        raise ValueError("precision %r: one of %s" % (precision, ", ".join(PRECISIONS)))
    if os.path.isdir(path):
        return FolderModel(path, max_seq, precision, use_graph)
    from .gguf import GGUFModel
    return GGUFModel(path, max_seq, kv_fp16=precision == "bfloat16", use_graph=use_graph)
