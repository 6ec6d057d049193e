"""CPU: the Tovasun oracle against itself (causality, masks), model-folder reading on the host, rotation tables, trace replay
bookkeeping and host-side validation."""
import ctypes as C
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from conftest import ROOT
from oracle import tovasun_oracle as T
from prometorch_amd import _lib, model as registry, trace
from prometorch_amd._lib import PtmError
from prometorch_amd.testing import folder_writer as fw
from tovasun_models import MODELS, YARN, variant

E_NULL, E_SHAPE, E_UNSUP, E_IO, E_FORMAT = -1, -2, -4, -8, -9


# ---- oracle ---------------------------------------------------------------------------------------
def test_oracle_is_causal_and_window_bounded():
    cfg = MODELS["plain"]
    w = fw.random_weights(cfg, 3)
    rng = np.random.default_rng(0)
    tokens = rng.integers(0, cfg["vocab"], 70)
    full = T.logits(tokens, w, cfg)
    assert np.allclose(full[:41], T.logits(tokens[:41], w, cfg), atol=1e-9)
    # two windows of 21 and 30: position i depends on tokens i - 20 - 29 .. i, and on the kept first one
    changed = tokens.copy()
    changed[10] = (changed[10] + 1) % cfg["vocab"]
    moved = np.abs(T.logits(changed, w, cfg) - full).max(axis=1) > 1e-9
    assert moved[10:60].all() and not moved[:10].any() and not moved[60:].any()


def test_oracle_masks_and_rotation():
    see = T.visible(12, {"size": 4, "keep_first": 2})
    assert see[9].tolist() == [True, True] + [False] * 4 + [True] * 4 + [False] * 2
    assert T.visible(5, None).sum() == 15
    x = np.random.default_rng(1).standard_normal((9, 2, 12))
    y = T.rotate(x, np.arange(9), {"base": 100.0, "dims": 8})
    assert np.array_equal(y[..., 8:], x[..., 8:]) and np.allclose(np.linalg.norm(y, axis=-1), np.linalg.norm(x, axis=-1))
    # scores depend on the distance only
    q = np.broadcast_to(x[:1], x.shape)
    r = T.rotate(q, np.arange(9), {"base": 100.0, "dims": 8})
    assert np.isclose((r[3] * r[1]).sum(), (r[8] * r[6]).sum())


def test_oracle_loop_order():
    cfg = MODELS["odd"]
    assert T.layer_runs(cfg) == [(0, None), (1, 0), (2, 0), (1, 1), (2, 1), (3, None)]


# ---- rotation tables --------------------------------------------------------------------------------
@pytest.mark.parametrize("scaling", [None, YARN, {"factor": 40.0, "fast": 32.0, "slow": 1.0, "original": 4096},
                                     {"factor": 1.5, "fast": 2.0, "slow": 2.0, "original": 64}])
def test_rotation_table(scaling):
    dims, n, base = 16, 300, 7000.0
    rot = _lib.Rotation(base=base, dims=dims)
    if scaling:
        rot.factor, rot.original, rot.fast, rot.slow = scaling["factor"], scaling["original"], scaling["fast"], scaling["slow"]
    table = np.empty((n, dims // 2, 2), np.float32)
    L = _lib.load()
    assert L.ptm_rope_pairs_host(table.ctypes.data, n, C.byref(rot)) == 0
    unit = np.zeros((n, 1, dims))
    unit[..., 0::2] = 1.0
    want = T.rotate(unit, np.arange(n), {"base": base, "dims": dims, "scaling": scaling})
    assert np.abs(table[..., 0] - want[:, 0, 0::2]).max() < 2e-7 * 2 and np.abs(table[..., 1] - want[:, 0, 1::2]).max() < 2e-7 * 2
    assert L.ptm_rope_pairs_host(table.ctypes.data, n, C.byref(_lib.Rotation(base=base, dims=7))) == E_SHAPE


# ---- model folders ----------------------------------------------------------------------------------
def open_safetensors(path):
    L = _lib.load()
    h = C.c_void_p()
    return L, h, L.ptm_safetensors_open(str(path).encode(), C.byref(h))


def test_safetensors_reader(tmp_path):
    p = tmp_path / "t.safetensors"
    a = np.arange(12, dtype=np.float32).reshape(3, 4)
    fw.write_safetensors(str(p), {"a é\"x": a, "b": fw.to_bf16(a[0]), "c": np.array([[7]], np.int32)})
    L, h, rc = open_safetensors(p)
    assert rc == 0 and L.ptm_safetensors_n_tensors(h) == 3
    t = _lib.StTensor()
    assert L.ptm_safetensors_find(h, "a é\"x".encode(), C.byref(t)) == 0
    assert t.dtype == b"F32" and list(t.dims[:t.n_dims]) == [3, 4] and t.nbytes == 48
    assert np.array_equal(np.frombuffer(C.string_at(t.data, 48), np.float32), a.ravel())
    assert L.ptm_safetensors_tensor_at(h, 1, C.byref(t)) == 0 and t.name == b"b" and t.dtype == b"BF16"
    assert np.array_equal(fw.from_bf16(np.frombuffer(C.string_at(t.data, 8), np.uint16)), a[0])
    assert L.ptm_safetensors_find(h, b"d", C.byref(t)) < 0 and L.ptm_safetensors_tensor_at(h, 3, C.byref(t)) < 0
    L.ptm_safetensors_close(h)


@pytest.mark.parametrize("damage", ["short", "length", "json", "offsets", "size"])
def test_safetensors_reader_refuses_damaged_files(tmp_path, damage):
    p = tmp_path / "t.safetensors"
    fw.write_safetensors(str(p), {"a": np.zeros((2, 3), np.float32)})
    raw = p.read_bytes()
    if damage == "short":
        raw = raw[:5]
    elif damage == "length":
        raw = b"\xff" * 8 + raw[8:]
    elif damage == "json":
        raw = raw[:8] + b"[" + raw[9:]
    elif damage == "offsets":
        raw = raw[:-1]
    else:
        raw = raw.replace(b"[2, 3]", b"[2, 4]")
    p.write_bytes(raw)
    _, h, rc = open_safetensors(p)
    assert rc == E_FORMAT and not h
    assert open_safetensors(tmp_path / "none")[2] == E_IO


def folder_error(tmp_path, cfg):
    (tmp_path / "config.json").write_text(cfg if isinstance(cfg, str) else json.dumps(cfg))
    if not (tmp_path / "model.safetensors").exists():
        fw.write_safetensors(str(tmp_path / "model.safetensors"), {"x": np.zeros(4, np.float32)})
    with pytest.raises(PtmError) as e:
        registry.load(str(tmp_path), max_seq=8)
    return e.value.code


def test_registry_refuses_what_it_does_not_know(tmp_path):
    with pytest.raises(PtmError) as e:
        registry.load(str(tmp_path), max_seq=8)
    assert e.value.code == E_IO                                   # a folder without config.json
    assert folder_error(tmp_path, "{") == E_FORMAT
    assert folder_error(tmp_path, {"architecture": "Nothing"}) == E_UNSUP
    assert folder_error(tmp_path, {"layers": []}) == E_FORMAT     # no architecture
    cfg = json.loads(json.dumps(MODELS["odd"]))
    for broken in ({"layers": []}, {"vocab": 0}, {"norm": {}}, {"loop": {"start": 2, "stop": 2, "times": 2}}, {"width": 7.5}):
        assert folder_error(tmp_path, {**cfg, **broken}) == E_FORMAT, broken
    with pytest.raises(ValueError):
        registry.load(str(tmp_path), max_seq=8, precision="float16")


def test_validation_codes():
    L = _lib.load()
    assert L.ptm_dense_cols(1) == 64 and L.ptm_dense_cols(128) == 128
    assert L.ptm_dense_gemv(None, 16, 16, 64, 4, 64, None) == E_NULL
    assert L.ptm_dense_gemv(16, 16, 16, 65, 4, 64, None) == E_SHAPE          # rows shorter than the padded width
    assert L.ptm_dense_gemm(16, 0, 64, 16, 64, 16, 8, 2, 8, 65, None) == E_SHAPE
    assert L.ptm_attention_rows(None, None) == E_NULL
    a = _lib.AttentionArgs(Q=16, K1=16, V=16, O=16, rows=1, heads=3, kv_heads=2, dim1=8, vdim=8)
    assert L.ptm_attention_rows(C.byref(a), None) == E_SHAPE                  # heads not a multiple of kv heads
    a = _lib.AttentionArgs(Q=16, K1=16, V=16, O=16, rows=1, heads=2, kv_heads=2, dim1=12, vdim=8)
    assert L.ptm_attention_rows(C.byref(a), None) == -3
    a = _lib.AttentionArgs(Q=16, K1=16, V=16, O=16, rows=1, heads=2, kv_heads=2, dim1=8, vdim=8, pos0=9, kv_pos0=4, window=8)
    assert L.ptm_attention_rows(C.byref(a), None) == -6                       # position 2 is visible and before the array
    h = C.c_void_p()
    assert L.ptm_decode_create_blocks(None, C.byref(h)) == E_NULL
    assert L.ptm_decode_create_blocks(C.byref(_lib.BlockConfig()), C.byref(h)) == E_NULL
    assert L.ptm_decode_prefill_logits(None, None, 1, 0, None, 0, None, None) == E_NULL


# ---- trace replay ------------------------------------------------------------------------------------
class FakeModel:
    """Logits that name (position, token); the calls made."""
    cfg = {"vocab": 3}

    def __init__(self):
        self.past, self.calls = None, []

    def set_past_len(self, n):
        self.past = n

    def _row(self, t):
        self.past += 1
        return np.array([self.past - 1, t, -1], np.float32)

    def step(self, t):
        self.calls.append(1)
        self.last = self._row(t)

    def logits(self):
        return self.last

    def prefill_logits(self, tokens, want):
        self.calls.append(len(tokens))
        rows = [self._row(t) for t in tokens]
        return np.stack([rows[w] for w in want]) if want else np.empty((0, 3), np.float32)

    def close(self):
        self.calls.append("closed")


def test_trace_replay(tmp_path, monkeypatch, capsys):
    fake = FakeModel()
    monkeypatch.setattr(trace.registry, "load", lambda path, max_seq, precision: fake)
    steps = [{"step": 4, "entries": [{"id": "u", "tokens": [8, 9, 7], "want": [2, 0]}], "end": []},
             {"step": 5, "entries": [{"id": "u", "tokens": [6], "want": []}], "end": []},
             {"step": 6, "entries": [{"id": "u", "tokens": [5], "want": [0]}], "end": ["u"]},
             {"step": 7, "entries": [{"id": "v", "tokens": [1, 2], "want": [1]}], "end": ["v"]}]
    monkeypatch.setattr(sys, "stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    assert trace.main(["--model", "m", "--dtype", "float32", "--out", str(tmp_path / "o"), "--max-tokens", "9"]) == 0
    assert capsys.readouterr().out.split("\n")[:4] == ["done 4", "done 5", "done 6", "done 7"]
    read = lambda n: np.fromfile(tmp_path / "o" / ("%d.f32" % n), "<f4").reshape(-1, 3)[:, :2].tolist()
    assert read(4) == [[2, 7], [0, 8]] and read(6) == [[4, 5]] and read(7) == [[1, 2]]
    assert not (tmp_path / "o" / "5.f32").exists() and fake.calls == [3, 1, 1, 2, "closed"]
    replay = trace.Replay(FakeModel())
    replay.run("a", [1], [])
    with pytest.raises(RuntimeError):
        replay.run("b", [1], [])


def test_trace_run_is_executable():
    exe = os.path.join(ROOT, "bin", "trace_run")
    assert os.access(exe, os.X_OK)
    r = subprocess.run([exe, "--help"], capture_output=True, text=True)
    assert r.returncode == 0 and "--max-tokens" in r.stdout


def test_command_line_arguments(monkeypatch, capsys):
    from prometorch_amd import __main__ as cli
    fake = FakeModel()
    fake.generate = lambda prompt, u, temperature, top_k, top_p, repeat_penalty, stop_ids: fake.calls.append(
        (prompt, len(u), temperature, top_k, list(stop_ids))) or [4, 2]
    opened = []
    monkeypatch.setattr(cli.registry, "load", lambda path, max_seq, precision: opened.append((path, max_seq, precision)) or fake)
    assert cli.main(["generate", "--model", "m", "--tokens", "3,1 2", "--max-new", "5", "--top-k", "7", "--stop", "9", "--dtype", "float32"]) == 0
    assert capsys.readouterr().out.split() == ["4", "2"]
    assert opened == [("m", 8, "float32")] and fake.calls == [([3, 1, 2], 5, 0.7, 7, [9]), "closed"]
    for bad in (["generate", "--model", "m"], ["generate", "--model", "m", "--tokens", "a"], ["generate", "--model", "m", "--tokens", ""]):
        with pytest.raises(SystemExit):
            cli.main(bad)


def test_planted_variants_differ():
    """The neighbours of a mask that the GPU tests compare against do change the oracle's logits."""
    cfg = MODELS["plain"]
    w = fw.random_weights(cfg, 5)
    tokens = np.random.default_rng(2).integers(0, cfg["vocab"], 60)
    base = T.logits(tokens, w, cfg)
    for change in ({"l0_size": 1}, {"l0_size": -1}, {"l0_keep_first": 1}, {"l0_keep_first": -1}, {"l1_size": 1}):
        d = T.logits(tokens, w, variant(cfg, **change)) - base
        assert np.sqrt((d[40:] ** 2).mean()) > 0.02 * base.std(), change
