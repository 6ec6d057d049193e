"""CPU: the Nadozen oracle against closed forms and itself, what the registry refuses, and the changes that the GPU tests rely on."""
import copy
import json

import numpy as np
import pytest

from nadozen_models import MODELS, model, parallel, random_model, variant, wkv
from oracle import nadozen_oracle as N
from prometorch_amd import _lib, model as registry
from prometorch_amd._lib import PtmError
from prometorch_amd.testing import folder_writer as fw

E_NULL, E_SHAPE, E_STATE, E_UNSUP, E_FORMAT = -1, -2, -5, -4, -9


# ---- oracle ---------------------------------------------------------------------------------------
def test_wkv_recurrence_equals_the_sum_over_pairs():
    """o_t = sum over j < t of (r_t . (decays between j and t) k_j) v_j, plus the bonus at t."""
    cfg = model([wkv(2, 5, 3)], 16, 10, 1)
    w = {k: v.astype(np.float64) for k, v in fw.random_weights(cfg, 1).items()}
    x, m, p = np.random.default_rng(0).standard_normal((9, 16)), cfg["layers"][0]["mixer"], "l0.mix."
    before = np.vstack([np.zeros((1, 16)), x[:-1]])
    mixed = {s: x + (before - x) * w[p + "mu." + s] for s in "rkvgw"}
    r, k, v = ((mixed[s] @ w[p + s].T).reshape(9, 2, 5) for s in "rkv")
    rate = np.exp(np.tanh(mixed["w"] @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]).reshape(9, 2, 5)
    o = np.zeros((9, 2, 5))
    for t in range(9):
        for a in range(2):
            for j in range(t):
                o[t, a] += (r[t, a] * k[j, a] * np.exp(-rate[j + 1:t, a].sum(axis=0))).sum() * v[j, a]
            o[t, a] += (r[t, a] * w[p + "u"][a] * k[t, a]).sum() * v[t, a]
    g = mixed["g"] @ w[p + "g"].T
    want = (N.rms(o, 1e-5).reshape(9, 10) * w[p + "norm"] * g / (1 + np.exp(-g))) @ w[p + "o"].T
    assert np.allclose(N.wkv(x, w, p, m, 1e-5), want, atol=1e-10)


def test_state_space_recurrence_equals_the_sum_over_pairs():
    cfg = model([parallel(2, 1, 4, 3, (4, 3, 5, 2, 3, 2))], 16, 10, 1)
    w = {k: v.astype(np.float64) for k, v in fw.random_weights(cfg, 2).items()}
    x, m, p = np.random.default_rng(1).standard_normal((8, 16)), cfg["layers"][0]["mixer"]["right"], "l0.mix.right."
    proj = x @ w[p + "in"].T
    z, xbc, dt = proj[:, :12], proj[:, 12:44], np.log1p(np.exp(proj[:, 44:] + w[p + "dt_bias"]))
    conv = np.zeros_like(xbc)
    for t in range(8):
        for j in range(min(t, 2) + 1):
            conv[t] += w[p + "conv"][:, 2 - j] * xbc[t - j]
    conv = conv + w[p + "conv.b"]
    conv = conv / (1 + np.exp(-conv))
    X, B, C = conv[:, :12].reshape(8, 4, 3), conv[:, 12:22].reshape(8, 2, 5), conv[:, 22:].reshape(8, 2, 5)
    y = X * w[p + "D"][None, :, None]
    for t in range(8):
        for a in range(4):
            for j in range(t + 1):
                y[t, a] += np.exp(-np.exp(w[p + "A_log"][a]) * dt[j + 1:t + 1, a].sum()) * dt[j, a] * (B[j, a // 2] @ C[t, a // 2]) * X[j, a]
    y = (y.reshape(8, 12) * z / (1 + np.exp(-z))).reshape(8, 2, 6)
    want = (N.rms(y, 1e-5).reshape(8, 12) * w[p + "norm"]) @ w[p + "o"].T
    assert np.allclose(N.ssm(x, w, p, m, 1e-5), want, atol=1e-10)


def test_layer_norm_sinusoid_and_sink():
    x = np.random.default_rng(2).standard_normal((3, 7)) * 4 + 2
    y = N.layer_norm(x, np.ones(7), np.zeros(7), 1e-6)
    assert np.allclose(y.mean(axis=1), 0) and np.allclose(y.var(axis=1), 1, atol=1e-5)
    s = N.sinusoid([0, 3], 5)
    assert s[0].tolist() == [0, 1, 0, 1, 0] and np.isclose(s[1, 0], np.sin(3.0)) and np.isclose(s[1, 3], np.cos(3.0 * 10000 ** -0.4))
    p = N.sink_softmax(np.array([[0.0, 0.0, -np.inf]]), np.log(2.0))
    assert np.allclose(p, [[0.25, 0.25, 0.0]])
    assert N.visible(6, {"size": 2}).sum(axis=1).tolist() == [1, 2, 2, 2, 2, 2]


def test_one_plain_stream_is_a_residual():
    w = {"in": np.ones(1), "out": np.ones(1), "mix": np.ones((1, 1))}
    x = np.random.default_rng(3).standard_normal((1, 4, 6))
    assert np.allclose(N.hyper_connect(x, w, "", lambda u: 2 * u), 3 * x)
    # from stream 0 to stream 1 only
    w = {"in": np.array([1.0, 0.0]), "out": np.array([0.0, 1.0]), "mix": np.array([[0.0, 1.0], [0.0, 0.0]])}
    x = np.random.default_rng(4).standard_normal((2, 4, 6))
    y = N.hyper_connect(x, w, "", lambda u: 5 * u)
    assert np.allclose(y[0], 0) and np.allclose(y[1], 6 * x[0])


@pytest.mark.parametrize("name", sorted(MODELS))
def test_oracle_is_causal(name):
    cfg = MODELS[name]
    w = fw.random_weights(cfg, 3)
    tokens = np.random.default_rng(0).integers(0, cfg["vocab"], 40)
    full = N.logits(tokens, w, cfg)
    assert np.isfinite(full).all() and np.allclose(full[:23], N.logits(tokens[:23], w, cfg), atol=1e-9)
    changed = tokens.copy()
    changed[10] = (changed[10] + 1) % cfg["vocab"]
    moved = np.abs(N.logits(changed, w, cfg) - full).max(axis=1)
    assert (moved[:10] < 1e-9).all() and moved[10] > 1e-3


def test_shared_weights():
    cfg = MODELS["odd"]
    assert [N.owner(cfg, i) for i in range(7)] == [0, 1, 0, 3, 1, 5, 3]
    shapes = fw.tensor_shapes(cfg)
    assert not any(n.startswith(("l2.", "l4.", "l6.")) for n in shapes) and "l0.hc2.mix" in shapes and "l3.hc2.mix" not in shapes


def test_window_variants_differ():
    cfg = MODELS["odd"]
    w = fw.random_weights(cfg, 13)
    tokens = np.random.default_rng(13).integers(0, cfg["vocab"], 80)
    base = N.logits(tokens, w, cfg)
    for d in (1, -1):
        assert np.sqrt(((N.logits(tokens, w, variant(cfg, 1, d)) - base)[30:] ** 2).mean()) > 0.05 * base.std()


def test_random_models_are_consistent():
    for seed in range(40):
        cfg = random_model(seed)
        for i, L in enumerate(cfg["layers"]):
            if L.get("weights_of") is not None:
                assert {k: v for k, v in L.items() if k != "weights_of"} == cfg["layers"][N.owner(cfg, i)]
        assert fw.tensor_shapes(cfg)


# ---- registry and host-side validation -------------------------------------------------------------
def folder_error(tmp_path, cfg):
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    fw.write_safetensors(str(tmp_path / "model.safetensors"), {"x": np.zeros(4, np.float32)})
    with pytest.raises(PtmError) as e:
        registry.load(str(tmp_path), max_seq=8)
    return e.value.code


def test_registry_refuses_broken_configurations(tmp_path):
    cfg = MODELS["odd"]
    for broken in ({"layers": []}, {"vocab": 0}, {"norm": {}}, {"streams": 0}, {"streams": None}, {"width": 7.5}, {"logit_scale": None},
                   {"logit_scale": 0}):
        assert folder_error(tmp_path, {**copy.deepcopy(cfg), **broken}) == E_FORMAT, broken


def test_block_validation_codes():
    """Sizes and pointers are checked on the host before anything is allocated or launched."""
    import ctypes as C
    L = _lib.load()

    def mat(rows, cols):
        return _lib.QWeight(data=1 << 12, ggml_type=30, rows=rows, cols=cols, row_stride_bytes=2 * L.ptm_dense_cols(cols))

    host = (C.c_float * 16)()
    hc = (C.c_void_p * 2)(C.addressof(host), C.addressof(host))

    def code(block=(), **config):
        b = _lib.Block(mixer=2, norm1=1 << 12, out=mat(32, 24), in_=mat(4 * 24 + 5, 32), hc_in=hc, hc_out=hc, hc_mix=hc,
                       wkv=_lib.Wkv(heads=3, dim=8, rank=5, mu=1 << 12, w2=mat(24, 5), w0=1 << 12, u=1 << 12, norm=1 << 12))
        for k, v in dict(block).items():
            setattr(b, k, v)
        c = _lib.BlockConfig(vocab=20, hidden=32, n_blocks=1, max_seq=16, eps=1e-5, blocks=C.pointer(b), embedding=mat(20, 32),
                             lm_head=mat(20, 32), out_norm=1 << 12, streams=2)
        for k, v in config.items():
            setattr(c, k, v)
        h = C.c_void_p()
        return L.ptm_decode_create_blocks(C.byref(c), C.byref(h))

    w = lambda **kw: _lib.Wkv(**{**dict(heads=3, dim=8, rank=5, mu=1 << 12, w2=mat(24, 5), w0=1 << 12, u=1 << 12, norm=1 << 12), **kw})
    assert code(streams=0) == E_UNSUP                                   # recurrent mixers live behind streams
    assert code(streams=17) == E_UNSUP and code(streams=-1) == E_SHAPE
    assert code(loop_times=2, loop_stop=1, loop_step=1 << 12) == E_UNSUP
    assert code({"norm1b": 1 << 12}) == E_UNSUP                         # no post-norm
    assert code({"wkv": w(dim=600, w2=mat(1800, 5))}) == E_UNSUP        # beyond the state's tile classes
    assert code({"wkv": w(rank=0)}) == E_SHAPE and code({"wkv": w(u=None)}) == E_NULL
    assert code({"wkv": w(w2=mat(24, 6))}) == E_SHAPE
    assert code({"in_": mat(4 * 24 + 6, 32)}) == E_SHAPE
    assert code({"hc_mix": (C.c_void_p * 2)()}) == E_NULL
    assert code({"ff": 8, "norm2": 1 << 12, "ff_kind": 1, "up": mat(8, 32), "down": mat(32, 8)}) == E_SHAPE   # gate rows missing
    assert code({"ff_kind": 2}) == E_UNSUP and code({"head_norm": 1}) == E_UNSUP
    ssm = dict(heads=4, vdim=3, state=5, groups=2, taps=3, norm_groups=2, **{n: 1 << 12 for n in ("conv", "conv_b", "dt_bias", "neg_a", "D", "norm")})
    att = dict(mixer=0, heads=2, kv_heads=1, dim=8, vdim=8, q_norm=1 << 12, k_norm=1 << 12, values_are_keys=1, out_gate=1)
    rows = 16 + 8 + 16 + 12 + (12 + 20) + 4
    assert code({**att, "ssm": _lib.Ssm(**{**ssm, "groups": 3}), "in_": mat(rows, 32)}) == E_SHAPE
    assert code({**att, "ssm": _lib.Ssm(**{**ssm, "norm_groups": 5}), "in_": mat(rows, 32)}) == E_SHAPE
    assert code({**att, "ssm": _lib.Ssm(**{**ssm, "D": None}), "in_": mat(rows, 32)}) == E_NULL
    assert code({**att, "ssm": _lib.Ssm(**ssm), "in_": mat(rows + 1, 32)}) == E_SHAPE
    assert code({**att, "vdim": 16, "ssm": _lib.Ssm(**ssm), "in_": mat(rows, 32)}) == E_SHAPE


def test_decode_attention_args_are_checked():
    L = _lib.load()
    import ctypes as C
    a = _lib.AttentionArgs(Q=16, K1=16, V=16, O=16, rows=1, heads=2, kv_heads=2, dim1=8, vdim=8, gate=16)
    assert L.ptm_attention_rows(C.byref(a), None) == E_SHAPE             # a gate without its columns
