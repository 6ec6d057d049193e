"""GPU: Nadozen models through the framework's decoder against the plain oracle - mechanism by mechanism, layer by layer, whole
prompts, portions, token by token, states used again, window edges, sinks, long contexts, generation - and the attention kernel's
sinks and gates by themselves."""
import ctypes as C

import numpy as np
import pytest

from folder_helpers import errors, portions
from nadozen_models import MODELS, model, parallel, random_model, variant, wkv
from oracle import nadozen_oracle as N
from prometorch_amd import _lib, model as registry, ops
from prometorch_amd.testing import folder_writer as fw

pytestmark = pytest.mark.gpu
# rms error of a position's logits over their deviation: (worst, 97th percentile, mean)
LIMITS = {"float32": (2e-4, 5e-5, 2e-5), "bfloat16": (0.2, 0.06, 0.02)}


def assert_close(got, want, precision, what=""):
    e = errors(got, want)
    worst, most, mean = LIMITS[precision]
    assert e.max() < worst and np.quantile(e, 0.97) < most and e.mean() < mean, (what, e.max(), np.quantile(e, 0.97), e.mean(), int(e.argmax()))


@pytest.fixture(scope="module")
def built(tmp_path_factory):
    """name -> (folder, cfg, weights, tokens, oracle logits at every position), made once."""
    cache = {}

    def get(name, n=150, seed=13):
        if name not in cache:
            cfg = MODELS[name]
            w = fw.random_weights(cfg, seed)
            path = fw.write_model_folder(str(tmp_path_factory.mktemp(name)), cfg, w)
            tokens = np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()
            cache[name] = (path, cfg, w, tokens, N.logits(tokens, w, cfg))
        return cache[name]
    return get


# ---- models -----------------------------------------------------------------------------------------
@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MODELS))
def test_prompt_portions_and_decode(dev, built, name, precision):
    path, cfg, w, tokens, want = built(name)
    m = registry.load(path, max_seq=160, precision=precision)
    assert m.layer_runs == len(cfg["layers"]) and m.cfg["vocab"] == cfg["vocab"]
    for sizes in ([len(tokens)], [2], [1], [7, 1, 1, 3, 2, 64, 5, 1, 31], [64], [66, 1], [1, 149]):
        assert_close(portions(m, tokens, sizes), want, precision, (name, sizes))
    m.close()


@pytest.mark.parametrize("seed", range(24))
def test_random_designs(dev, tmp_path, seed):
    cfg = random_model(seed)
    w = fw.random_weights(cfg, seed + 200)
    tokens = np.random.default_rng(seed).integers(0, cfg["vocab"], 170).tolist()
    want = N.logits(tokens, w, cfg)
    path = fw.write_model_folder(str(tmp_path / "m"), cfg, w)
    for precision in ("float32", "bfloat16"):
        m = registry.load(path, max_seq=171, precision=precision)
        for sizes in ([170], [97, 2, 1, 1, 1, 33, 1], [1]):
            assert_close(portions(m, tokens, sizes), want, precision, (seed, precision, sizes))
        m.close()


@pytest.mark.parametrize("name", sorted(MODELS))
def test_layers_one_by_one(dev, built, name):
    """Sum of the streams after every layer, prompt pass and decode step, in 32-bit."""
    path, cfg, w, tokens, _ = built(name)
    tokens = tokens[:40]
    want = N.residuals(tokens, w, cfg)
    m = registry.load(path, max_seq=64, precision="float32")
    scale = want.std(axis=(1, 2), keepdims=True)
    assert (np.abs(m.prefill_trace(tokens) - want) / scale).max() < 2e-4
    m.set_past_len(0)
    for i, t in enumerate(tokens):
        _, trace = m.step_trace(t)
        assert (np.abs(trace[:, 1] - want[:, i]) / scale[:, 0]).max() < 2e-4, i
    m.close()


# ---- mechanisms by themselves ---------------------------------------------------------------------------
def silent(*names):
    """Weights of the named matrices set to zero: what they carry is out of the model."""
    def change(w):
        for n in names:
            w[n] = np.zeros_like(w[n])
    return change


def loud_keys(w):
    """No decay to speak of, so that the first token still shows hundreds of tokens later."""
    w["l0.mix.w0"] = np.full_like(w["l0.mix.w0"], -9.0)
    w["l0.mix.w2"] = np.zeros_like(w["l0.mix.w2"])


def long_memory(w):
    w["l0.mix.right.dt_bias"] = np.full_like(w["l0.mix.right.dt_bias"], -4.0)
    w["l0.mix.right.A_log"] = np.full_like(w["l0.mix.right.A_log"], -4.0)


ONE_LAYER = parallel(4, 2, 24, 20, (4, 12, 20, 2, 4, 2))
MECHANISMS = {
    # embedding, sinusoid, final norm and head: the only layer writes nothing
    "embedding": ([wkv(2, 8, 4)], 1, silent("l0.mix.o")),
    # blends of the streams without any branch
    "streams": ([wkv(2, 8, 4), wkv(2, 8, 4)], 3, silent("l0.mix.o", "l1.mix.o")),
    "feed_forward": ([wkv(2, 8, 4, ff=43)], 1, silent("l0.mix.o")),
    "wkv": ([wkv(3, 24, 10)], 1, None),
    "wkv_undecayed": ([wkv(3, 24, 10)], 2, loud_keys),
    # no key, no value from the state: only the current token's bonus
    "wkv_bonus": ([wkv(3, 24, 10)], 1, lambda w: w.update({"l0.mix.w0": np.full_like(w["l0.mix.w0"], 6.0)})),
    "attention": ([ONE_LAYER], 1, silent("l0.mix.right.o")),
    "attention_one_gate": ([ONE_LAYER], 1, silent("l0.mix.right.o", "l0.mix.left.g")),
    "state_space": ([ONE_LAYER], 1, silent("l0.mix.left.o")),
    "state_space_long": ([ONE_LAYER], 1, lambda w: (silent("l0.mix.left.o")(w), long_memory(w))),
    # state without decay per step and without the skip
    "state_space_no_skip": ([ONE_LAYER], 1, silent("l0.mix.left.o", "l0.mix.right.D")),
    "shared": ([ONE_LAYER, 0, 0], 2, None),
}


@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism(dev, tmp_path, name):
    layers, streams, change = MECHANISMS[name]
    cfg = model(layers, 50, 70, streams)
    w = fw.random_weights(cfg, 31)
    if change:
        change(w)
        w = {k: fw.from_bf16(fw.to_bf16(v)) for k, v in w.items()}
    tokens = np.random.default_rng(3).integers(0, 70, 260).tolist()
    want = N.logits(tokens, w, cfg)
    path = fw.write_model_folder(str(tmp_path / "m"), cfg, w)
    for precision in ("float32", "bfloat16"):
        m = registry.load(path, max_seq=261, precision=precision)
        for sizes in ([260], [130, 1], [1], [17, 2, 3]):
            assert_close(portions(m, tokens, sizes), want, precision, (name, precision, sizes))
        m.close()


def standing_key(window, width=64):
    """One attention layer in which token 1 looks for token 0 and nothing else stands out: the queries read the input with its
    halves swapped, and token 1 is token 0 with its halves swapped."""
    cfg = model([parallel(2, 1, 32, window, (1, 8, 4, 1, 2, 1), sharp=2.0)], width, 40, 1)
    w = fw.random_weights(cfg, 5)
    w["embed"] = fw.from_bf16(fw.to_bf16(w["embed"] * 8.0))
    w["embed"][1] = np.roll(w["embed"][0], width // 2)
    w["l0.norm1"], w["l0.norm1.b"] = np.ones(width, np.float32), np.zeros(width, np.float32)
    k = np.roll(w["l0.mix.left.k"], width // 2, axis=1)
    w["l0.mix.left.q"] = np.concatenate([k, k])
    w["l0.mix.left.q.norm"] = w["l0.mix.left.k.norm"] = np.ones(32, np.float32)
    w["l0.mix.left.o"] = w["l0.mix.left.o"] * 32.0
    return cfg, w


@pytest.mark.parametrize("window", [3, 64, 65, 100, 128])
def test_keys_at_the_window_edge(dev, tmp_path, window):
    """A key that takes most of the softmax, the window's last position or one further back, at several places relative to
    tiles and portions, in prompts and decoded."""
    cfg, w = standing_key(window)
    path = fw.write_model_folder(str(tmp_path / "m"), cfg, w)
    rng = np.random.default_rng(window)
    for precision in ("float32", "bfloat16"):
        m = registry.load(path, max_seq=400, precision=precision)
        for at in (0, 1, 62, 63, 64, 129):
            tokens = rng.integers(2, 40, at + window + 6)
            tokens[at] = 0
            tokens[at + window - 1:at + window + 1] = 1  # the first still sees token 0, the second does not
            tokens = tokens.tolist()
            want = N.logits(tokens, w, cfg)
            near = [N.logits(tokens, w, variant(cfg, 0, d)) for d in (1, -1)]
            inside, outside = at + window - 1, at + window
            assert errors(near[1], want)[inside] > 0.4 and errors(near[0], want)[outside] > 0.4
            for sizes in ([len(tokens)], [at + window - 1, 1], [at + window, 2], [5]):
                assert_close(portions(m, tokens, sizes)[-9:], want[-9:], precision, (window, at, sizes))
        m.close()


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
def test_window_neighbours(dev, built, precision):
    path, cfg, w, tokens, want = built("odd")
    m = registry.load(path, max_seq=160, precision=precision)
    for sizes in ([150], [1], [9]):
        got = portions(m, tokens, sizes)
        mine = errors(got, want)[50:].mean()
        for delta in (1, -1):
            other = errors(got, N.logits(tokens, w, variant(cfg, 1, delta)))[50:].mean()
            assert other > (1000 if precision == "float32" else 5) * mine, (delta, other, mine)
    m.close()


@pytest.mark.parametrize("sink", [-30.0, 4.0, 30.0])
def test_sinks(dev, tmp_path, sink):
    """From no weight at all to nearly all of it; also where the window holds the first token only."""
    cfg = model([parallel(3, 1, 16, 5, (2, 4, 3, 1, 2, 1))], 30, 31, 1)
    w = fw.random_weights(cfg, 8)
    w["l0.mix.left.sink"] = np.array([sink, 0.0, -sink], np.float32)
    w["l0.mix.left.o"] = fw.from_bf16(fw.to_bf16(w["l0.mix.left.o"] * 4.0))
    tokens = np.random.default_rng(1).integers(0, 31, 40).tolist()
    want = N.logits(tokens, w, cfg)
    path = fw.write_model_folder(str(tmp_path / "m"), cfg, w)
    for precision in ("float32", "bfloat16"):
        m = registry.load(path, max_seq=41, precision=precision)
        for sizes in ([40], [1]):
            assert_close(portions(m, tokens, sizes), want, precision, sizes)
        m.close()


# ---- state over time ----------------------------------------------------------------------------------
@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "whole"])
def test_state_is_used_again(dev, built, precision, name):
    """A second request over the first one's caches and states, shorter and longer, gives what a fresh model gives."""
    path, cfg, w, tokens, want = built(name)
    m = registry.load(path, max_seq=160, precision=precision)
    portions(m, tokens[::-1], [150])
    a = portions(m, tokens[:30], [12, 1, 1, 16])
    portions(m, tokens[::-1], [70, 1])
    b = portions(m, tokens, [100, 1])
    c = portions(m, tokens, [1, 2, 1])
    m.close()
    fresh = registry.load(path, max_seq=160, precision=precision)
    assert np.array_equal(a, portions(fresh, tokens[:30], [12, 1, 1, 16]))
    assert np.array_equal(b, portions(fresh, tokens, [100, 1]))
    assert np.array_equal(c, portions(fresh, tokens, [1, 2, 1]))
    assert_close(b, want, precision)
    fresh.close()


def test_state_does_not_go_back(dev, built):
    """Recurrent state starts over or goes on; a place in between is refused and leaves everything as it is."""
    path, cfg, w, tokens, want = built("odd")
    m = registry.load(path, max_seq=160, precision="float32")
    m.prefill(tokens[:20])
    for place in (19, 1, 21):
        with pytest.raises(_lib.PtmError):
            m.set_past_len(place)
    m.set_past_len(20)
    m.step(tokens[20])
    assert errors(m.logits()[None], want[20:21])[0] < LIMITS["float32"][0]
    m.close()


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
def test_eager_steps_equal_graph_steps(dev, built, precision):
    path, cfg, w, tokens, _ = built("odd")
    a = registry.load(path, max_seq=160, precision=precision, use_graph=True)
    b = registry.load(path, max_seq=160, precision=precision, use_graph=False)
    ya, yb = portions(a, tokens[:60], [20, 1]), portions(b, tokens[:60], [20, 1])
    assert np.array_equal(ya, yb)
    assert a.L.ptm_decode_graph_state(a.h, 0) == 1 and b.L.ptm_decode_graph_state(b.h, 0) == 0
    a.close()
    b.close()


def test_long_prompts_and_decoding(dev, tmp_path):
    """Prompts of several chunks and hundreds of decoded tokens, with states that forget slowly."""
    cfg = model([wkv(2, 12, 4), parallel(2, 1, 12, 300, (2, 8, 6, 1, 4, 1)), 0], 24, 40, 2)
    w = fw.random_weights(cfg, 17)
    loud_keys(w)
    w = {k: fw.from_bf16(fw.to_bf16(v)) for k, v in w.items()}
    tokens = np.random.default_rng(5).integers(0, 40, 2900).tolist()
    want = N.logits(tokens, w, cfg)
    path = fw.write_model_folder(str(tmp_path / "m"), cfg, w)
    for precision in ("float32", "bfloat16"):
        m = registry.load(path, max_seq=2900, precision=precision)
        got = [m.prefill_logits(tokens[:2300], range(2200, 2300))]
        for t in tokens[2300:]:
            m.step(t)
            got.append(m.logits()[None])
        assert_close(np.concatenate(got), want[2200:], precision)
        m.set_past_len(0)
        assert_close(m.prefill_logits(tokens, range(2880, 2900), chunk_rows=700), want[2880:], precision)
        m.close()


# ---- generation ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
def test_greedy_generation(dev, built, precision):
    """Greedy tokens through prefill + greedy and through generate(); every token is the oracle's best on that very text, or within
    rounding of it.  A stop token inside a run leaves the state where the text ends."""
    path, cfg, w, tokens, _ = built("odd")
    prompt, n = tokens[:23], 60
    m = registry.load(path, max_seq=160, precision=precision)
    first = m.prefill(prompt)
    out = [first] + m.greedy(first, n - 1)
    m.set_past_len(0)
    kw = dict(temperature=0.0, top_k=1, top_p=1.0)
    assert m.generate(prompt, [0.5] * n, **kw) == out
    lg = N.logits(prompt + out, w, cfg)
    lg, after = lg[len(prompt) - 1:-1], lg[len(prompt):]
    gap = (lg.max(axis=1) - lg[np.arange(n), out]) / lg.std()
    assert gap.max() < LIMITS[precision][0], gap.max()
    if precision == "float32":
        assert gap.max() == 0.0
    for stop in sorted(set(out), key=out.index)[1::4]:
        cut = out.index(stop)
        m.set_past_len(0)
        assert m.generate(prompt, [0.5] * n, stop_ids=[stop], **kw) == out[:cut]
        m.step(stop)  # the text goes on behind the stop token
        assert errors(m.logits()[None], after[cut:cut + 1])[0] < LIMITS[precision][0], cut
    m.close()


def test_command_line(dev, built, capsys):
    """Token ids in, the same greedy ids out as through the Python interface."""
    from prometorch_amd.__main__ import main
    path, cfg, w, tokens, _ = built("whole")
    m = registry.load(path, max_seq=64)
    want = m.generate(tokens[:9], [0.0] * 12, temperature=0.0, top_k=1, top_p=1.0)
    m.close()
    args = ["generate", "--model", path, "--tokens", ",".join(map(str, tokens[:9])), "--max-new", "12", "--temperature", "0"]
    assert main(args) == 0
    assert capsys.readouterr().out.split() == [str(t) for t in want]


def test_sampled_generation(dev, built):
    """The same draws give the same tokens again, picked from the logits a stepped run reads back."""
    path, cfg, w, tokens, _ = built("odd")
    m = registry.load(path, max_seq=160, precision="bfloat16")
    u = ops.mt19937_uniforms(7, 0, 30)
    kw = dict(temperature=0.8, top_k=12, top_p=0.9)
    a = m.generate(tokens[:10], u, **kw)
    m.set_past_len(0)
    assert m.generate(tokens[:10], u, **kw) == a and len(set(a)) > 3
    m.set_past_len(0)
    m.prefill(tokens[:9])
    t = tokens[9]
    for i in range(30):
        m.step(t)
        lg = m.logits().astype(np.float64) / kw["temperature"]
        top = np.argsort(-lg, kind="stable")[:12]
        p = np.exp(lg[top] - lg[top].max())
        p /= p.sum()
        assert a[i] in top[:int((np.cumsum(p) < 0.9).sum()) + 1], i
        t = a[i]
    m.close()


def test_folder_errors_on_load(dev, built, tmp_path):
    path, cfg, w, _, _ = built("odd")
    for name in ("l0.mix.mu.w", "l1.mix.left.sink", "l1.mix.right.conv.b", "l1.hc2.mix", "l3.norm1.b", "final.norm.b", "l0.mix.w1"):
        with pytest.raises(_lib.PtmError) as e:
            registry.load(fw.write_model_folder(str(tmp_path / "missing"), cfg, {k: v for k, v in w.items() if k != name}), max_seq=16)
        assert e.value.code == -10, name
    for name in ("l0.mix.w2", "l1.mix.right.in", "l0.mix.u", "l1.hc1.in"):
        with pytest.raises(_lib.PtmError) as e:
            registry.load(fw.write_model_folder(str(tmp_path / "shape"), cfg, dict(w, **{name: w[name][:-1]})), max_seq=16)
        assert e.value.code == -2, name
    m = registry.load(path, max_seq=16)
    with pytest.raises(_lib.PtmError):
        m.prefill([0] * 17)          # past the cache
    m.close()


# ---- attention kernel: sinks, output gate, scale ------------------------------------------------------------
@pytest.mark.parametrize("fp32", [False, True])
@pytest.mark.parametrize("case", [(5, 4, 2, 16, 0, 0), (70, 3, 1, 64, 20, 130), (130, 2, 2, 120, 64, 5), (33, 6, 3, 200, 7, 64), (9, 2, 1, 272, 4, 3)])
def test_attention_rows_sink_and_gate(dev, case, fp32):
    """rows, heads, kv heads, size, window, position of row 0; three values per head are outside the gate's columns."""
    import torch
    rows, H, G, d, window, pos0 = case
    rng = np.random.default_rng(sum(case))
    n = pos0 + rows
    rnd = (lambda *s: rng.standard_normal(s, np.float32)) if fp32 else (lambda *s: fw.from_bf16(fw.to_bf16(rng.standard_normal(s, np.float32))))
    q, k, v = rnd(rows, H, d), rnd(n, G, d), rnd(n, G, d)
    gate = rng.standard_normal((rows, H, d - 3), np.float32)
    sink = rng.standard_normal(H).astype(np.float32) * 2 + 1
    scale, see = 2.0 / np.sqrt(d), N.visible(n, {"size": window} if window else None)[pos0:]
    want = np.zeros((rows, H, d))
    for h in range(H):
        g = h // (H // G)
        s = np.where(see, q[:, h].astype(np.float64) @ k[:, g].T.astype(np.float64) * scale, -np.inf)
        want[:, h] = N.sink_softmax(s, float(sink[h])) @ v[:, g] * 0.7
        want[:, h, :d - 3] *= N.sigmoid(gate[:, h].astype(np.float64))
    put = lambda a: torch.from_numpy(a if fp32 else fw.to_bf16(a).view(np.int16)).cuda()
    Q, K, V = put(q), put(k), put(v)
    O = torch.zeros((rows, H, d), dtype=torch.float32 if fp32 else torch.bfloat16, device="cuda")
    S, Gt = torch.from_numpy(sink).cuda(), torch.from_numpy(gate).cuda()
    a = _lib.AttentionArgs(Q=Q.data_ptr(), K1=K.data_ptr(), V=V.data_ptr(), O=O.data_ptr(), q_row=H * d, k1_row=G * d, k1_head=d,
                           v_row=G * d, v_head=d, o_row=H * d, rows=rows, heads=H, kv_heads=G, dim1=d, vdim=d, window=window, pos0=pos0,
                           scale=scale, fp32=int(fp32), sink=S.data_ptr(), gate=Gt.data_ptr(), gate_row=H * (d - 3), gate_head=d - 3,
                           out_scale=0.7)
    _lib.check(_lib.load().ptm_attention_rows(C.byref(a), None), "attention_rows")
    torch.cuda.synchronize()
    err = np.abs(O.float().cpu().numpy() - want)
    assert err.max() < (2e-5 if fp32 else 2.5e-2), err.max()


# ---- products with the gated epilogue are reached through the models; shapes around their tile edges -------------
@pytest.mark.parametrize("ff", [1, 15, 16, 17, 64, 100, 257])
def test_feed_forward_sizes(dev, tmp_path, ff):
    cfg = model([wkv(1, 8, 3, ff=ff)], 40, 33, 1)
    w = fw.random_weights(cfg, ff)
    silent("l0.mix.o")(w)
    w["l0.mlp.down"] = fw.from_bf16(fw.to_bf16(w["l0.mlp.down"] * 3.0))
    tokens = np.random.default_rng(ff).integers(0, 33, 140).tolist()
    want = N.logits(tokens, w, cfg)
    path = fw.write_model_folder(str(tmp_path / "m"), cfg, w)
    for precision in ("float32", "bfloat16"):
        m = registry.load(path, max_seq=141, precision=precision)
        for sizes in ([140], [50, 20, 1]):
            assert_close(portions(m, tokens, sizes), want, precision, (ff, sizes))
        m.close()
