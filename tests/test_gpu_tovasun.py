"""GPU: Tovasun models through the framework's decoder against the plain oracle - layer by layer, whole prompts, portions,
token by token, reused caches, window and kept-token edges, long contexts, generation - and the kernels by themselves."""
import ctypes as C

import numpy as np
import pytest

from folder_helpers import errors, portions
from oracle import tovasun_oracle as T
from prometorch_amd import _lib, model as registry, ops
from prometorch_amd.testing import folder_writer as fw, synth
from tovasun_models import MODELS, attention, latent, layer, model, random_model, variant

pytestmark = pytest.mark.gpu
# rms error of a position's logits over their deviation: (worst, 97th percentile, mean).  bfloat16: where two keys of a sharp
# softmax compete, the rounding of q, k and v moves a few positions a long way; rounding the oracle's own q, k, v and norms gives
# the same positions and the same size (up to 0.16, mean 0.018).
LIMITS = {"float32": (2e-4, 1e-4, 3e-5), "bfloat16": (0.4, 0.1, 0.03)}


def assert_close(got, want, precision, what=""):
    e = errors(got, want)
    worst, most, mean = LIMITS[precision]
    assert e.max() < worst and np.quantile(e, 0.97) < most and e.mean() < mean, (what, e.max(), e.mean(), int(e.argmax()))


@pytest.fixture(scope="module")
def built(tmp_path_factory):
    """name -> (folder, cfg, weights, tokens, oracle logits at every position), made once."""
    cache = {}

    def get(name, n=150, seed=11):
        if name not in cache:
            cfg = MODELS[name]
            w = fw.random_weights(cfg, seed)
            path = fw.write_model_folder(str(tmp_path_factory.mktemp(name)), cfg, w)
            tokens = np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()
            cache[name] = (path, cfg, w, tokens, T.logits(tokens, w, cfg))
        return cache[name]
    return get


# ---- models -----------------------------------------------------------------------------------------
@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MODELS))
def test_prompt_portions_and_decode(dev, built, name, precision):
    path, cfg, w, tokens, want = built(name)
    m = registry.load(path, max_seq=160, precision=precision)
    assert m.layer_runs == len(T.layer_runs(cfg)) and m.cfg["vocab"] == cfg["vocab"]
    for sizes in ([len(tokens)], [2], [1], [7, 1, 1, 3, 2, 64, 5, 1, 31], [64], [66, 1]):
        assert_close(portions(m, tokens, sizes), want, precision, (name, sizes))
    m.close()


@pytest.mark.parametrize("seed", range(24))
def test_random_designs(dev, tmp_path, seed):
    cfg = random_model(seed)
    w = fw.random_weights(cfg, seed + 100)
    tokens = np.random.default_rng(seed).integers(0, cfg["vocab"], 170).tolist()
    want = T.logits(tokens, w, cfg)
    path = fw.write_model_folder(str(tmp_path / "m"), cfg, w)
    for precision in ("float32", "bfloat16"):
        m = registry.load(path, max_seq=171, precision=precision)
        for sizes in ([170], [97, 2, 1, 1, 1, 33, 1], [1]):
            got = portions(m, tokens, sizes)
            if precision == "float32":
                assert_close(got, want, precision, (seed, sizes))
            else:  # some of these softmaxes turn over on the last bit (single positions up to 0.7 in a rounded oracle too)
                e = errors(got, want)
                assert np.quantile(e, 0.9) < 0.1 and e.mean() < 0.05, (seed, sizes, e.mean(), np.quantile(e, 0.9))
        m.close()


@pytest.mark.parametrize("name", ["odd", "all_looped", "large_heads", "beyond_classes"])
def test_layers_one_by_one(dev, built, name):
    """Residual after every layer run, prompt pass and decode step, in 32-bit; the mixer branch's own trace is finite and
    different from the layer's."""
    path, cfg, w, tokens, _ = built(name)
    tokens = tokens[:40]
    want = T.residuals(tokens, w, cfg)
    m = registry.load(path, max_seq=64, precision="float32")
    scale = want.std(axis=(1, 2), keepdims=True)
    assert (np.abs(m.prefill_trace(tokens) - want) / scale).max() < 2e-3
    m.set_past_len(0)
    for i, t in enumerate(tokens):
        _, trace = m.step_trace(t)
        assert (np.abs(trace[:, 1] - want[:, i]) / scale[:, 0]).max() < 2e-3, i
    m.close()


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [[150], [1], [9]])
def test_window_and_kept_token_edges(dev, built, precision, sizes):
    """The logits match the model's own masks and none of their neighbours: a window one longer or shorter, a kept token
    more or less."""
    path, cfg, w, tokens, want = built("plain")
    m = registry.load(path, max_seq=160, precision=precision)
    got = portions(m, tokens, sizes)
    m.close()
    mine = errors(got, want)[50:].mean()
    for change in ({"l0_size": 1}, {"l0_size": -1}, {"l0_keep_first": 1}, {"l0_keep_first": -1}, {"l1_size": 1}, {"l1_size": -1}):
        other = errors(got, T.logits(tokens, w, variant(cfg, **change)))[50:].mean()
        assert other > (20 if precision == "float32" else 2) * mine, (change, other, mine)


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
def test_cache_is_used_again(dev, built, precision):
    """A second request over the first one's cache, shorter and longer, gives what a fresh model gives."""
    path, cfg, w, tokens, want = built("odd")
    m = registry.load(path, max_seq=160, precision=precision)
    portions(m, tokens[::-1], [150])
    a = portions(m, tokens[:30], [12, 1, 1, 16])
    portions(m, tokens[::-1], [70, 1])
    b = portions(m, tokens, [100, 1])
    m.close()
    fresh = registry.load(path, max_seq=160, precision=precision)
    assert np.array_equal(a, portions(fresh, tokens[:30], [12, 1, 1, 16]))
    assert np.array_equal(b, portions(fresh, tokens, [100, 1]))
    assert_close(b, want, precision)
    fresh.close()


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


def test_long_context_and_far_keys(dev, tmp_path):
    """Over 8192 positions: more chunks than the decode attention has workgroups, prompts of several chunks.  One key at the
    far end is made to stand out: the last tokens must find it."""
    cfg = model([layer(attention(4, 4, 16, 16, rot=4, sharp=2.0), 32), layer(latent(3, 16, 4, 24, 16, sharp=2.0))], 32, 50)
    w = fw.random_weights(cfg, 21)
    n = 8400
    rng = np.random.default_rng(4)
    tokens = rng.integers(1, 50, n)
    tokens[3] = tokens[-1] = tokens[-2] = 0          # a token that occurs three times: its key lies along its query
    w["l0.mix.k"] = w["l0.mix.q"].copy()
    w["l0.mix.k.norm"] = w["l0.mix.q.norm"].copy()
    path = fw.write_model_folder(str(tmp_path / "long"), cfg, w)
    # the oracle at the last places only: all keys, few queries
    eps = cfg["norm"]["eps"]
    want = last_logits(tokens, w, cfg, 4)
    for precision in ("float32", "bfloat16"):
        m = registry.load(path, max_seq=n + 8, precision=precision)
        m.prefill(tokens[:-2].tolist())
        got = [m.prefill_logits(tokens[-2:].tolist(), [0, 1])]
        m.set_past_len(n - 2)
        for t in tokens[-2:]:
            m.step(int(t))
            got.append(m.logits()[None])
        got = np.concatenate(got)
        e = errors(got, np.concatenate([want[-2:], want[-2:]]))
        assert e.max() < (3e-4 if precision == "float32" else 0.1), (precision, e)
        m.close()


def last_logits(tokens, w, cfg, n_last):
    """Two-layer models without windows: the first layer in full in blocks of queries, the second for the last places."""
    eps = cfg["norm"]["eps"]
    full = cfg["layers"][0]["mixer"], cfg["layers"][1]["mixer"]
    x = w["embed"][tokens].astype(np.float64)
    n = len(tokens)
    pos = np.arange(n)

    def attend(q, k, v, scale, first):
        out = []
        for a in range(0, len(q), 700):
            qs = q[a:a + 700]
            i = first + a + np.arange(len(qs))
            out.append(np.stack([soft(qs[:, h] @ k[:, h].T * scale, i) @ v[:, h] for h in range(q.shape[1])], axis=1))
        return np.concatenate(out)

    def soft(s, i):
        s = np.where(pos[None, :] <= i[:, None], s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        return p / p.sum(axis=1, keepdims=True)

    m = full[0]
    h = T.rms_norm(x, w["l0.norm1"], eps)
    shape = lambda y, d: y.reshape(n, m["heads"], d)
    q = T.rotate(shape(T.rms_norm(h @ w["l0.mix.q"].T, w["l0.mix.q.norm"], eps), m["dim"]), pos, m["rot"])
    k = T.rotate(shape(T.rms_norm(h @ w["l0.mix.k"].T, w["l0.mix.k.norm"], eps), m["dim"]), pos, m["rot"])
    v = shape(h @ w["l0.mix.v"].T, m["vdim"])
    o = attend(q, k, v, m["scale"], 0).reshape(n, -1) @ w["l0.mix.o"].T
    x = x + T.rms_norm(o, w["l0.norm1b"], eps)
    x = x + T.rms_norm(T.dense_ff(T.rms_norm(x, w["l0.norm2"], eps), w, "l0.mlp."), w["l0.norm2b"], eps)
    m = full[1]
    h = T.rms_norm(x, w["l1.norm1"], eps)
    down = h @ w["l1.mix.dkv"].T
    c = T.rms_norm(down[:, :m["kv_rank"]], w["l1.mix.dkv.norm"], eps)
    kr = T.rotate(down[:, None, m["kv_rank"]:], pos, m["rot"])
    H = m["heads"]
    q = (h[-n_last:] @ w["l1.mix.q"].T).reshape(n_last, H, -1)
    q = np.concatenate([q[..., :m["dim"]], T.rotate(q[..., m["dim"]:], pos[-n_last:], m["rot"])], axis=2)
    k = np.concatenate([(c @ w["l1.mix.uk"].T).reshape(n, H, -1), np.broadcast_to(kr, (n, H, m["rot_dim"]))], axis=2)
    o = attend(q, k, (c @ w["l1.mix.uv"].T).reshape(n, H, -1), m["scale"], n - n_last).reshape(n_last, -1) @ w["l1.mix.o"].T
    x = x[-n_last:] + T.rms_norm(o, w["l1.norm1b"], eps)
    return T.rms_norm(x, w["final.norm"], eps) @ w["head"].T


@pytest.mark.parametrize("precision", ["float32", "bfloat16"])
def test_greedy_generation(dev, built, precision):
    """Greedy tokens through prefill + greedy and through generate(); every token is the oracle's best on that very text, or
    within rounding of it."""
    path, cfg, w, tokens, _ = built("odd")
    prompt, n = tokens[:23], 60
    m = registry.load(path, max_seq=160, precision=precision)
    first = m.prefill(prompt)
    out = [first] + m.greedy(first, n - 1)
    m.set_past_len(0)
    assert m.generate(prompt, [0.5] * n, temperature=0.0, top_k=1, top_p=1.0) == out
    m.set_past_len(0)
    stop = out[20]
    cut = out.index(stop)
    assert m.generate(prompt, [0.5] * n, temperature=0.0, top_k=1, top_p=1.0, stop_ids=[stop]) == out[:cut]
    lg = T.logits(prompt + out, w, cfg)[len(prompt) - 1:-1]
    gap = (lg.max(axis=1) - lg[np.arange(n), out]) / lg.std()
    assert gap.max() < LIMITS[precision][0], gap.max()
    if precision == "float32":
        assert gap.max() == 0.0
    m.close()


def test_command_line(dev, built, capsys):
    """Token ids in, the same greedy ids out as through the Python interface."""
    from prometorch_amd.__main__ import main
    path, cfg, w, tokens, _ = built("odd")
    m = registry.load(path, max_seq=64)
    want = m.generate(tokens[:9], [0.0] * 12, temperature=0.0, top_k=1, top_p=1.0)
    m.close()
    args = ["generate", "--model", path, "--tokens", ",".join(map(str, tokens[:9])), "--max-new", "12", "--temperature", "0"]
    assert main(args) == 0
    assert capsys.readouterr().out.split() == [str(t) for t in want]


def test_sampled_generation(dev, built):
    """The sampler over these logits: the same draws give the same tokens again, and they are the tokens the sampler picks
    from logits read back step by step."""
    import torch
    path, cfg, w, tokens, _ = built("all_looped")
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
    for name, code in (("l1.mix.q.norm", -10), ("side.embed", -10), ("loop.step", -10)):
        bad = {k: v for k, v in w.items() if k != name}
        with pytest.raises(_lib.PtmError) as e:
            registry.load(fw.write_model_folder(str(tmp_path / "missing"), cfg, bad), max_seq=16)
        assert e.value.code == code, name
    bad = dict(w, **{"l0.mix.uk": w["l0.mix.uk"][:-1]})
    with pytest.raises(_lib.PtmError) as e:
        registry.load(fw.write_model_folder(str(tmp_path / "shape"), cfg, bad), max_seq=16)
    assert e.value.code == -2
    m = registry.load(path, max_seq=16, precision="bfloat16")
    with pytest.raises(_lib.PtmError):
        m.prefill([0] * 17)          # past the cache
    with pytest.raises(_lib.PtmError):
        m.step(cfg["vocab"])         # no such token
    m.close()


# ---- the framework's other models: the shared calls --------------------------------------------------
def test_prefill_logits_of_a_quantised_model(dev):
    from prometorch_amd.decode import Decoder
    cfg = dict(synth.TINY)
    layers = [synth.make_layer(7, i, cfg) for i in range(cfg["n_layers"])]
    d = Decoder(cfg, layers, synth.make_head(7, cfg), max_seq=64)
    tokens = [3, 9, 27, 1, 5, 8, 13, 2, 40, 6]
    d.set_past_len(0)
    rows = d.prefill_logits(tokens, [0, 4, 9], chunk_rows=4)
    assert np.array_equal(rows[2], d.logits())
    for i, p in enumerate((0, 4, 9)):
        d.set_past_len(0)
        d.prefill(tokens[:p + 1], chunk_rows=4)
        assert errors(rows[i][None], d.logits()[None])[0] < 2e-2, p
    assert d.layer_runs == cfg["n_layers"]
    d.close()


# ---- kernels ------------------------------------------------------------------------------------------
def padded(a, cols=None):
    """Rows padded to a multiple of 64 columns with zeros."""
    c = (a.shape[-1] + 63) // 64 * 64
    out = np.zeros(a.shape[:-1] + (c,), a.dtype)
    out[..., :a.shape[-1]] = a
    return out


@pytest.mark.parametrize("N,K", [(5, 8), (70, 64), (33, 100), (500, 200), (130, 257), (77, 512), (300, 1000), (64, 2000),
                                 (5000, 2048), (200, 3000), (4100, 3100), (513, 4096), (96, 9000), (12, 20000)])
def test_dense_gemv(dev, N, K):
    import torch
    L = _lib.load()
    rng = np.random.default_rng(N + K)
    W = fw.to_bf16(rng.standard_normal((N, K), np.float32))
    x = rng.standard_normal(K, np.float32)
    Wd = torch.from_numpy(padded(W).view(np.int16)).cuda()
    xd = torch.from_numpy(padded(x)).cuda()
    y = torch.full((N + 3,), 7.0, device="cuda")
    _lib.check(L.ptm_dense_gemv(Wd.data_ptr(), xd.data_ptr(), y.data_ptr(), K, N, Wd.shape[1], None), "gemv")
    torch.cuda.synchronize()
    y = y.cpu().numpy()
    ref = fw.from_bf16(W).astype(np.float64) @ x
    assert np.abs(y[:N] - ref).max() < 2e-6 * np.sqrt(K) * np.abs(ref).std() + 1e-5 and (y[N:] == 7.0).all()


@pytest.mark.parametrize("fp32", [False, True])
@pytest.mark.parametrize("M,N,K", [(1, 3, 8), (2, 70, 40), (31, 257, 100), (33, 65, 320), (64, 64, 64), (100, 130, 192),
                                   (150, 1000, 72), (300, 4100, 200), (1030, 2050, 136)])
def test_dense_gemm(dev, M, N, K, fp32):
    import torch
    L = _lib.load()
    rng = np.random.default_rng(M * N + K)
    W = fw.to_bf16(rng.standard_normal((N, K), np.float32))
    A = rng.standard_normal((M, K), np.float32)
    if not fp32:
        A = fw.from_bf16(fw.to_bf16(A))
    Wd = torch.from_numpy(padded(W).view(np.int16)).cuda()
    Ad = torch.from_numpy(padded(A) if fp32 else padded(fw.to_bf16(A)).view(np.int16)).cuda()
    Cd = torch.full((M + 1, N + 1), 7.0, device="cuda")
    _lib.check(L.ptm_dense_gemm(Ad.data_ptr(), int(fp32), Ad.shape[1], Wd.data_ptr(), Wd.shape[1], Cd.data_ptr(), N + 1, M, N, K, None), "gemm")
    torch.cuda.synchronize()
    got = Cd.cpu().numpy()
    ref = A.astype(np.float64) @ fw.from_bf16(W).astype(np.float64).T
    assert np.abs(got[:M, :N] - ref).max() < 3e-6 * K ** 0.5 * ref.std() + 1e-5
    assert (got[M] == 7.0).all() and (got[:, N] == 7.0).all()


CASES = [  # rows, heads, kv heads, dim1, dim2, vdim, window, keep, pos0, softcap
    (5, 4, 2, 16, 0, 16, 0, 0, 0, 0.0), (40, 6, 2, 24, 8, 40, 7, 0, 0, 0.0), (130, 3, 3, 64, 0, 64, 64, 0, 5, 10.0),
    (70, 8, 1, 64, 0, 128, 20, 70, 300, 0.0), (257, 2, 2, 128, 64, 128, 65, 0, 64, 0.0), (33, 40, 1, 32, 0, 32, 33, 3, 100, 5.0),
    (2, 4, 4, 96, 32, 96, 63, 1, 126, 0.0), (90, 2, 1, 200, 40, 256, 0, 0, 37, 0.0), (20, 2, 2, 264, 0, 296, 9, 2, 50, 0.0)]


@pytest.mark.parametrize("fp32", [False, True])
@pytest.mark.parametrize("case", CASES)
def test_attention_rows_kernel(dev, case, fp32):
    """Random keys, and for three query rows one key each that stands out: the last position of the window, one position
    outside, and (if tokens are kept) the last kept one and the first that is not."""
    import torch
    L = _lib.load()
    rows, H, G, d1, d2, dv, window, keep, pos0, cap = case
    rng = np.random.default_rng(sum(case[:9]))
    n = pos0 + rows
    rnd = (lambda *s: rng.standard_normal(s, np.float32)) if fp32 else (lambda *s: fw.from_bf16(fw.to_bf16(rng.standard_normal(s, np.float32))))
    q, k1, k2, v = rnd(rows, H, d1 + d2), rnd(n, G, d1), rnd(n, max(d2, 8)), rnd(n, G, dv)
    for r, off in ((rows - 1, 0), (rows // 2, 1), (rows // 3, -1)):
        if window and pos0 + r - window + off >= 0:
            k1[pos0 + r - window + off] = q[r, ::H // G, :d1] * 2      # off 0: just outside; 1: just inside
    if keep and keep < n:
        k1[keep - 1] = q[rows - 1, ::H // G, :d1]
        k1[keep] = q[rows - 1, ::H // G, :d1]
    scale = 1.5 / np.sqrt(d1 + d2)
    full_k = np.concatenate([k1, np.broadcast_to(k2[:, None, :d2], (n, G, d2))], axis=2)
    big_q = np.zeros((n, H, d1 + d2))
    big_q[pos0:] = q
    want = T.softmax_attend(big_q, full_k.astype(np.float64), v.astype(np.float64), scale, T.visible(n, {"size": window, "keep_first": keep}), cap)[pos0:]
    put = lambda a: torch.from_numpy(a if fp32 else fw.to_bf16(a).view(np.int16)).cuda()
    Q, K1, K2, V = put(q), put(k1), put(k2), put(v)
    O = torch.zeros((rows, H, dv), dtype=torch.float32 if fp32 else torch.bfloat16, device="cuda")
    a = _lib.AttentionArgs(Q=Q.data_ptr(), K1=K1.data_ptr(), K2=K2.data_ptr() if d2 else None, V=V.data_ptr(), O=O.data_ptr(),
                           q_row=H * (d1 + d2), k1_row=G * d1, k1_head=d1, k2_row=max(d2, 8), v_row=G * dv, v_head=dv, o_row=H * dv,
                           rows=rows, heads=H, kv_heads=G, dim1=d1, dim2=d2, vdim=dv, window=window, keep_first=keep, pos0=pos0,
                           kv_pos0=0, scale=scale, softcap=cap, fp32=int(fp32))
    _lib.check(L.ptm_attention_rows(C.byref(a), None), "attention_rows")
    torch.cuda.synchronize()
    err = np.abs(O.float().cpu().numpy() - want)
    assert err.max() < (2e-5 if fp32 else 2.5e-2), err.max()  # bfloat16: the output's own rounding
    # the same rows with the array starting at the first visible position
    lo = pos0 - window + 1
    if window and not keep and lo > 0:
        O2 = torch.zeros_like(O)
        es = 4 if fp32 else 2
        b = _lib.AttentionArgs.from_buffer_copy(a)
        b.O, b.kv_pos0 = O2.data_ptr(), lo
        b.K1, b.V = K1.data_ptr() + lo * G * d1 * es, V.data_ptr() + lo * G * dv * es
        if d2:
            b.K2 = K2.data_ptr() + lo * max(d2, 8) * es
        _lib.check(L.ptm_attention_rows(C.byref(b), None), "attention_rows")
        torch.cuda.synchronize()
        assert torch.equal(O, O2)
