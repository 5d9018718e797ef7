"""Layer-list decoders on the device against the plain numpy restatement (oracle/hybrid_ref.py)."""
import io
import json
import subprocess
import sys

import numpy as np
import pytest

import hybridgen as G
from kalosm_amd import synth
from kalosm_amd.fusor import FusorHipError, GpuMirostat2SamplerParams, GpuStandardSamplerParams, QMatrix, Tensor
from oracle import hybrid_ref as R

pytestmark = pytest.mark.gpu

TOL = {"float32": 3e-5, "bfloat16": 4e-2}  # of the logits' standard deviation
_ref = {}


def reference(name, T=150, seed=0):
    key = (name, T, seed)
    if key not in _ref:
        cfg = G.CONFIGS[name]
        w = G.weights(cfg, seed)
        toks = np.random.default_rng(seed + 3).integers(0, cfg["vocab"], T)
        _ref[key] = (cfg, w, toks, *R.forward(cfg, w, toks))
    return _ref[key]


def run_portions(m, toks, sizes):
    """Logits of every position, the tokens fed in portions of the given sizes (the last size repeats)."""
    m.reset()
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(sizes[min(i, len(sizes) - 1)], len(toks) - at)
        out.append(m.forward(toks[at:at + n], want=list(range(n))))
        at += n
        i += 1
    return np.concatenate(out)


def close(got, want, tol, what=""):
    e = G.rel_err(got, want)
    if tol == TOL["bfloat16"] and len(e) > 30:
        # random routers have close calls that rounded activations decide the other way now and then
        assert np.mean(e > tol) <= 0.03, f"{what}: {np.mean(e > tol):.1%} of the positions are off by more than {tol}"
        tol = 10 * tol
    assert e.max() <= tol, f"{what}: position {int(e.argmax())} is off by {e.max():.3g} (tolerance {tol})"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_whole_prompt_and_layers(dev, name, dtype):
    cfg, w, toks, want, layers = reference(name)
    m = G.build(dev, cfg, w, dtype)
    m.keep_layers()
    got = run_portions(m, toks, [len(toks)])
    close(got, want, TOL[dtype], "logits")
    for i in range(len(layers)):
        close(m.layer_output(i, len(toks)), layers[i], TOL[dtype], f"layer {i}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_token_by_token(dev, name, dtype):
    """Every token through the decode step: caches of wrapped rings, states and convolution tails."""
    cfg, w, toks, want, _ = reference(name)
    close(run_portions(G.build(dev, cfg, w, dtype), toks, [1]), want, TOL[dtype])


@pytest.mark.parametrize("sizes", [[2], [3, 2], [7], [21, 1, 20, 22], [33], [64, 1, 64], [65], [100, 1, 1, 2]])
@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_portions(dev, name, sizes):
    cfg, w, toks, want, _ = reference(name)
    close(run_portions(G.build(dev, cfg, w), toks, sizes), want, TOL["float32"])


@pytest.mark.parametrize("sizes", [[2], [37], [90, 1]])
def test_portions_bf16(dev, sizes):
    cfg, w, toks, want, _ = reference("odd")
    close(run_portions(G.build(dev, cfg, w, "bfloat16"), toks, sizes), want, TOL["bfloat16"])


@pytest.mark.parametrize("kernel", [1, 2])
@pytest.mark.parametrize("name", ["odd", "ones", "large"])
def test_both_forms_of_the_recurrence(dev, name, kernel):
    cfg, w, toks, want, _ = reference(name)
    m = G.build(dev, cfg, w)
    dev.set_option("recurrent_kernel", kernel)
    try:
        for sizes in ([150], [2, 63, 64, 1, 20]):
            close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))
    finally:
        dev.set_option("recurrent_kernel", 0)


def test_sequences_one_after_the_other(dev):
    """What an earlier sequence leaves in caches and states is not seen by the next one, whatever the lengths."""
    cfg, w, toks, want, _ = reference("odd")
    m = G.build(dev, cfg, w)
    other = np.random.default_rng(9).integers(0, cfg["vocab"], 90)
    for length, sizes in ((1, [1]), (90, [1]), (3, [3]), (60, [60]), (2, [1])):
        run_portions(m, other[:length], sizes)
        close(run_portions(m, toks[:40], [5, 1]), want[:40], TOL["float32"], f"after {length} tokens")


@pytest.mark.parametrize("window", [5, 16, 33, 64])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_window_edges(dev, window, dtype):
    """A token whose partner stands exactly inside, just outside or far outside the window: the attention looks for
    partners, so seeing or missing one changes the result far beyond the tolerance."""
    cfg = G.config([G.with_mlp(G.latent(heads=2, dim=32, rot_dim=8, vdim=32, kv_rank=64, window=window), None)], width=128, vocab=97)
    w = G.matching_latent(cfg, G.weights(cfg, 2), 0, 4.0, [(i, 5 + i) for i in range(5)])
    toks = np.random.default_rng(4).integers(10, 97, 3 * window + 80)
    marks = []
    for d, tok in ((window - 1, 0), (window, 1), (window - 2, 2), (2 * window, 3), (1, 4)):
        p = 3 + 7 * len(marks)
        while toks[p] < 10 or toks[p + d] < 10:
            p += 1
        toks[p], toks[p + d] = 5 + tok, tok
        marks.append(p + d)
    want, _ = R.forward(cfg, w, toks)
    lap, _ = R.forward(G.config([dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], mask={"size": window + 1}))], 128, 97), w, toks)
    lap2, _ = R.forward(G.config([dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], mask={"size": window - 1}))], 128, 97), w, toks)
    assert G.rel_err(lap, want)[marks[1]] > 10 * TOL[dtype] and G.rel_err(lap2, want)[marks[0]] > 10 * TOL[dtype]
    m = G.build(dev, cfg, w, dtype)
    for sizes in ([len(toks)], [1], [window], [window + 1, 2], [40, 1, 1, 1]):
        close(run_portions(m, toks, sizes), want, TOL[dtype], str(sizes))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_keys_without_a_window(dev, dtype):
    """One partner among hundreds of keys, at the first position, at cache growth borders and at the end."""
    cfg = G.config([G.with_mlp(G.latent(heads=3, dim=32, rot_dim=8, vdim=32, kv_rank=64, window=0), None)], width=128, vocab=400)
    places = (0, 63, 64, 255, 256, 257, 511, 512)
    w = G.matching_latent(cfg, G.weights(cfg, 2), 0, 4.0, [(i, 10 + i) for i in range(8)])
    toks = np.random.default_rng(4).integers(20, 400, 560)
    toks[list(places)] = 10 + np.arange(8)
    toks[540:548] = np.arange(8)
    want, _ = R.forward(cfg, w, toks)
    for i, p in enumerate(places):  # each partner matters
        other = toks.copy()
        other[p] = 399
        assert G.rel_err(R.forward(cfg, w, other)[0], want)[540 + i] > 10 * TOL[dtype]
    m = G.build(dev, cfg, w, dtype)
    for sizes in ([560], [255, 1, 1, 2, 200, 1], [530, 1]):
        close(run_portions(m, toks, sizes), want, TOL[dtype], str(sizes))


def test_first_tokens(dev):
    cfg, w, toks, want, _ = reference("odd")
    m = G.build(dev, cfg, w)
    for n in (1, 2, 3, 4, 5):
        close(run_portions(m, toks[:n], [n]), want[:n], TOL["float32"], f"{n} tokens")


@pytest.mark.parametrize("sink", [4.0, -30.0])
def test_sink_sizes(dev, sink):
    cfg = G.config([G.with_mlp(G.latent(window=9), None)])
    w = G.weights(cfg)
    w["l0.mix.sink"] = np.full_like(w["l0.mix.sink"], sink)
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 30)
    want, _ = R.forward(cfg, w, toks)
    if sink > 0:
        bare, _ = R.forward(cfg, {k: v for k, v in w.items() if not k.endswith("sink")}, toks)
        assert G.rel_err(bare, want).min() > 1e-2
    m = G.build(dev, cfg, w)
    close(run_portions(m, toks, [30]), want, TOL["float32"])
    close(run_portions(m, toks, [1]), want, TOL["float32"])


@pytest.mark.parametrize("mixer", ["delta", "mamba2"])
@pytest.mark.parametrize("a_log,dt", [(-12.0, 0.0), (3.0, 2.0)])
def test_decays_near_one_and_near_zero(dev, mixer, a_log, dt):
    """A state that forgets nothing over a long prompt, and one that forgets at once."""
    cfg = G.config([G.with_mlp(G.delta(2, 1, 32, 24, 5) if mixer == "delta" else G.mamba2(2, 40, 32, 1, 2, 3), None)], 128, 64)
    w = G.weights(cfg)
    w["l0.mix.A_log"] = np.full_like(w["l0.mix.A_log"], a_log)
    w["l0.mix.dt_bias"] = np.full_like(w["l0.mix.dt_bias"], dt)
    toks = np.random.default_rng(1).integers(0, 64, 200)
    want, _ = R.forward(cfg, w, toks)
    m = G.build(dev, cfg, w)
    for sizes in ([200], [1], [70, 2, 64]):
        close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))


def test_experts_without_tokens(dev):
    """A router that sends every token to the same experts: the others' row groups are empty."""
    cfg = G.config([G.with_mlp(G.latent(), G.moe(experts=9, top=2, ff=40, shared=0))])
    w = G.weights(cfg)
    w["embed"][:, 0] = 4.0
    r = w["l0.mlp.router"] * 0.1
    r[:, 0] = np.linspace(-2, 2, 9)
    w["l0.mlp.router"] = G.round_bf16(r)
    w = {k: G.round_bf16(v) for k, v in w.items()}
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 140)
    want, _ = R.forward(cfg, w, toks)
    m = G.build(dev, cfg, w)
    close(run_portions(m, toks, [140]), want, TOL["float32"])
    close(run_portions(m, toks[:20], [1]), want[:20], TOL["float32"])


@pytest.mark.parametrize("name", ["odd", "full"])
def test_long_decode_follows_the_reference(dev, name):
    """Greedy tokens of the device loop (captured step, replayed) fed to the reference: each is the best or next to it."""
    cfg, w, toks, _, _ = reference(name)
    m = G.build(dev, cfg, w)
    prompt = toks[:11]
    out = m.generate(prompt, 330)
    assert out.shape == (330,)
    want, _ = R.forward(cfg, w, np.concatenate([prompt, out[:-1]]))
    rows = want[10:]
    best = rows.max(axis=1)
    assert (rows[np.arange(330), out] >= best - 1e-3 * rows.std()).all()
    # the sequence goes on from where the loop ended
    more = m.forward([int(out[-1])])
    full, _ = R.forward(cfg, w, np.concatenate([prompt, out]))
    close(more[None], full[-1:], TOL["float32"])


def test_captured_and_eager_steps_agree(dev):
    cfg, w, toks, _, _ = reference("odd")
    m = G.build(dev, cfg, w, "bfloat16")
    a = m.generate(toks[:20], 60)
    dev.set_option("step_eager", 1)
    try:
        m.reset()
        b = m.generate(toks[:20], 60)
    finally:
        dev.set_option("step_eager", 0)
    assert a.tolist() == b.tolist()
    m.reset()
    assert m.generate(toks[:20], 60).tolist() == a.tolist()


def test_sampling_uses_the_shared_samplers(dev):
    cfg, w, toks, _, _ = reference("odd")
    m = G.build(dev, cfg, w)
    std = GpuStandardSamplerParams(1, 1.0, 1.0, 1.0, 0.0, 0.0)  # one candidate: greedy
    greedy = m.generate(toks[:9], 20)
    m.reset()
    assert m.generate(toks[:9], 20, std).tolist() == greedy.tolist()
    m.reset()
    a = m.generate(toks[:9], 20, GpuMirostat2SamplerParams(32, 0.8, 1.3, 5.0, 0.1, 0.0), seed=3)
    m.reset()
    b = m.generate(toks[:9], 20, GpuMirostat2SamplerParams(32, 0.8, 1.3, 5.0, 0.1, 0.0), seed=3)
    assert a.tolist() == b.tolist() and len(set(a.tolist())) > 1


def test_context_is_trimmed_like_any_decoder(dev):
    """When the context is full the tail of all tokens runs again from position 0."""
    cfg, w, toks, _, _ = reference("odd")
    m = G.build(dev, cfg, w, ctx=64)
    m.forward(toks[:60])
    got = m.forward(toks[60:70])
    want, _ = R.forward(cfg, w, toks[70 - 32:70])
    close(got[None], want[-1:], TOL["float32"])
    assert m.position == 32


def test_long_prompt_in_portions_of_its_own(dev):
    """A prompt beyond the largest portion is cut by the decoder."""
    cfg = G.config([G.with_mlp(G.delta(1, 1, 16, 16, 4), None), G.with_mlp(G.latent(heads=1, dim=16, rot_dim=8, vdim=16, kv_rank=16, window=30), None)], 64, 50)
    w = G.weights(cfg)
    toks = np.random.default_rng(1).integers(0, 50, 2500)
    want, _ = R.forward(cfg, w, toks)
    m = G.build(dev, cfg, w)
    places = [0, 2046, 2047, 2048, 2049, 2077, 2078, 2079, 2499]
    close(m.forward(toks, want=places), want[places], TOL["float32"])


# ------------------------------------------------------------------ files, registry, command line, replay
def test_model_folder_through_registry_command_line_and_replay(dev, tmp_path):
    from kalosm_amd import registry, trace

    cfg, w, toks, want, _ = reference("odd")
    G.save(tmp_path, cfg, w)
    assert registry.architecture(str(tmp_path)) == "Fidasun"
    m = registry.load(dev, str(tmp_path), dtype="float32", ctx=512)
    assert (m.vocab, m.d_model, m.n_layers) == (cfg["vocab"], cfg["width"], len(cfg["layers"]))
    close(run_portions(m, toks[:50], [50]), want[:50], TOL["float32"])
    m.reset()
    ids = m.generate(toks[:8], 12)
    r = subprocess.run([sys.executable, "-m", "kalosm_amd", "generate", str(tmp_path), "--dtype", "float32", "--tokens",
                        ",".join(str(int(t)) for t in toks[:8]), "--new", "12"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert json.loads(r.stdout)["tokens"] == ids.tolist()
    out_dir, out = tmp_path / "out", io.StringIO()
    out_dir.mkdir()
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:30].tolist(), "want": [4, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[30:32].tolist(), "want": [1]}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[32:33].tolist(), "want": [0]}], "end": ["x"]}]
    assert trace.run(str(tmp_path), "float32", str(out_dir), 64, lines=[json.dumps(s) for s in steps], out=out) == 0
    assert out.getvalue().split("\n")[:3] == ["done 0", "done 1", "done 2"]
    for n, places in ((0, [4, 29]), (1, [31]), (2, [32])):
        close(np.fromfile(out_dir / f"{n}.f32", "<f4").reshape(len(places), -1), want[places], TOL["float32"])


def test_wrong_files_and_configurations_are_refused(dev, tmp_path):
    from kalosm_amd.hybrid import HybridModel

    cfg = G.CONFIGS["ones"]
    w = G.weights(cfg)
    m = HybridModel(dev, cfg)
    with pytest.raises(FusorHipError, match="unknown tensor"):
        m.load_tensor("l0.mix.extra", synth.W_BF16, 4, 0, np.zeros(4, np.uint16))
    with pytest.raises(FusorHipError, match="expected"):
        m.load_tensor("final.norm", synth.W_BF16, 4, 0, np.zeros(4, np.uint16))
    with pytest.raises(FusorHipError, match="missing"):
        m.load_all(t for t in G.tensors(w) if t[0] != "l1.mix.A_log")
    with pytest.raises(FusorHipError, match="not finalized"):
        m.forward([1])
    for change, text in (({"architecture": "Other"}, "unknown architecture"), ({"norm": {}}, "eps"), ({"layers": []}, "layers"),
                         ({"layers": [{"type": "other", "mixer": {}}]}, "unknown mixer")):
        with pytest.raises(FusorHipError, match=text):
            HybridModel(dev, dict(cfg, **change))
    G.save(tmp_path, cfg, w)
    data = (tmp_path / "model.safetensors").read_bytes()
    (tmp_path / "model.safetensors").write_bytes(data[:len(data) // 2])
    with pytest.raises(FusorHipError, match="outside the file"):
        HybridModel.open(dev, str(tmp_path))


# ------------------------------------------------------------------ dense bf16 weights as QMatrix
@pytest.mark.parametrize("n,k", [(1, 1), (7, 33), (130, 200), (300, 64), (64, 520)])
def test_bf16_qmatrix(dev, n, k):
    rng = np.random.default_rng(n + k)
    w = G.round_bf16(rng.standard_normal((n, k)))
    q = QMatrix.from_raw_bytes(dev, (n, k), synth.to_bf16_bits(w.reshape(-1)), synth.W_BF16)
    assert np.array_equal(q.dequantize().as_slice(), w)
    ids = rng.integers(0, n, 5)
    assert np.array_equal(q.embed(ids).as_slice(), w[ids])
    for m in (1, 2, 17, 70):
        x = rng.standard_normal((m, k)).astype(np.float32)
        y = Tensor.from_slice(dev, x).q_mat_mul(q).as_slice()
        want = x.astype(np.float64) @ w.T.astype(np.float64)
        assert np.abs(y - want).max() <= 2e-6 * np.abs(x).max() * np.abs(w).max() * k + 1e-6
        xb = synth.to_bf16_bits(x)
        yb = Tensor.from_slice(dev, xb, "bf16").q_mat_mul(q).as_slice()
        want = synth.from_bf16_bits(xb).astype(np.float64) @ w.T.astype(np.float64)
        assert np.abs(yb - want).max() <= 2e-6 * np.abs(x).max() * np.abs(w).max() * k + 1e-6
    both = QMatrix.concat_rows([q, q])
    assert np.array_equal(both.dequantize().as_slice(), np.concatenate([w, w]))


def test_yarn_tables(dev):
    import ctypes as C

    from kalosm_amd import _lib

    sc = {"factor": 4.0, "original": 256, "fast": 16.0, "slow": 2.0}
    for s in (None, sc):
        cos, sin = Tensor(dev, (300, 16), "f32"), Tensor(dev, (300, 16), "f32")
        y = None if s is None else C.byref(_lib.YarnScaling(*[s[n] for n in ("factor", "original", "fast", "slow")]))
        _lib.check(dev._lib.fh_rope_tables_yarn(dev._h, 32, 300, 10000.0, y, C.c_void_p(cos.ptr), C.c_void_p(sin.ptr)))
        f, amp = R.yarn_frequencies(10000.0, 32, s)
        a = np.arange(300)[:, None] * f[None, :]
        assert np.abs(cos.as_slice() - np.cos(a) * amp).max() < 4e-5 and np.abs(sin.as_slice() - np.sin(a) * amp).max() < 4e-5
