"""Decoders whose sublayers are normed at their end (Zovovik) on the device: windows with kept first tokens, sinks, decays,
the token shift and what they leave for the next portion or sequence.  The configurations of `hybridgen` run through the
general tests of test_gpu_hybrid.py as well."""
import io
import json
import subprocess
import sys

import numpy as np
import pytest

import hybridgen as G
from kalosm_amd.fusor import FusorHipError
from oracle import hybrid_ref as R
from test_gpu_hybrid import TOL, close, reference, run_portions

pytestmark = pytest.mark.gpu


def attention_only(window, keep, heads=4, kv_heads=2, dim=32, vdim=32, vocab=97, positions=2048):
    """One layer whose attention decides the result."""
    return G.config_apart([G.with_mlp(G.pair(G.attention(heads, kv_heads, dim, vdim, window, keep, 2, scale=dim ** -0.5),
                                             {"heads": 2, "dim": 16}, (1.0, 0.05)), None)], width=128, vocab=vocab, positions=positions)


def masked(cfg, **change):
    """The same model with another mask."""
    layer = cfg["layers"][0]
    left = dict(layer["mixer"]["left"], mask=dict(layer["mixer"]["left"]["mask"], **change))
    return dict(cfg, layers=[dict(layer, mixer=dict(layer["mixer"], left=left))])


@pytest.mark.parametrize("window,keep", [(5, 3), (16, 16), (33, 1), (64, 70), (20, 0), (90, 7)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_window_and_kept_edges(dev, window, keep, dtype):
    """Partners of a query exactly inside and outside the window, among the kept tokens, and right behind the last of them; a
    mask that is one off in either number changes the marked positions far beyond the tolerance."""
    cfg = attention_only(window, keep)
    w = G.matching_attention(cfg, G.weights(cfg, 2), 0, 2.5, [(i, 10 + i) for i in range(8)])
    n = keep + 4 * window + 90
    toks = np.random.default_rng(4).integers(20, 97, n)
    marks = {}

    def put(name, key, query):  # token `name` of the pairs: its partner at `key`, itself at `query`
        i = len(marks)
        while toks[key] < 20 or toks[query] < 20:
            query += 1
            key += 0 if name.startswith("first") else 1
        toks[key], toks[query] = 10 + i, i
        marks[name] = query

    if keep:
        put("first_in", keep - 1, n - 30)
    put("first_out", keep, n - 20)
    base = keep + window + 3
    put("in", base, base + window - 1)
    put("out", base + 1, base + 1 + window)
    put("inside", base + 5, base + 5 + max(window - 2, 1))
    if keep > 2:
        put("first_0", 0, n - 10)
    want, _ = R.forward(cfg, w, toks)
    off = {}
    for name, change in (("out", {"size": window + 1}), ("in", {"size": window - 1}), ("first_out", {"keep_first": keep + 1}),
                         ("first_in", {"keep_first": keep - 1})):
        if name in marks:
            off[name] = G.rel_err(R.forward(masked(cfg, **change), w, toks)[0], want)[marks[name]]
    assert min(off.values()) > 5 * TOL[dtype], off
    m = G.build(dev, cfg, w, dtype)
    for sizes in ([n], [1], [window], [window + 1, 2], [40, 1, 1, 1], [max(keep, 2)], [n - 40, 1]):
        close(run_portions(m, toks, sizes), want, TOL[dtype], str(sizes))


@pytest.mark.parametrize("window", [600, 5000])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_one_key_among_hundreds(dev, window, dtype):
    """At the first position, where the cache grows, and near the end; a window of 600 rows wraps on the way."""
    cfg = attention_only(window, 4, vocab=400)
    places = (0, 63, 64, 255, 256, 257, 511, 512)
    w = G.matching_attention(cfg, G.weights(cfg, 2), 0, 2.5, [(i, 10 + i) for i in range(8)])
    toks = np.random.default_rng(4).integers(20, 400, 700)
    toks[list(places)] = 10 + np.arange(8)
    toks[590:598] = np.arange(8)
    toks[690:698] = np.arange(8)
    want, _ = R.forward(cfg, w, toks)
    for i, p in enumerate(places):  # each partner matters
        other = toks[:600].copy()
        other[p] = 399
        assert G.rel_err(R.forward(cfg, w, other)[0], want[:600])[590 + i] > 5 * TOL[dtype]
    m = G.build(dev, cfg, w, dtype)
    for sizes in ([700], [255, 1, 1, 2, 200, 1], [580, 1]):
        close(run_portions(m, toks, sizes), want, TOL[dtype], str(sizes))


@pytest.mark.parametrize("sink", [5.0, -40.0])
def test_sink_sizes(dev, sink):
    cfg = attention_only(9, 2)
    w = G.weights(cfg)
    w["l0.mix.left.sink"] = np.full_like(w["l0.mix.left.sink"], sink)
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 30)
    want, _ = R.forward(cfg, w, toks)
    if sink > 0:  # values far below the sink: without it the time mixing beside them would hardly count
        bare, _ = R.forward(cfg, {k: v for k, v in w.items() if not k.endswith("sink")}, toks)
        assert G.rel_err(bare, want).min() > 1e-2
    m = G.build(dev, cfg, w)
    for sizes in ([30], [1], [4, 2]):
        close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))


@pytest.mark.parametrize("decay", [[1.0, 0.0, 0.99951171875], [0.5, 1e-30, 1.0]])
def test_constant_decays(dev, decay):
    """States that keep everything, nothing, or nearly everything, in one layer."""
    cfg = G.config_apart([G.with_mlp(G.retention(3, 24, 20, 16, decay=decay), G.dense(40))], 128, 64)
    w = G.weights(cfg)
    toks = np.random.default_rng(1).integers(0, 64, 300)
    want, _ = R.forward(cfg, w, toks)
    m = G.build(dev, cfg, w)
    for sizes in ([300], [1], [70, 2, 64, 23, 25]):
        close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))


@pytest.mark.parametrize("w0", [-14.0, 0.0, 1.5, 3.2, 9.0, None])
@pytest.mark.parametrize("dim", [16, 64, 120, 144])
def test_channel_decays(dev, w0, dim):
    """Channels that forget nothing, at once, or (None) every one at a rate of its own, from e^-0.0001 to e^-400 per token,
    through the chunked form and token by token."""
    cfg = G.config_apart([G.with_mlp(G.pair(G.attention(2, 1, 8, 8, 6, 1, 4), {"heads": 2, "dim": dim}, (0.01, 1.0)), None)], 128, 64)
    w = G.weights(cfg)
    p = "l0.mix.right."
    values = np.full(2 * dim, w0) if w0 is not None else np.random.default_rng(3).uniform(-9.0, 6.0, 2 * dim)
    w[p + "w0"] = G.round_bf16(values)
    w[p + "w2"] = G.round_bf16(w[p + "w2"] * 2.0)
    toks = np.random.default_rng(1).integers(0, 64, 210)
    want, _ = R.forward(cfg, w, toks)
    m = G.build(dev, cfg, w)
    for sizes in ([210], [1], [70, 2, 64, 23, 25]):
        close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))


def test_bonus_counts_for_the_current_token_only(dev):
    cfg = G.config_apart([G.with_mlp(G.pair(G.attention(1, 1, 8, 8, 6, 1, 4), {"heads": 3, "dim": 20}, (0.01, 1.0)), None)], 96, 64)
    w = G.weights(cfg)
    w["l0.mix.right.u"] = G.round_bf16(w["l0.mix.right.u"] * 6.0)
    toks = np.random.default_rng(1).integers(0, 64, 100)
    want, _ = R.forward(cfg, w, toks)
    without, _ = R.forward(cfg, dict(w, **{"l0.mix.right.u": np.ones_like(w["l0.mix.right.u"])}), toks)
    assert np.median(G.rel_err(without, want)) > 1e-2
    m = G.build(dev, cfg, w)
    for sizes in ([100], [1], [26, 2]):
        close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))


@pytest.mark.parametrize("part", ["r", "k", "v", "g", "w"])
def test_token_shift_of_each_input(dev, part):
    """One input reads the previous token alone (its mu is one), the others the current one."""
    cfg = G.config_apart([G.with_mlp(G.pair(G.attention(1, 1, 8, 8, 6, 1, 4), {"heads": 3, "dim": 20}, (0.01, 1.0)), None)] * 2, 96, 64)
    w = G.weights(cfg)
    for n in "rkvgw":
        w["l0.mix.right.mu." + n][:] = float(n == part)
    toks = np.random.default_rng(1).integers(0, 64, 90)
    want, _ = R.forward(cfg, w, toks)
    m = G.build(dev, cfg, w)
    for sizes in ([90], [1], [2], [3, 2, 1, 4, 30]):
        close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))


@pytest.mark.parametrize("rank", [1, 7, 64, 130])
def test_low_rank_of_the_decays_is_the_files(dev, rank):
    from kalosm_amd import synth
    from kalosm_amd.hybrid import HybridModel

    cfg = G.config_apart([G.with_mlp(G.pair(), G.dense())])
    w = {n: synth.from_bf16_bits(synth.hybrid_random_tensor(n, a, b, 0, False)).reshape((a, b) if b else (a,))
         for n, a, b in synth.hybrid_tensor_specs(cfg, rank)}
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 60)
    want, _ = R.forward(cfg, w, toks)
    m = G.build(dev, cfg, w)
    for sizes in ([60], [1], [30, 2]):
        close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))
    m = HybridModel(dev, cfg)
    bad = dict(w, **{"l0.mix.right.w2": np.zeros((120, rank + 1), np.float32)})
    with pytest.raises(FusorHipError, match="low rank"):
        m.load_all(G.tensors(bad))


@pytest.mark.parametrize("name", ["apart", "apart_full", "apart_large"])
def test_sequences_one_after_the_other(dev, name):
    """What an earlier sequence leaves in caches, states and shift rows is not seen by the next one."""
    cfg, w, toks, want, _ = reference(name)
    m = G.build(dev, cfg, w)
    other = np.random.default_rng(9).integers(0, cfg["vocab"], 90)
    for length, sizes in ((1, [1]), (90, [1]), (3, [3]), (60, [60]), (2, [1]), (89, [89])):
        run_portions(m, other[:length], sizes)
        close(run_portions(m, toks[:40], [5, 1]), want[:40], TOL["float32"], f"after {length} tokens")
        run_portions(m, other[:length], sizes)
        close(run_portions(m, toks[:40], [40]), want[:40], TOL["float32"], f"whole after {length} tokens")


@pytest.mark.parametrize("name", ["apart", "apart_ones", "apart_full"])
def test_first_tokens(dev, name):
    cfg, w, toks, want, _ = reference(name)
    m = G.build(dev, cfg, w)
    for n in (1, 2, 3, 4, 5, 6):
        close(run_portions(m, toks[:n], [n]), want[:n], TOL["float32"], f"{n} tokens")


def test_portions_bf16(dev):
    for name in ("apart", "apart_large"):
        cfg, w, toks, want, _ = reference(name)
        m = G.build(dev, cfg, w, "bfloat16")
        for sizes in ([2], [37], [90, 1]):
            close(run_portions(m, toks, sizes), want, TOL["bfloat16"], f"{name} {sizes}")


@pytest.mark.parametrize("kernel", [1, 2])
@pytest.mark.parametrize("name", ["apart", "apart_ones", "apart_large"])
def test_both_forms_of_the_recurrences(dev, name, kernel):
    cfg, w, toks, want, _ = reference(name)
    m = G.build(dev, cfg, w)
    dev.set_option("recurrent_kernel", kernel)
    try:
        for sizes in ([150], [2, 63, 64, 1, 20]):
            close(run_portions(m, toks, sizes), want, TOL["float32"], str(sizes))
    finally:
        dev.set_option("recurrent_kernel", 0)


def test_long_decode_follows_the_reference(dev):
    """Greedy tokens of the device loop (captured step, replayed, over ring and growth borders) fed to the reference: each is
    the best or next to it."""
    cfg, w, toks, _, _ = reference("apart")
    m = G.build(dev, cfg, w)
    out = m.generate(toks[:11], 400)
    want, _ = R.forward(cfg, w, np.concatenate([toks[:11], out]))
    rows = want[10:410]
    assert (rows[np.arange(400), out] >= rows.max(axis=1) - 1e-3 * rows.std()).all()
    close(m.forward([int(out[-1])])[None], want[-1:], TOL["float32"])  # the sequence goes on from where the loop ended
    dev.set_option("step_eager", 1)
    try:
        m.reset()
        assert m.generate(toks[:11], 60).tolist() == out[:60].tolist()
    finally:
        dev.set_option("step_eager", 0)
    m.reset()
    assert m.generate(toks[:11], 60).tolist() == out[:60].tolist()


def test_long_prompt_in_portions_of_its_own(dev):
    """A prompt beyond the largest portion is cut by the decoder; the kept tokens are still seen behind the cut."""
    cfg = attention_only(30, 6, 2, 1, 16, 16, vocab=60, positions=2600)
    cfg = dict(cfg, width=64, layers=cfg["layers"] + [G.with_mlp(G.retention(1, 16, 16, 8), G.dense(20))])
    w = G.matching_attention(cfg, G.weights(cfg), 0, 2.5, [(0, 10)])
    toks = np.random.default_rng(1).integers(20, 60, 2500)
    toks[3], toks[2490] = 10, 0
    want, _ = R.forward(cfg, w, toks)
    m = G.build(dev, cfg, w)
    places = [0, 2046, 2047, 2048, 2049, 2077, 2078, 2079, 2490, 2499]
    close(m.forward(toks, want=places), want[places], TOL["float32"])


def test_context_ends_where_the_positions_end(dev):
    """The learned positions bound the context; when it is full the tail of all tokens runs again from position 0."""
    cfg = G.config_apart([G.with_mlp(G.pair(), G.dense())], positions=64)
    w = G.weights(cfg)
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 80)
    m = G.build(dev, cfg, w, ctx=4096)
    assert m.context == 64
    want, _ = R.forward(cfg, w, toks[:64])
    close(run_portions(m, toks[:64], [60, 1]), want, TOL["float32"])
    got = m.forward(toks[64:70])
    want, _ = R.forward(cfg, w, toks[70 - 32:70])
    close(got[None], want[-1:], TOL["float32"])


def test_model_folder_through_registry_command_line_and_replay(dev, tmp_path):
    from kalosm_amd import registry, trace

    cfg, w, toks, want, _ = reference("apart")
    G.save(tmp_path, cfg, w)
    assert registry.architecture(str(tmp_path)) == "Zovovik"
    m = registry.load(dev, str(tmp_path), dtype="float32", ctx=512)
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
             {"step": 1, "entries": [{"id": "x", "tokens": toks[30:32].tolist(), "want": [1]}], "end": ["x"]},
             {"step": 2, "entries": [{"id": "y", "tokens": toks[:1].tolist(), "want": [0]}], "end": ["y"]}]
    assert trace.run(str(tmp_path), "float32", str(out_dir), 64, lines=[json.dumps(s) for s in steps], out=out) == 0
    for n, places in ((0, [4, 29]), (1, [31]), (2, [0])):
        close(np.fromfile(out_dir / f"{n}.f32", "<f4").reshape(len(places), -1), want[places], TOL["float32"])


def test_configurations_that_do_not_fit_are_refused(dev):
    from kalosm_amd.hybrid import HybridModel

    cfg = G.CONFIGS["apart_ones"]
    ret, pr = G.retention(2), G.pair()
    bad_heads = G.pair(G.attention(heads=5, kv_heads=2))
    for change, text in (({"layers": [G.with_mlp(G.delta(), None)]}, "has no mixer"), ({"max_positions": 0}, "max_positions"),
                         ({"layers": [G.with_mlp(dict(ret, mixer=dict(ret["mixer"], decay=[0.5])), None)]}, "one decay per head"),
                         ({"layers": [G.with_mlp(dict(ret, mixer=dict(ret["mixer"], decay=[0.5, 1.5])), None)]}, "between 0 and 1"),
                         ({"layers": [G.with_mlp(pr, G.moe())]}, "feed-forward"),
                         ({"layers": [G.with_mlp(bad_heads, None)]}, "share")):
        with pytest.raises(FusorHipError, match=text):
            HybridModel(dev, dict(cfg, **change))
    with pytest.raises(FusorHipError, match="has no mixer"):
        HybridModel(dev, G.config([G.with_mlp(ret, None)]))
