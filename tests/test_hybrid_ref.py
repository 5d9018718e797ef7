"""The plain numpy restatement of the layer-list mechanisms (oracle/hybrid_ref.py) against closed forms and independent
formulations, and the host side of the trace replay.  No device."""
import io
import json
import math

import numpy as np
import pytest

import hybridgen as G
from oracle import hybrid_ref as R

rng = np.random.default_rng(11)


def test_norm_weights_are_distances_from_one():
    x = rng.standard_normal((3, 10))
    assert np.allclose(R.norm_one_plus(x, np.zeros(10), 0.0), x / np.sqrt((x * x).mean(-1, keepdims=True)))
    assert np.allclose(R.norm_one_plus(x, np.ones(10), 1e-3), 2 * R.rms(x, 1e-3))


def test_rotation_is_a_complex_product_and_leaves_the_rest():
    f, amp = R.yarn_frequencies(100.0, 6)
    assert amp == 1.0 and np.allclose(f, [1.0, 100 ** (-1 / 3), 100 ** (-2 / 3)])
    x = rng.standard_normal((4, 8))
    y = R.rotate_interleaved(x, np.arange(4), f, 1.0, angle32=False)
    z = (x[:, 0:6:2] + 1j * x[:, 1:6:2]) * np.exp(1j * np.arange(4)[:, None] * f)
    assert np.allclose(y[:, 0:6:2], z.real) and np.allclose(y[:, 1:6:2], z.imag) and np.array_equal(y[:, 6:], x[:, 6:])


def test_yarn_keeps_fast_pairs_and_stretches_slow_ones():
    sc = {"factor": 4.0, "original": 256, "fast": 16.0, "slow": 2.0}
    f0, _ = R.yarn_frequencies(10000.0, 32)
    f, amp = R.yarn_frequencies(10000.0, 32, sc)
    assert math.isclose(amp, 0.1 * math.log(4.0) + 1.0)
    lo = max(math.floor(32 * math.log(256 / (2 * math.pi * 16)) / (2 * math.log(10000.0))), 0)
    hi = min(math.ceil(32 * math.log(256 / (2 * math.pi * 2)) / (2 * math.log(10000.0))), 31)
    assert 0 < lo < hi < 15
    assert np.allclose(f[:lo + 1], f0[:lo + 1]) and np.allclose(f[hi:], f0[hi:] / 4)
    mid = (f0 / f)[lo:hi + 1]
    assert (np.diff(mid) > 0).all()


def test_sink_joins_the_denominator_only():
    s, vis = rng.standard_normal((2, 5)), np.array([[1, 1, 0, 0, 0], [0, 1, 1, 1, 0]], bool)
    p = R.sink_softmax(s, vis, 0.7)
    for r in range(2):
        e = np.exp(s[r]) * vis[r]
        assert np.allclose(p[r], e / (e.sum() + np.exp(0.7)))
    assert np.allclose(R.sink_softmax(s, vis, -np.inf).sum(-1), 1.0)


def test_latent_attention_window_and_expansion():
    """Against a direct evaluation with the query moved through W_uk (the form a decode step uses)."""
    cfg = G.config([G.with_mlp(G.latent(window=4), None)])
    w = {k: v.astype(np.float64) for k, v in G.weights(cfg).items()}
    c, p = cfg["layers"][0]["mixer"], {k[len("l0.mix."):]: v for k, v in w.items() if k.startswith("l0.mix.")}
    h = rng.standard_normal((9, cfg["width"]))
    got = R.latent_attention(h, p, c, 1e-5)
    H, dn, dr, dv, rank = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    f, amp = R.yarn_frequencies(c["rot"]["base"], dr, c["rot"]["scaling"])
    lat = R.rms((h @ p["dkv"].T)[:, :rank], 1e-5) * p["dkv.norm"]
    kr = R.rotate_interleaved((h @ p["dkv"].T)[:, rank:], np.arange(9), f, amp)
    want = np.zeros((9, H * dv))
    for i in range(9):
        for n in range(H):
            q = (h[i] @ p["q"].T).reshape(H, dn + dr)[n]
            qr = R.rotate_interleaved(q[None, dn:], [i], f, amp)[0]
            qa = q[:dn] @ p["uk"].reshape(H, dn, rank)[n]
            js = range(max(0, i - 3), i + 1)
            e = np.exp([(qa @ lat[j] + qr @ kr[j]) * c["scale"] for j in js])
            o = sum(x * lat[j] for x, j in zip(e, js)) / (e.sum() + np.exp(p["sink"][n]))
            want[i, n * dv:(n + 1) * dv] = p["uv"].reshape(H, dv, rank)[n] @ o
    assert np.allclose(got, want @ p["o"].T)


def test_short_convolution_is_causal():
    x, w = rng.standard_normal((6, 3)), rng.standard_normal((3, 4))
    y = R.short_conv(x, w)
    for ch in range(3):
        assert np.allclose(y[:, ch], np.convolve(x[:, ch], w[ch, ::-1])[:6])
    assert np.allclose(R.short_conv(x, w[:, -1:]), x * w[:, -1])


def test_delta_rule_overwrites_the_value_of_a_key():
    """With no decay and beta 1 a repeated unit key reads its newest value; with beta 0 nothing is written."""
    k = np.zeros((3, 4))
    k[0, 1] = k[1, 2] = k[2, 1] = 1.0
    v = rng.standard_normal((3, 5))
    o = R.gated_delta(k, k, v, np.ones(3), np.ones(3))
    assert np.allclose(o, v)
    assert np.allclose(R.gated_delta(k, k, v, np.ones(3), np.zeros(3)), 0.0)


def test_delta_rule_solves_the_chunk_equations():
    """(1 + L) U = beta (V - decayed K S): the triangular system behind the recurrence."""
    T, d, e = 20, 6, 3
    q, k, v = rng.standard_normal((T, d)), R.unit(rng.standard_normal((T, d))), rng.standard_normal((T, e))
    g, beta = rng.uniform(0.5, 1.0, T), rng.uniform(0.0, 1.0, T)
    c = np.cumsum(np.log(g))
    D = np.exp(np.minimum(c[:, None] - c[None, :], 0.0))
    L = np.tril(beta[:, None] * D * (k @ k.T), -1)
    U = np.linalg.solve(np.eye(T) + L, beta[:, None] * v)
    assert np.allclose(R.gated_delta(q, k, v, g, beta), np.tril(D * (q @ k.T)) @ U)


def test_state_space_is_a_decayed_sum():
    T = 15
    x, B, C, dt = rng.standard_normal((T, 3)), rng.standard_normal((T, 4)), rng.standard_normal((T, 4)), rng.uniform(0.1, 1.0, T)
    y = R.state_space(x, B, C, dt, -0.3, 0.5)
    a = np.exp(-np.exp(-0.3) * dt)
    want = np.array([sum(np.prod(a[s + 1:t + 1]) * dt[s] * (B[s] @ C[t]) * x[s] for s in range(t + 1)) for t in range(T)]) + 0.5 * x
    assert np.allclose(y, want)


def test_router_weights_are_not_renormalised():
    z = np.array([0.1, 2.0, -1.0, 2.0, 0.5])
    idx, wts = R.route(z, 3, 1.9)
    s = np.exp(z) / np.exp(z).sum()
    assert list(idx) == [1, 3, 4] and np.allclose(wts, 1.9 * s[[1, 3, 4]])


def test_tensor_names_of_a_configuration():
    from kalosm_amd import synth

    names = [n for n, _, _ in synth.hybrid_tensor_specs(G.CONFIGS["odd"])]
    assert len(names) == len(set(names))
    assert {"embed", "head", "final.norm", "l0.mix.sink", "l1.mix.v.conv", "l2.mix.conv.b", "l3.mlp.e6.down", "l0.mlp.shared.up"} <= set(names)
    assert not any(n.startswith("l2.mlp") or n.startswith("l1.mlp.shared") for n in names)


class EchoModel:
    """Records what a replay feeds; a token's logits are the tokens of its sequence so far."""

    def __init__(self):
        self.seq, self.calls = [], []

    def reset(self):
        self.seq = []

    def forward(self, tokens, want=None):
        at = len(self.seq)
        self.seq += list(tokens)
        self.calls.append(list(tokens))
        return np.array([[at + p, self.seq[at + p]] for p in want], np.float32).reshape(len(want), 2)


def test_replay_feeds_each_step_once_and_writes_wanted_rows(tmp_path):
    from kalosm_amd import trace

    m, out = EchoModel(), io.StringIO()
    r = trace.Replay(m, str(tmp_path))
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [5, 6, 7], "want": [0, 2]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [8], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [9], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": [4, 3], "want": [1]}], "end": ["b"]}]
    for s in steps:
        r.step(json.loads(json.dumps(s)))
    assert m.calls == [[5, 6, 7], [8], [9], [4, 3]]
    read = lambda n: np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, 2).tolist()
    assert read(0) == [[0, 5], [2, 7]] and read(2) == [[4, 9]] and read(3) == [[1, 3]]
    assert not (tmp_path / "1.f32").exists()
    r.step(steps[0])
    with pytest.raises(trace.TraceError):
        r.step({"step": 9, "entries": [{"id": "c", "tokens": [1], "want": []}], "end": []})


def test_unknown_architectures_are_refused(tmp_path):
    from kalosm_amd import registry

    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nothing"}))
    assert registry.architecture(str(tmp_path)) == "Nothing"
    with pytest.raises(ValueError, match="unknown architecture"):
        registry.load(None, str(tmp_path))


# ------------------------------------------------------------------ sublayers normed at their end
def test_rotated_halves_are_complex_products():
    f, _ = R.yarn_frequencies(50.0, 6)
    x = rng.standard_normal((5, 9))
    y = R.rotated_halves(x, np.arange(5), f)
    z = (x[:, :3] + 1j * x[:, 3:6]) * np.exp(1j * np.arange(5)[:, None] * f)
    assert np.allclose(y[:, :3], z.real, atol=1e-6) and np.allclose(y[:, 3:6], z.imag, atol=1e-6)
    assert np.array_equal(y[:, 6:], x[:, 6:])


def test_kept_window_by_counting():
    v = R.kept_window(12, 3, 2)
    for i in range(12):
        assert set(np.flatnonzero(v[i])) == {j for j in range(i + 1) if j > i - 3 or j in (0, 1)}
    assert np.array_equal(R.kept_window(6, 6, 0), np.tri(6, dtype=bool))


def test_grouped_attention_head_by_head():
    cfg = G.config_apart([G.with_mlp(G.pair(G.attention(window=4, keep=2)), None)])
    c, D = cfg["layers"][0]["mixer"]["left"], cfg["width"]
    w = {k[len("l0.mix.left."):]: v.astype(np.float64) for k, v in G.weights(cfg).items() if k.startswith("l0.mix.left.")}
    h = rng.standard_normal((10, D))
    got = R.grouped_attention(h, w, c, 1e-4)
    H, d, dv, rep = c["heads"], c["dim"], c["vdim"], c["heads"] // c["kv_heads"]
    f = np.array([c["rot"]["base"] ** (-2.0 * i / c["rot"]["dims"]) for i in range(c["rot"]["dims"] // 2)])

    def turned(x, p, weight):
        x = x / np.sqrt((x @ x) / d + 1e-4) * weight
        z = (x[0:2 * len(f):2] + 1j * x[1:2 * len(f):2]) * np.exp(1j * np.float64(p) * f)
        return np.concatenate([np.stack([z.real, z.imag], 1).reshape(-1), x[2 * len(f):]])

    out = np.zeros((10, H * dv))
    for i in range(10):
        for n in range(H):
            g = n // rep
            q = turned((w["q"] @ h[i])[n * d:(n + 1) * d], i, w["q.norm"])
            den, num = np.exp(w["sink"][n]), np.zeros(dv)
            for j in range(i + 1):
                if i - j < 4 or j < 2:
                    e = np.exp(q @ turned((w["k"] @ h[j])[g * d:(g + 1) * d], j, w["k.norm"]) * c["scale"])
                    den, num = den + e, num + e * (w["v"] @ h[j])[g * dv:(g + 1) * dv]
            out[i, n * dv:(n + 1) * dv] = num / den
    assert np.allclose(got, out @ w["o"].T, atol=1e-5)


def test_fixed_decay_is_a_masked_product():
    q, k, v = (rng.standard_normal((9, n)) for n in (4, 4, 3))
    t = np.arange(9)
    m = np.where(t[:, None] >= t[None, :], 0.8 ** (t[:, None] - t[None, :]).astype(float), 0.0)
    assert np.allclose(R.fixed_decay(q, k, v, 0.8), (q @ k.T * m) @ v)


def test_channel_decay_term_by_term():
    r, k, g = rng.standard_normal((7, 4)), rng.standard_normal((7, 4)), rng.uniform(0.1, 1.0, (7, 4))
    v, u = rng.standard_normal((7, 3)), rng.standard_normal(4)
    want = np.zeros((7, 3))
    for t in range(7):
        want[t] += (r[t] * u * k[t]).sum() * v[t]
        for s in range(t):  # forgotten at every token between the two
            want[t] += (r[t] * k[s] * np.prod(g[s + 1:t], axis=0)).sum() * v[s]
    assert np.allclose(R.channel_decay(r, k, v, g, u), want)
    same = R.channel_decay(r, k, v, np.full((7, 4), 0.5), np.ones(4))
    assert np.allclose(same[1:] - (r * k).sum(1)[1:, None] * v[1:], R.fixed_decay(r[1:], k[:-1], v[:-1], 0.5))


def test_shift_reads_zeros_ahead_of_the_first_token():
    h, mu = rng.standard_normal((4, 5)), rng.uniform(0, 1, 5)
    y = R.shifted(h, mu)
    assert np.allclose(y[0], h[0] * (1 - mu)) and np.allclose(y[2], h[2] * (1 - mu) + h[1] * mu)


def test_output_norm_layers_add_unit_vectors():
    """Whatever the scale of a sublayer's matrices, what joins the residual stream has the norm weight's root mean square."""
    cfg = G.config_apart([G.with_mlp(G.retention(), G.dense())], eps=1e-12)
    w = G.weights(cfg)
    w["l0.norm1"][:], w["l0.norm2"][:] = 3.0, 2.0
    toks = rng.integers(0, cfg["vocab"], 6)
    bare, layers = R.forward(dict(cfg, layers=[dict(cfg["layers"][0], mlp=None)]), w, toks)
    x0 = w["embed"][toks] + w["pos"][:6]
    assert np.allclose(np.sqrt(np.mean((layers[0] - x0) ** 2, axis=1)), 3.0, rtol=1e-6)
    w["l0.mlp.up"] *= 7.0
    full, both = R.forward(cfg, w, toks)
    assert np.allclose(np.sqrt(np.mean((both[0] - layers[0]) ** 2, axis=1)), 2.0, rtol=1e-6)
