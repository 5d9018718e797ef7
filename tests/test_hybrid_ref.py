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
