"""The plain Guduzen implementation pinned by what fixes it beside the design's equations, and the framework's
declarations for the design (configuration, tensors, cache and state needs, random weights): everything that needs no
GPU."""
import json
import math

import numpy as np
import pytest

import plain_guduzen as P
from guduzen_models import CONFIGS, RANKS, SEEDS, tensor_shapes, write_folder


# -- the plain mechanisms -------------------------------------------------------------------------------------------

def test_streams_are_read_mixed_and_written_from_the_old_ones():
    rng = np.random.default_rng(0)
    X = rng.standard_normal((3, 4, 5))
    w_in, w_out, mix, y = rng.standard_normal(3), rng.standard_normal(3), rng.standard_normal((3, 3)), rng.standard_normal((4, 5))
    np.testing.assert_allclose(P.read_streams(X, w_in), w_in[0] * X[0] + w_in[1] * X[1] + w_in[2] * X[2], rtol=1e-12)
    got = P.write_streams(X, mix, w_out, y)
    for t in range(3):                        # stream t takes column t of the mix
        np.testing.assert_allclose(got[t], mix[0, t] * X[0] + mix[1, t] * X[1] + mix[2, t] * X[2] + w_out[t] * y, rtol=1e-12)
    # with one stream, weights of one: the plain residual sum
    one = P.spread(X[0], 1)
    np.testing.assert_array_equal(P.read_streams(one, [1.0]), X[0])
    np.testing.assert_allclose(P.write_streams(one, np.ones((1, 1)), [1.0], y)[0], X[0] + y, rtol=1e-12)


def test_norm_weights_around_zero():
    x = np.array([[3.0, 4.0]])
    r = math.sqrt(12.5 + 1e-3)
    np.testing.assert_allclose(P.rmsnorm_around_zero(x, [0.0, -0.5], 1e-3), [[3.0 / r, 2.0 / r]], rtol=1e-12)


def test_a_window_holds_itself_and_the_keys_before_it():
    seen = P.window_visible(6, 3)
    assert seen[0].tolist() == [True] + [False] * 5
    assert seen[4].tolist() == [False, False, True, True, True, False]
    assert P.window_visible(4, 1).tolist() == np.eye(4, dtype=bool).tolist()
    assert P.window_visible(3, None)[2].all()


def test_attention_by_hand():
    rng = np.random.default_rng(1)
    H, T, eps = 5, 6, 1e-6
    m = {"heads": 4, "kv_heads": 2, "dim": 3, "vdim": 2, "scale": 0.7, "mask": {"size": 3}}
    w = {"a.q": rng.standard_normal((12, H)), "a.q.b": rng.standard_normal(12), "a.k": rng.standard_normal((6, H)), "a.k.b": rng.standard_normal(6),
         "a.v": rng.standard_normal((4, H)), "a.v.b": rng.standard_normal(4), "a.o": np.eye(8)}
    h = rng.standard_normal((T, H))
    got = P.attention(h, w, "a", m, eps, P.attention_kv(h, w, "a", m, eps))
    t = 5
    for a in range(4):
        g = a // 2
        q = h[t] @ w["a.q"][3 * a:3 * a + 3].T + w["a.q.b"][3 * a:3 * a + 3]
        q = q / math.sqrt((q * q).mean() + eps)
        s, v = [], []
        for j in (3, 4, 5):
            k = h[j] @ w["a.k"][3 * g:3 * g + 3].T + w["a.k.b"][3 * g:3 * g + 3]
            s.append((q @ k) / math.sqrt((k * k).mean() + eps) * 0.7)
            v.append(h[j] @ w["a.v"][2 * g:2 * g + 2].T + w["a.v.b"][2 * g:2 * g + 2])
        e = np.exp(s) / np.exp(s).sum()
        np.testing.assert_allclose(got[t, 2 * a:2 * a + 2], e @ np.array(v), rtol=1e-10)


def test_latent_attention_equals_attention_over_the_latents_themselves():
    """The keys' up-projection moved to the queries and the values' behind the sum: the same numbers (what lets a cache
    hold one latent a token)."""
    rng = np.random.default_rng(2)
    H, T, eps = 6, 7, 1e-6
    m = {"heads": 3, "dim": 4, "vdim": 5, "kv_rank": 6, "q_rank": 4, "scale": 0.4}
    w = {"a.dq": rng.standard_normal((4, H)), "a.dq.norm": rng.standard_normal(4), "a.uq": rng.standard_normal((12, 4)),
         "a.dkv": rng.standard_normal((6, H)), "a.dkv.norm": rng.standard_normal(6), "a.uk": rng.standard_normal((12, 6)),
         "a.uv": rng.standard_normal((15, 6)), "a.o": np.eye(15)}
    h = rng.standard_normal((T, H))
    got = P.latent_attention(h, w, "a", m, eps)
    c = P.rmsnorm(h @ w["a.dkv"].T, w["a.dkv.norm"], eps)
    q = P.rmsnorm(h @ w["a.dq"].T, w["a.dq.norm"], eps) @ w["a.uq"].T
    for a in range(3):
        qc = q[:, 4 * a:4 * a + 4] @ w["a.uk"][4 * a:4 * a + 4]
        p = P.softmax(qc @ c.T * 0.4, P.window_visible(T, None))
        np.testing.assert_allclose(got[:, 5 * a:5 * a + 5], (p @ c) @ w["a.uv"][5 * a:5 * a + 5].T, rtol=1e-9, atol=1e-12)


def test_delta_rule_with_a_decay_a_channel():
    rng = np.random.default_rng(3)
    T, D, V = 5, 3, 4
    q, k, v = rng.standard_normal((T, D)), P.unit(rng.standard_normal((T, D))), rng.standard_normal((T, V))
    g, beta = rng.random((T, D)), rng.random(T)
    # the state as a product of matrices (I - beta k k^T) diag(g) applied to what was written before
    S = np.zeros((D, V))
    for t in range(T):
        A = (np.eye(D) - beta[t] * np.outer(k[t], k[t])) @ np.diag(g[t])
        S = A @ S + beta[t] * np.outer(k[t], v[t])
        np.testing.assert_allclose(P.delta_scan(q[:t + 1], k[:t + 1], v[:t + 1], g[:t + 1], beta[:t + 1])[t], S.T @ q[t], rtol=1e-10)
    # writing with strength one replaces what the key held; decays of one and a repeated key: the last value stays
    e = np.eye(D)[:1].repeat(T, axis=0)
    np.testing.assert_allclose(P.delta_scan(e, e, v, np.ones((T, D)), np.ones(T)), v, rtol=1e-12)


def test_short_convolution_and_channel_decay_by_hand():
    x = np.arange(1.0, 9.0).reshape(4, 2)
    taps = np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 1.0]])
    y = np.array([[100 * 1.0, 2.0], [10 * 1 + 100 * 3.0, 4.0], [1 + 30 + 500.0, 6.0], [3 + 50 + 700.0, 8.0]])
    np.testing.assert_allclose(P.short_conv(x, taps), y / (1 + np.exp(-y)), rtol=1e-12)
    w = {"m.a1": np.array([[2.0]]), "m.a2": np.array([[0.5], [1.0], [-1.0], [0.0]]), "m.dt_bias": np.array([0.0, 1.0, 2.0, -3.0]), "m.A_log": np.array([0.0, math.log(3.0)])}
    g = P.channel_decay(np.array([[1.5]]), w, "m", 2, 2)[0]
    z = 3.0 * np.array([0.5, 1.0, -1.0, 0.0]) + w["m.dt_bias"]
    np.testing.assert_allclose(g.ravel(), np.exp(-np.array([1.0, 1.0, 3.0, 3.0]) * np.log1p(np.exp(z))), rtol=1e-12)


def test_gelu_tanh_gate_and_capped_logits():
    z = np.array([-2.0, 0.0, 0.5, 3.0])
    want = 0.5 * z * (1 + np.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))
    np.testing.assert_allclose(P.gelu_tanh(z), want, rtol=1e-12)
    np.testing.assert_allclose(P.capped(np.array([1e9, -1e9, 1e-6]), 5.0), [5.0, -5.0, 1e-6], rtol=1e-9)


def test_a_row_sees_nothing_later_and_the_cut_of_a_prompt_does_not_matter(tmp_path):
    folder = write_folder(tmp_path / "a", CONFIGS["a"], SEEDS["a"], ranks=RANKS["a"])
    cfg, w = P.read_folder(folder)
    tokens = list(np.random.default_rng(4).integers(0, cfg["vocab"], 40))
    whole = P.forward(cfg, w, tokens)
    np.testing.assert_allclose(P.forward(cfg, w, tokens[:25]), whole[:25], rtol=1e-9, atol=1e-9)
    other = tokens[:30] + [(tokens[30] + 1) % cfg["vocab"]] + tokens[31:]
    np.testing.assert_allclose(P.forward(cfg, w, other)[:30], whole[:30], rtol=1e-9, atol=1e-9)
    assert np.abs(P.forward(cfg, w, other)[30:] - whole[30:]).max() > 1e-3
    assert np.abs(whole).max() < cfg["logit_softcap"]


# -- the framework's declarations -------------------------------------------------------------------------------------

@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_declared_tensors_and_needs(name):
    from runtime.engine.loading import build_from_config_dict
    from runtime.cache.pages import KVNeed
    raw = CONFIGS[name]
    arch, typed, model = build_from_config_dict(raw)
    assert arch.name == "Guduzen"
    specs = {s.name: s for s in model.tensor_specs()}
    shapes = tensor_shapes(raw, RANKS[name])
    assert set(specs) == set(shapes)
    assert all(specs[n].fits(shape) for n, shape in shapes.items())
    assert typed.to_dict() == json.loads(json.dumps(raw))
    caches, states = model.cache_needs(), model.state_needs()
    for i, layer in enumerate(raw["layers"]):
        m = layer["mixer"]
        if layer["type"] == "attention":
            if "kv_from" in m:
                assert i not in caches and model.site_of(i) == m["kv_from"]
                continue
            # a layer keeps as many keys as the one among it and its readers that looks back furthest
            windows = [(other["mixer"].get("mask") or {}).get("size") for j, other in enumerate(raw["layers"])
                       if j == i or other["mixer"].get("kv_from") == i]
            keep = None if None in windows else max(windows)
            assert caches[i] == KVNeed(m["kv_heads"], -(-max(m["dim"], m["vdim"]) // 8) * 8, keep)
        elif layer["type"] == "latent_attention":
            assert caches[i] == KVNeed(1, -(-m["kv_rank"] // 8) * 8)      # one latent a token, whatever the number of heads
        else:
            channels = 2 * m["kv_heads"] * m["dim"] + m["heads"] * m["vdim"]
            assert states[i].shape == (m["heads"] * m["dim"] * m["vdim"] + (m["conv"] - 1) * channels,) and states[i].dtype == "float32"
            assert i not in caches


def test_configuration_errors_name_their_place():
    from runtime.config import ConfigError, GuduzenConfig
    good = json.loads(json.dumps(CONFIGS["a"]))

    def broken(change):
        raw = json.loads(json.dumps(good))
        change(raw)
        with pytest.raises(ConfigError) as err:
            GuduzenConfig.from_dict(raw)
        return str(err.value)

    assert "layers[0].mixer" in broken(lambda r: r["layers"][0]["mixer"].pop("vdim"))
    assert "kv_heads" in broken(lambda r: r["layers"][0]["mixer"].update(heads=3))
    assert "layers[3].mixer" in broken(lambda r: r["layers"][3]["mixer"].pop("kv_rank"))
    assert "layers[1].mixer" in broken(lambda r: r["layers"][1]["mixer"].update(conv=0))
    assert "kv_from" in broken(lambda r: r["layers"][2]["mixer"].update(kv_from=1))          # no attention layer
    assert "kv_from" in broken(lambda r: r["layers"][2]["mixer"].update(kv_from=2))          # itself
    assert "equal layer 0" in broken(lambda r: r["layers"][2]["mixer"].update(vdim=24))
    assert "type" in broken(lambda r: r["layers"][1].update(type="delta"))
    assert "dense" in broken(lambda r: r["layers"][0]["mlp"].update(kind="moe"))
    assert "mask.size" in broken(lambda r: r["layers"][0]["mixer"]["mask"].update(size=0))
    assert "streams" in broken(lambda r: r.update(streams=9))
    assert "logit_softcap" in broken(lambda r: r.update(logit_softcap=0))
    assert "norm" in broken(lambda r: r.pop("norm"))


def test_low_rank_projections_that_disagree_are_named(tmp_path):
    import torch
    from runtime.parts import make_part
    mixer = make_part("mixer", "channel_delta_rule", name="m", hidden=16, heads=2, kv_heads=1, dim=8, vdim=8, taps=2, eps=1e-5)
    tensors = {s.name: torch.zeros(s.drawn_shape()) for s in mixer.tensor_specs()}
    mixer.bind(tensors, torch.float32)
    tensors["m.a2"] = torch.zeros(16, 5)
    with pytest.raises(ValueError, match="a1"):
        mixer.bind(tensors, torch.float32)


def test_arrangement_refuses_parts_that_do_not_read_its_streams():
    from runtime.parts import make_part
    mixer = make_part("mixer", "channel_delta_rule", name="m", hidden=16, heads=2, kv_heads=1, dim=8, vdim=8, taps=2, eps=1e-5)
    plain = make_part("norm", "rmsnorm", name="n", dim=16, eps=1e-5)
    three = make_part("norm", "streams_norm", name="n", dim=16, eps=1e-5, streams=3)
    for norm in (plain, three):
        with pytest.raises(ValueError, match="streams"):
            make_part("block", "hyper_connected", name="l", streams=2, mixer_norm=norm, mixer=mixer)


def test_random_weights_mode_writes_a_folder_that_the_plain_implementation_reads(tmp_path):
    from runtime.engine import write_random_model
    from runtime.config import preset
    folder = write_random_model(tmp_path / "r", "guduzen-tiny", seed=3)
    cfg, w = P.read_folder(folder)
    dim = preset("guduzen-tiny")["layers"][0]["mixer"]["dim"]
    assert {k: tuple(v.shape) for k, v in w.items()} == tensor_shapes(preset("guduzen-tiny"), (dim, dim))
    assert np.abs(w["l0.hc1.mix"] - np.eye(cfg["streams"])).max() < 0.2 and np.abs(w["l0.norm1"]).max() < 0.2
    logits = P.forward(cfg, w, [1, 2, 3, 4, 5])
    assert logits.shape == (5, cfg["vocab"]) and np.isfinite(logits).all()
