"""The plain Movazen implementation pinned by what fixes it beside the design's equations, and the framework's
declarations for the design (configuration, tensors, cache and state needs, pages given back, random weights):
everything that needs no GPU."""
import json
import math

import numpy as np
import pytest

import plain_movazen as P
from movazen_models import CONFIGS, SEEDS, make_weights, tensor_shapes, write_folder


# -- the plain mechanisms -------------------------------------------------------------------------------------------

def test_sinusoids_by_hand():
    s = P.sinusoids([0, 1, 7], 6)
    np.testing.assert_array_equal(s[0], [0, 1, 0, 1, 0, 1])
    np.testing.assert_allclose(s[2], [math.sin(7), math.cos(7), math.sin(7 * 10000 ** (-1 / 3)), math.cos(7 * 10000 ** (-1 / 3)),
                                      math.sin(7 * 10000 ** (-2 / 3)), math.cos(7 * 10000 ** (-2 / 3))], atol=1e-15)
    assert P.sinusoids([3], 5).shape == (1, 5)


def test_the_window_keeps_the_first_keys():
    seen = P.visible(8, 3, 2)
    assert seen[1].tolist() == [True, True] + [False] * 6
    assert seen[3].tolist() == [True, True, True, True] + [False] * 4          # 0 and 1 kept, 1 .. 3 in the window
    assert seen[6].tolist() == [True, True, False, False, True, True, True, False]
    assert P.visible(5)[4].all() and not P.visible(5)[3, 4]
    assert P.visible(5, 2, 0)[4].tolist() == [False, False, False, True, True]


def test_slopes_halve_in_equal_steps_and_end_at_two_to_the_minus_eight():
    from runtime.parts import distance_slopes
    np.testing.assert_allclose(P.head_slopes(8), [2.0 ** -(h + 1) for h in range(8)])
    assert P.head_slopes(3)[-1] == 2.0 ** -8
    for H in (1, 6, 20):
        np.testing.assert_allclose(distance_slopes(H), P.head_slopes(H), rtol=1e-15)


def test_one_head_by_hand_with_slope_and_sink():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((4, 1, 3)), rng.standard_normal((4, 1, 3)), rng.standard_normal((4, 1, 2))
    got = P.softmax_heads(q, k, v, 0.5, P.visible(4), slopes=np.array([0.25]), sink=0.0)[3, 0]
    e = [math.exp(0.5 * float(q[3, 0] @ k[j, 0]) - 0.25 * (3 - j)) for j in range(4)]
    np.testing.assert_allclose(got, sum(e[j] * v[j, 0] for j in range(4)) / (1.0 + sum(e)), rtol=1e-12)
    # without a sink a slope on the key's position alone is the same
    a = P.softmax_heads(q, k, v, 0.5, P.visible(4), slopes=np.array([0.25]))[3, 0]
    f = [math.exp(0.5 * float(q[3, 0] @ k[j, 0]) + 0.25 * j) for j in range(4)]
    np.testing.assert_allclose(a, sum(f[j] * v[j, 0] for j in range(4)) / sum(f), rtol=1e-12)


def test_query_heads_read_their_group_s_key_head():
    rng = np.random.default_rng(1)
    q, k, v = rng.standard_normal((5, 6, 4)), rng.standard_normal((5, 2, 4)), rng.standard_normal((5, 2, 3))
    got = P.softmax_heads(q, k, v, 1.0, P.visible(5))
    again = P.softmax_heads(q, np.repeat(k, 3, axis=1), np.repeat(v, 3, axis=1), 1.0, P.visible(5))
    np.testing.assert_allclose(got, again)


def test_temperature_rises_in_steps():
    t = P.temperature(np.arange(12), 0.3, 5)
    assert t[:4].tolist() == [1.0] * 4                                   # p + 1 below the step: ln 1
    np.testing.assert_allclose(t[4:9], 1 + 0.3 * math.log(2))
    np.testing.assert_allclose(t[9:], 1 + 0.3 * math.log(3))


def test_the_memory_against_its_sum_and_with_a_carried_state():
    rng = np.random.default_rng(2)
    q, k, v = (rng.standard_normal((9, n)) for n in (4, 4, 3))
    o, S = P.decayed_memory(q, k, v, 0.8)
    for t in range(9):
        np.testing.assert_allclose(o[t], sum(0.8 ** (t - j) * (q[t] @ k[j]) * v[j] for j in range(t + 1)), atol=1e-12)
    first, half = P.decayed_memory(q[:4], k[:4], v[:4], 0.8)
    second, end = P.decayed_memory(q[4:], k[4:], v[4:], 0.8, half)
    np.testing.assert_allclose(np.concatenate([first, second]), o, atol=1e-12)
    np.testing.assert_allclose(end, S, atol=1e-12)


def test_an_expert_s_clamps_by_hand():
    w = {"e.gate": np.eye(1), "e.up": np.array([[2.0]]), "e.down": np.array([[3.0]])}
    for x in (-4.0, -0.3, 0.2, 5.0):
        g, u = min(x, 1.5), max(-1.5, min(2.0 * x, 1.5))
        want = 3.0 * g / (1.0 + math.exp(-1.702 * g)) * (u + 1.0)
        assert abs(P.clamped_expert(np.array([[x]]), w, "e", 1.5)[0, 0] - want) < 1e-12


def test_routing_by_pairs_of_a_group_with_negative_choices():
    logit = lambda s: np.log(np.asarray(s) / (1 - np.asarray(s)))
    s = np.array([[0.9, 0.1, 0.6, 0.5, 0.3, 0.2]])
    # groups (0, 1), (2, 3), (4, 5): the best pair is the second although the best single score is in the first
    chosen, weights, _ = P.route(logit(s), np.zeros(6), 2, {"count": 3, "keep": 1})
    assert chosen[0].tolist() == [2, 3]
    np.testing.assert_allclose(weights[0], [0.6 / 1.1, 0.5 / 1.1])
    # choice scores may be negative: a dropped group counts as minus infinity, so a kept negative score is chosen before it
    chosen, weights, _ = P.route(logit(s), np.array([-2.0, -2.0, 0.0, -3.0, -2.5, -2.5]), 2, {"count": 3, "keep": 1})
    assert chosen[0].tolist() == [2, 3]
    np.testing.assert_allclose(weights[0], [0.6 / 1.1, 0.5 / 1.1])       # the weights are the scores without the correction
    # groups of one expert: the score of a group is that expert's
    chosen, _, _ = P.route(logit(s), np.zeros(6), 2, {"count": 6, "keep": 3})
    assert chosen[0].tolist() == [0, 2]
    chosen, weights, _ = P.route(logit(s), np.zeros(6), 6)
    np.testing.assert_allclose(weights[0].sum(), 1.0)


def test_the_side_s_part_of_a_row_belongs_to_its_layer():
    rng = np.random.default_rng(3)
    w = {"side.embed": rng.standard_normal((5, 6)), "l1.side.gate": rng.standard_normal((3, 4)), "l1.side.proj": rng.standard_normal((4, 3)),
         "l1.side.norm": np.ones(4)}
    x = rng.standard_normal((2, 4))
    got = P.token_side(x, np.array([4, 0]), w, "l1", 1, 3, 0.0)
    z = w["l1.side.gate"] @ x[0]
    g = 0.5 * z * (1 + np.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3))) * w["side.embed"][4, 3:6]
    y = w["l1.side.proj"] @ g
    np.testing.assert_allclose(got[0], y / math.sqrt(np.mean(y * y)), rtol=1e-12)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_later_token_changes_nothing_before_it(name, tmp_path):
    cfg, w = P.read_folder(write_folder(tmp_path / "m", CONFIGS[name], SEEDS[name], sharp=name == "s"))
    tokens = np.random.default_rng(5).integers(0, cfg["vocab"], 40)
    a = P.forward(cfg, w, tokens)
    tokens[30] = (tokens[30] + 1) % cfg["vocab"]
    b = P.forward(cfg, w, tokens)
    np.testing.assert_allclose(a[:30], b[:30], atol=1e-10)
    assert np.abs(a[30:] - b[30:]).max() > 1e-3


# -- the framework's declarations -------------------------------------------------------------------------------------

@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_declared_tensors_and_needs(name):
    from runtime.engine.loading import build_from_config_dict
    from runtime.cache.pages import KeptWindowNeed, KVNeed, StateNeed
    arch, config, model = build_from_config_dict(CONFIGS[name])
    assert arch.name == "Movazen" and type(config).from_dict(config.to_dict()) == config
    assert {s.name: tuple(s.shape) for s in model.tensor_specs()} == tensor_shapes(CONFIGS[name])
    caches, states = model.cache_needs(), model.state_needs()
    for i, layer in enumerate(CONFIGS[name]["layers"]):
        m = layer["mixer"]
        a = m if layer["type"] == "attention" else m["left"]
        pad = -(-max(a["dim"], a["vdim"]) // 8) * 8
        mask = a.get("mask") or {}
        want = KVNeed(a["kv_heads"], pad, mask.get("size"))
        if mask.get("keep_first"):
            want = KeptWindowNeed(a["kv_heads"], pad, mask["size"], mask["keep_first"])
        assert caches[i] == want
        if layer["type"] == "parallel":
            assert states[i] == StateNeed((m["right"]["heads"], m["right"]["dim"], m["right"]["vdim"]), "float32")
        else:
            assert i not in states


@pytest.mark.parametrize("window, keep, page", [(20, 6, 8), (20, 8, 8), (8, 9, 8), (1, 3, 4), (33, 40, 16)])
def test_pages_between_the_kept_keys_and_the_window_go_back(window, keep, page):
    from runtime.cache import CacheManager
    from runtime.cache.pages import KeptWindowNeed
    need = KeptWindowNeed(2, 8, window, keep)
    m = CacheManager({0: need}, 64, page, 2)
    m.create("r")
    rng = np.random.default_rng(1)
    total, most = 0, 0
    for _ in range(60):
        n = int(rng.integers(1, 12))
        m.append_many([("r", n)])
        total += n
        m.trim("r")
        table = m.table(0, "r")
        held = [j for j, p in enumerate(table) if p >= 0]
        most = max(most, len(held))
        # what any token from the next one on can see is there, and no page that holds none of it
        seen = {j for j in range(total) if total - j < window or j < keep}
        assert {j // page for j in seen} <= set(held)
        assert all(any(p * page + o in seen or p * page + o == total for o in range(page)) for p in held)
        m.check()
    assert most <= m.most_pages_held(total, 12)[0]
    m.release("r")
    assert m.free_pages() == [64]


def test_configuration_errors_name_the_place():
    from runtime.config import ConfigError, MovazenConfig

    def broken(change):
        raw = json.loads(json.dumps(CONFIGS["a"]))
        change(raw)
        with pytest.raises(ConfigError) as e:
            MovazenConfig.from_dict(raw)
        return str(e.value)

    assert "layers[0].mixer" in broken(lambda r: r["layers"][0]["mixer"].pop("vdim"))
    assert "kv_heads" in broken(lambda r: r["layers"][0]["mixer"].update(heads=3))
    assert "layers[0].mixer.mask" in broken(lambda r: r["layers"][0]["mixer"]["mask"].update(size=0))
    assert "keep_first" in broken(lambda r: r["layers"][0]["mixer"]["mask"].update(keep_first=-1))
    assert "layers[1].mixer.right.decay" in broken(lambda r: r["layers"][1]["mixer"]["right"].update(decay=[0.5]))
    assert "q_temp" in broken(lambda r: r["layers"][1]["mixer"]["left"]["q_temp"].update(every=0))
    assert "left_scale" in broken(lambda r: r["layers"][1]["mixer"].pop("left_scale"))
    assert "not moe" in broken(lambda r: r["layers"][0]["mlp"].update(kind="dense"))
    assert "limit" in broken(lambda r: r["layers"][0]["mlp"]["shared"].update(limit=0))
    assert "groups" in broken(lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(count=4))
    assert "cannot be chosen" in broken(lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(keep=1))
    assert "neither attention nor parallel" in broken(lambda r: r["layers"][1].update(type="serial"))
    assert "token_side" in broken(lambda r: r.pop("token_side"))
    assert "scale" in broken(lambda r: r["embedding"].pop("scale"))


def test_parts_refuse_what_they_cannot_do():
    from runtime.parts import LightningAttention, NormedGatedAttention, SandwichBlock
    at = dict(name="m", hidden=8, heads=2, kv_heads=1, dim=8, vdim=8, scale=1.0, eps=1e-5)
    for bad in (dict(slopes=[1.0]), dict(sink=[0.0] * 3), dict(keep_first=2), dict(window=4, keep_first=-1), dict(q_temp=(0.1, 0))):
        with pytest.raises(ValueError):
            NormedGatedAttention(**at, **bad)
    with pytest.raises(ValueError):
        NormedGatedAttention(**at).ride(np.zeros((2, 8)))            # rows in the activations' type: nothing may ride
    with pytest.raises(ValueError):
        LightningAttention("m", 8, 2, 4, 4, [0.5], 1e-5)
    with pytest.raises(ValueError):
        SandwichBlock(None, object(), None)


def test_random_weights_mode_writes_a_folder_that_the_plain_implementation_reads(tmp_path):
    from runtime.engine import write_random_model
    from runtime.config import preset
    folder = write_random_model(tmp_path / "r", "movazen-tiny", seed=3)
    cfg, w = P.read_folder(folder)
    assert {k: tuple(v.shape) for k, v in w.items()} == tensor_shapes(preset("movazen-tiny"))
    logits = P.forward(cfg, w, [1, 2, 3, 4, 5])
    assert logits.shape == (5, cfg["vocab"]) and np.isfinite(logits).all()
