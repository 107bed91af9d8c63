"""Pugavik without a GPU: its configuration (every key's absence and every impossible value named), the specification built
from it (tensor names and shapes against the plain implementation's own list, the run order of a looped stretch and where
the embedding is added again, caches and state per run), and the plain implementation against itself."""
import copy
import math

import numpy as np
import pytest

import plain_pugavik as pp
from prelude_amd import models  # noqa: F401
from prelude_amd.config import ConfigError, PugavikConfig
from prelude_amd.config.registry import resolve_architecture
from prelude_amd.models.causal_lm import CausalLM
from prelude_amd.models.pugavik import pugavik_spec, run_order

CONFIGS = [pp.tiny_config_s, pp.tiny_config_u, pp.tiny_config_w]


def build(cfg):
    arch = resolve_architecture(cfg)
    assert arch.name == "pugavik"
    return CausalLM(arch.build_spec(arch.parse_config(cfg)))


@pytest.mark.parametrize("make", CONFIGS)
def test_the_model_asks_for_the_tensors_a_file_holds(make):
    cfg = make()
    req = build(cfg).tensor_requests()
    want = pp.tensor_shapes(cfg)
    assert set(req) == set(want)
    for name, shape in want.items():
        # the inner size of the decays' projection is the tensors' own
        assert len(req[name].shape) == len(shape) and all(a in (-1, b) for a, b in zip(req[name].shape, shape)), name
        if not name.endswith((".a1", ".a2")):
            assert tuple(req[name].shape) == tuple(shape), name
    if any(lc["type"] == "gla" for lc in cfg["layers"]):
        for lc in cfg["layers"]:
            if lc["type"] == "gla":
                lc["mixer"]["rank"] = 6
        req = build(cfg).tensor_requests()
        assert all(tuple(req[n].shape) == s for n, s in pp.tensor_shapes(cfg).items())


def test_the_run_order_of_a_looped_stretch():
    cfg = PugavikConfig.from_dict(pp.tiny_config_s())
    assert run_order(cfg) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]
    assert run_order(cfg) == [(i, t if i == 1 else None) for i, t in pp.run_order(pp.tiny_config_s())]
    spec = pugavik_spec(cfg)
    assert [r.layer for r in spec.order] == [0, 1, 2, 1, 2, 1, 2, 3] and spec.stream_rows == ("loop.step", 3)
    # the embedding once more in front of every pass but the first, the pass's vector in front of every pass
    assert [r.stream_row for r in spec.order] == [None, 0, None, 1, None, 2, None, None]
    assert [r.add_embedding for r in spec.order] == [False, False, False, True, False, True, False, False]
    whole = PugavikConfig.from_dict(pp.tiny_config_u())
    assert [i for i, _ in run_order(whole)] == [0, 1, 2, 3, 0, 1, 2, 3]
    none = PugavikConfig.from_dict(pp.tiny_config_w())
    assert run_order(none) == [(i, None) for i in range(4)] and pugavik_spec(none).stream_rows is None
    empty = pp.tiny_config_w()
    empty["loop"] = {"start": 2, "stop": 2, "times": 4}
    assert [i for i, _ in run_order(PugavikConfig.from_dict(empty))] == [0, 1, 2, 3]
    assert build(empty).tensor_requests()["loop.step"].shape == (4, 36)     # the file holds them all the same
    tail = pp.tiny_config_w()
    tail["loop"] = {"start": 3, "stop": 4, "times": 2}
    assert run_order(PugavikConfig.from_dict(tail)) == [(0, None), (1, None), (2, None), (3, 0), (3, 1)]


def test_every_run_has_caches_and_state_of_its_own():
    m = build(pp.tiny_config_s())
    assert len(m.cache_slots) == 8 and m.embedding_cache is None
    # a mixer beside a feed-forward hands its cache on as the only member that keeps something; alone it is its own
    assert m.run_cache == [(0,), (1,), 2, (3,), 4, (5,), 6, (7,)]
    kinds = [type(c.spec).__name__ for c in m.cache_slots]
    assert kinds == ["SharedValueKVCacheSpec", "StateSpec", "LatentCacheSpec", "StateSpec", "LatentCacheSpec", "StateSpec",
                     "LatentCacheSpec", "SharedValueKVCacheSpec"]
    a = m.cache_slots[0].spec          # one key of all key heads side by side, a value per key head
    assert (a.num_kv_heads, a.head_dim, a.num_value_heads, a.v_dim, a.window) == (1, 32, 2, 24, 24)
    assert m.cache_slots[2].spec.window == 0 and (m.cache_slots[2].spec.rank, m.cache_slots[2].spec.rot) == (40, 8)
    assert m.cache_slots[1].spec.tensors[0][1] == (3, 16, 24)
    assert m.needs_state and m.graph_safe and m.graph_safe_portions and not m.atomic_prefill
    stateless = pp.model([pp.attention_layer(), pp.latent_layer()])
    assert not build(stateless).needs_state


def _without(cfg, path):
    cfg = copy.deepcopy(cfg)
    node = cfg
    for k in path[:-1]:
        node = node[k]
    del node[path[-1]]
    return cfg


def _with(cfg, path, value):
    cfg = copy.deepcopy(cfg)
    node = cfg
    for k in path[:-1]:
        node = node[k]
    node[path[-1]] = value
    return cfg


@pytest.mark.parametrize("path,named", [
    (("vocab",), "vocab"), (("width",), "width"), (("norm",), "norm"), (("norm", "eps"), "norm.eps"), (("embedding",), "embedding"),
    (("embedding", "scale"), "embedding.scale"), (("layers",), "layers"), (("layers", 0, "type"), "type"),
    (("layers", 0, "mixer"), "layers[0].mixer"), (("layers", 0, "mixer", "heads"), "layers[0].mixer.heads"),
    (("layers", 0, "mixer", "kv_heads"), "layers[0].mixer.kv_heads"), (("layers", 0, "mixer", "dim"), "layers[0].mixer.dim"),
    (("layers", 0, "mixer", "vdim"), "layers[0].mixer.vdim"), (("layers", 0, "mixer", "scale"), "layers[0].mixer.scale"),
    (("layers", 0, "mixer", "mask"), "layers[0].mixer.mask"), (("layers", 0, "mixer", "mask", "size"), "layers[0].mixer.mask.size"),
    (("layers", 0, "mixer", "rot", "base"), "layers[0].mixer.rot.base"), (("layers", 0, "mixer", "rot", "dims"), "layers[0].mixer.rot.dims"),
    (("layers", 1, "mixer", "tau"), "layers[1].mixer.tau"), (("layers", 1, "mixer", "vdim"), "layers[1].mixer.vdim"),
    (("layers", 2, "mixer", "kv_rank"), "layers[2].mixer.kv_rank"), (("layers", 2, "mixer", "rot_dim"), "layers[2].mixer.rot_dim"),
    (("layers", 2, "mixer", "rot"), "layers[2].mixer.rot"), (("layers", 2, "mixer", "scale"), "layers[2].mixer.scale"),
    (("layers", 0, "mlp", "ff"), "layers[0].mlp.ff"), (("loop", "times"), "loop.times"), (("loop", "start"), "loop.start"),
    (("loop", "stop"), "loop.stop")])
def test_a_missing_key_is_named(path, named):
    with pytest.raises(ConfigError, match=named.replace("[", r"\[").replace("]", r"\]").replace(".", r"\.")):
        PugavikConfig.from_dict(_without(pp.tiny_config_s(), path))


@pytest.mark.parametrize("path,value,named", [
    (("layers", 0, "mixer", "kv_heads"), 3, "kv_heads"), (("layers", 0, "mixer", "rot", "dims"), 7, "rot.dims"),
    (("layers", 0, "mixer", "rot", "dims"), 18, "rot.dims"), (("layers", 0, "type"), "retention", "type"),
    (("layers", 0, "mlp", "kind"), "moe", "kind"), (("layers", 2, "mixer", "rot", "dims"), 6, "rot.dims"),
    (("layers", 1, "mixer", "tau"), 0.0, "tau"), (("layers", 1, "mixer", "rank"), 0, "rank"), (("loop", "stop"), 5, "loop"),
    (("loop", "start"), 4, "loop"), (("loop", "times"), 0, "loop.times"), (("layers",), [], "layers"),
    (("layers", 0, "mixer", "mask", "size"), 0, "mask.size"), (("embedding", "scale"), "big", "embedding.scale")])
def test_an_impossible_value_is_named(path, value, named):
    with pytest.raises(ConfigError, match=named.replace(".", r"\.")):
        PugavikConfig.from_dict(_with(pp.tiny_config_s(), path, value))


def test_what_may_go_unsaid():
    cfg = pp.tiny_config_s()
    c = PugavikConfig.from_dict(_without(cfg, ("loop",)))
    assert (c.loop_start, c.loop_stop, c.loop_times, c.has_loop) == (0, 0, 1, False)
    c = PugavikConfig.from_dict(_without(cfg, ("layers", 0, "mixer", "rot")))
    assert c.layers[0].mixer.rot_dims == 0
    assert c.layers[2].ff == 0 and c.layers[0].ff == 40 and c.layers[1].mixer.rank is None
    assert PugavikConfig.from_dict(_without(cfg, ("layers", 0, "mlp"))).layers[0].ff == 0


# ---- the plain implementation against itself -------------------------------------------------------------------------------
def test_rotation_in_pairs_and_relative_positions():
    x = np.random.default_rng(0).standard_normal((5, 2, 12))
    y = pp.rotate_pairs(x, [3, 4, 5, 6, 7], 8, 100.0)
    assert np.allclose(y[..., 8:], x[..., 8:]) and np.allclose((y ** 2).sum(-1), (x ** 2).sum(-1))
    assert np.allclose(pp.rotate_pairs(x, [0] * 5, 8, 100.0), x)
    a = pp.rotate_pairs(x[:1], [10], 8, 100.0)[0, 0] @ pp.rotate_pairs(x[1:2], [7], 8, 100.0)[0, 0]
    b = pp.rotate_pairs(x[:1], [110], 8, 100.0)[0, 0] @ pp.rotate_pairs(x[1:2], [107], 8, 100.0)[0, 0]
    assert abs(a - b) < 1e-9                                    # q.k depends on the distance alone
    p = pp.rotate_pairs(x, [1] * 5, 4, 100.0)
    assert np.allclose(p[..., 0], x[..., 0] * math.cos(1) - x[..., 1] * math.sin(1))
    assert np.allclose(p[..., 3], x[..., 3] * math.cos(0.1) + x[..., 2] * math.sin(0.1))


def test_norms_and_the_activation():
    x = np.random.default_rng(1).standard_normal((4, 9)) * 3 + 2
    y = pp.layer_norm(x, np.ones(9), np.zeros(9), 0.0)
    assert np.allclose(y.mean(1), 0) and np.allclose((y ** 2).mean(1), 1)
    assert np.allclose(pp.layer_norm(x, np.full(9, 2.0), np.full(9, 0.5), 0.0), 2 * y + 0.5)
    assert np.allclose((pp.rms_unit(x, 0.0) ** 2).mean(1), 1)
    z = np.array([-4.0, -1.0, 0.0, 1.0, 4.0])
    exact = np.array([0.5 * t * (1 + math.erf(t / math.sqrt(2))) for t in z])
    assert np.abs(pp.gelu_tanh(z) - exact).max() < 2e-3 and pp.gelu_tanh(z)[2] == 0
    u = math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)
    assert np.allclose(pp.gelu_tanh(z), z * pp.sigmoid(2 * u))  # the form the kernels take


def test_window_and_sink():
    g = np.random.default_rng(2)
    s, v = g.standard_normal((30, 30)), g.standard_normal((30, 5))
    assert np.allclose(pp.softmax_sum(s, pp.visible(30, 1), v), v)                 # a window of one: the token's own value
    full, w7 = pp.softmax_sum(s, pp.visible(30), v), pp.softmax_sum(s, pp.visible(30, 7), v)
    assert np.allclose(w7[:7], full[:7]) and not np.allclose(w7[7], full[7])
    s2 = s.copy()
    s2[:, 10] += 5.0                                                                # the key at 10 is seen by 10 .. 16 only
    moved = np.abs(pp.softmax_sum(s2, pp.visible(30, 7), v) - w7).max(1)
    assert (moved[10:17] > 0).all() and (moved[:10] == 0).all() and (moved[17:] == 0).all()
    assert np.allclose(pp.softmax_sum(s, pp.visible(30, 7), v, sink=-60.0), w7)
    assert np.allclose(pp.softmax_sum(s[:1, :1], pp.visible(1), v[:1], sink=float(s[0, 0])), 0.5 * v[:1])


def test_mixed_scores_are_scores_of_mixed_queries():
    """What the product rests on: sum_g T[h, g] (q_g . k_kv(g)) is one dot product with all key heads side by side."""
    g = np.random.default_rng(3)
    H, G, d = 6, 3, 5
    q, k, talk = g.standard_normal((7, H, d)), g.standard_normal((9, G, d)), g.standard_normal((H, H))
    s = pp.mix_scores(np.stack([q[:, a] @ k[:, a // 2].T for a in range(H)]), talk)
    mixed = np.zeros((7, H, G, d))
    for h in range(H):
        for a in range(H):
            mixed[:, h, a // 2] += talk[h, a] * q[:, a]
    assert np.allclose(np.einsum("thx,jx->htj", mixed.reshape(7, H, G * d), k.reshape(9, G * d)), s)
    assert np.allclose(pp.mix_scores(s, np.eye(H)), s)


def test_the_recurrence_is_a_decayed_sum_and_can_be_cut():
    g = np.random.default_rng(4)
    T, H, d, e = 12, 2, 4, 3
    q, k, v, a = g.standard_normal((T, H, d)), g.standard_normal((T, H, d)), g.standard_normal((T, H, e)), g.random((T, H, d))
    o, S = pp.gla_recurrence(q, k, v, a)
    want = np.zeros_like(v)
    for t in range(T):
        for j in range(t + 1):
            keep = np.prod(a[j + 1: t + 1], axis=0)
            want[t] += (q[t] * keep * k[j]).sum(-1, keepdims=True) * v[j]
    assert np.allclose(o, want)
    o1, S1 = pp.gla_recurrence(q[:5], k[:5], v[:5], a[:5])
    o2, S2 = pp.gla_recurrence(q[5:], k[5:], v[5:], a[5:], S1)
    assert np.allclose(np.concatenate([o1, o2]), o) and np.allclose(S2, S)


def test_the_embedding_and_the_loop():
    cfg = pp.tiny_config_s()
    w = pp.random_weights(cfg, 5)
    toks = [3, 70, 70, 12]
    streams = []
    pp.forward(cfg, w, toks, streams)
    assert len(streams) == 8
    w2 = dict(w, **{"loop.step": w["loop.step"].copy()})
    w2["loop.step"][2] += 1.0                        # the third pass's vector: the runs before it are as they were
    other = []
    pp.forward(cfg, w2, toks, other)
    assert all(np.array_equal(a, b) for a, b in zip(streams[:5], other[:5])) and not np.allclose(streams[5], other[5])
    # a pass by hand: the embedding again, the pass's vector, the layer
    e = w["embed"][toks] * 2.0
    x = pp.layer(streams[2] + e + w["loop.step"][1], range(4), cfg, w, 1)
    assert np.allclose(x, streams[3])
    assert np.allclose(pp.layer(streams[0] + w["loop.step"][0], range(4), cfg, w, 1), streams[1])


@pytest.mark.parametrize("make,over,edge", [(pp.attention_layer, dict(window=24), 24), (pp.attention_layer, dict(window=1), 1),
                                            (pp.gla_layer, dict(), None), (pp.latent_layer, dict(), None)])
def test_what_the_edge_tests_rest_on(make, over, edge):
    """In a one-layer model a changed token moves the last plain logits at the window's oldest key and not at all one place
    further back; the recurrence and attention without a window see every token."""
    cfg = pp.model([make(**over)])
    w = pp.random_weights(cfg, 60)
    n = 60
    toks = list(np.random.default_rng(61).integers(0, cfg["vocab"], n))
    ref = pp.forward(cfg, w, toks)[-1]
    for c, moves in ((n - (edge or n - 20), True), (n - edge - 1 if edge else 20, edge is None)):
        t = list(toks)
        t[c] = (t[c] + 1 + c) % cfg["vocab"]
        moved = np.abs(pp.forward(cfg, w, t)[-1] - ref).max()
        assert (moved > 1e-4 * ref.std()) == moves and (moves or moved == 0.0), (make.__name__, c, moved)
