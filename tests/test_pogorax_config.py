"""Pogorax without a GPU: its configuration (every key's absence and every impossible value named), the specification built from it
(tensor names and shapes against the plain implementation's own list, caches and state per layer), pages of chunks, and the plain
implementation against itself."""
import copy
import math

import numpy as np
import pytest

import plain_pogorax as pp
from prelude_amd import models  # noqa: F401
from prelude_amd.config import ConfigError, PogoraxConfig
from prelude_amd.config.registry import resolve_architecture
from prelude_amd.models.causal_lm import CausalLM

CONFIGS = [pp.tiny_config_s, pp.tiny_config_u, pp.tiny_config_w]


def build(cfg):
    arch = resolve_architecture(cfg)
    assert arch.name == "pogorax"
    return CausalLM(arch.build_spec(arch.parse_config(cfg)))


@pytest.mark.parametrize("make", CONFIGS)
def test_the_model_asks_for_the_tensors_a_file_holds(make):
    cfg = make()
    req = {n: tuple(r.shape) for n, r in build(cfg).tensor_requests().items()}
    assert req == pp.tensor_shapes(cfg)


def test_what_every_layer_keeps():
    m = build(pp.tiny_config_s())
    assert m.run_cache == [(0, 1), 2, (3, 4), (5, 6), 7] and m.embedding_cache is None
    kinds = [type(c.spec).__name__ for c in m.cache_slots]
    assert kinds == ["ChunkedKVCacheSpec", "StateSpec", "StateSpec", "KVCacheSpec", "StateSpec", "ChunkedKVCacheSpec",
                     "StateSpec", "StateSpec"]
    a = m.cache_slots[0].spec
    assert (a.num_kv_heads, a.head_dim, a.v_dim, a.window, a.chunk) == (2, 16, 24, 20, 20)
    b = m.cache_slots[3].spec
    assert (b.num_kv_heads, b.head_dim, b.v_dim, b.window) == (2, 16, 24, 0) and getattr(b, "chunk", 0) == 0
    shapes = lambda i: {n: s for n, s, _ in m.cache_slots[i].spec.tensors}
    assert shapes(1) == {"s": (3, 16, 24), "n": (3, 16), "m": (3, 2)}
    assert shapes(2) == {"s": (6, 24, 16), "conv": (2, 6 * 16 + 2 * 3 * 24)}
    assert shapes(4) == {"s": (48,), "conv": (4, 48)}
    assert m.needs_state and m.graph_safe and m.graph_safe_portions and not m.atomic_prefill
    one_tap = build(pp.model([pp.mamba2_layer(conv=1), pp.parallel2_layer(conv=1)]))
    assert all("conv" not in {n for n, _, _ in c.spec.tensors} for c in one_tap.cache_slots if hasattr(c.spec, "tensors"))


def test_pages_of_a_chunk_go_when_the_next_one_begins():
    from prelude_amd.cache.manager import CacheError, PageTables, plan_groups
    from prelude_amd.parts.attention import ChunkedKVCacheSpec
    from prelude_amd.parts.base import KVCacheSpec
    t = PageTables(4, [(12, 10, 0, 10), (40, 10)], 0)
    t.open(1)
    n = 0
    for k in (3, 6, 1, 1, 9, 1, 1, 17, 1):
        t.reserve(1, n + k)
        first = n // 10 * 10                           # what the portion's first position still sees
        live = {j for j, p in enumerate(t.table(1, 0)) if p >= 0}
        assert live == set(range(first // 4, -(-(n + k) // 4))), f"{n} + {k}"
        window = {j for j, p in enumerate(t.table(1, 1)) if p >= 0}
        assert live <= window and window == set(range(max(0, n - 9) // 4, -(-(n + k) // 4)))
        n += k
        t.commit(1, n)
        assert t.audit() == ""
    assert t.reservable_len(1) >= n + 8
    t.close(1)
    assert t.audit() == "" and t.free_pages(0) == 12
    with pytest.raises(CacheError, match="chunk"):
        PageTables(4, [(12, 10, 0, 9)], 0)
    with pytest.raises(CacheError, match="chunk"):
        PageTables(4, [(12, 10, 3, 10)], 0)
    specs = [ChunkedKVCacheSpec(2, 16, 20, 24, 20), KVCacheSpec(2, 16, 20, 24), ChunkedKVCacheSpec(2, 16, 20, 24, 20), ChunkedKVCacheSpec(2, 16, 33, 24, 33)]
    groups, of = plan_groups(specs)
    assert of == [0, 1, 0, 2], "a window of as many places is another group than a chunk"


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


def _m(i, *keys):
    return ("layers", i, "mixer", *keys)


@pytest.mark.parametrize("path,named", [
    (("vocab",), "vocab"), (("width",), "width"), (("norm",), "norm"), (("norm", "eps"), "norm.eps"), (("embedding",), "embedding"),
    (("embedding", "scale"), "embedding.scale"), (("layers",), "layers"), (("layers", 0, "type"), "type"), (_m(0), "layers[0].mixer"),
    (_m(0, "left"), "layers[0].mixer.left"), (_m(0, "right"), "layers[0].mixer.right")] +
    [(_m(0, "left", k), f"layers[0].mixer.left.{k}") for k in ("heads", "kv_heads", "dim", "vdim", "scale", "mask")] +
    [(_m(0, "left", "mask", "size"), "layers[0].mixer.left.mask.size")] +
    [(_m(0, "right", k), f"layers[0].mixer.right.{k}") for k in ("heads", "dim", "vdim", "gate_cap")] +
    [(_m(1, k), f"layers[1].mixer.{k}") for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")] +
    [(_m(2, "left", "rot"), "layers[2].mixer.left.rot"), (_m(2, "left", "rot", "base"), "layers[2].mixer.left.rot.base"),
     (_m(2, "left", "rot", "dims"), "layers[2].mixer.left.rot.dims")] +
    [(_m(2, "right", k), f"layers[2].mixer.right.{k}") for k in ("width", "blocks", "conv")] + [(("layers", 0, "mlp", "ff"), "layers[0].mlp.ff")])
def test_a_missing_key_is_named(path, named):
    with pytest.raises(ConfigError, match=named.replace("[", r"\[").replace("]", r"\]").replace(".", r"\.")):
        PogoraxConfig.from_dict(_without(pp.tiny_config_s(), path))


@pytest.mark.parametrize("path,value,named", [
    (_m(0, "left", "kv_heads"), 3, "kv_heads"), (_m(0, "left", "mask", "size"), 0, "mask.size"), (_m(0, "right", "gate_cap"), 0.0, "gate_cap"),
    (_m(1, "groups"), 4, "groups"), (_m(1, "norm_groups"), 5, "norm_groups"), (_m(1, "conv"), 0, "conv"), (_m(2, "left", "rot", "dims"), 7, "rot.dims"),
    (_m(2, "left", "rot", "dims"), 18, "rot.dims"), (_m(2, "right", "blocks"), 5, "blocks"), (("layers", 0, "type"), "retention", "type"),
    (("layers", 0, "mlp", "kind"), "moe", "kind"), (("layers",), [], "layers"), (("embedding", "scale"), "big", "embedding.scale"),
    (("norm", "eps"), 0.0, "norm.eps")])
def test_an_impossible_value_is_named(path, value, named):
    with pytest.raises(ConfigError, match=named.replace(".", r"\.")):
        PogoraxConfig.from_dict(_with(pp.tiny_config_s(), path, value))


def test_what_may_go_unsaid():
    c = PogoraxConfig.from_dict(pp.tiny_config_s())
    assert [lc.ff for lc in c.layers] == [40, 32, 40, 0, 0]
    assert PogoraxConfig.from_dict(_without(pp.tiny_config_s(), ("layers", 0, "mlp"))).layers[0].ff == 0
    still = PogoraxConfig.from_dict(_with(pp.tiny_config_s(), _m(2, "left", "rot", "dims"), 0))
    assert still.layers[2].mixer.left.rot_dims == 0 and build(_with(pp.tiny_config_s(), _m(2, "left", "rot", "dims"), 0)).shared == {}


# ---- the plain implementation against itself -------------------------------------------------------------------------------
def test_chunks_and_rotation():
    see = pp.visible(12, 5)
    assert see[4].tolist() == [True] * 5 + [False] * 7 and see[5].tolist() == [False] * 5 + [True] + [False] * 6
    assert see[11].tolist() == [False] * 10 + [True] * 2 and (pp.visible(12, 12) == pp.visible(12)).all()
    g = np.random.default_rng(0)
    x = g.standard_normal((5, 2, 12))
    y = pp.rotate_pairs(x, [3, 4, 5, 6, 7], 8, 100.0)
    assert np.allclose(y[..., 8:], x[..., 8:])
    # turning leaves a head's root mean square as it is: what the product rests on when it takes it in front of the rotation
    assert np.allclose(pp.rms_unit(y, 1e-3), pp.rotate_pairs(pp.rms_unit(x, 1e-3), [3, 4, 5, 6, 7], 8, 100.0))
    p = pp.rotate_pairs(x, [1] * 5, 4, 100.0)
    assert np.allclose(p[..., 0], x[..., 0] * math.cos(1) - x[..., 1] * math.sin(1))
    assert np.allclose(p[..., 3], x[..., 3] * math.cos(0.1) + x[..., 2] * math.sin(0.1))


def test_the_convolution_and_the_gates():
    g = np.random.default_rng(1)
    x, w, b = g.standard_normal((9, 3)), g.standard_normal((3, 4)), g.standard_normal(3)
    y = pp.short_conv(x, w, b)
    assert np.allclose(y[0], w[:, 3] * x[0] + b) and np.allclose(y[8], sum(w[:, j] * x[5 + j] for j in range(4)) + b)
    z = np.array([-800.0, -30.0, -1.0, 0.0, 1.0, 30.0, 800.0])
    assert np.allclose(pp.log_sigmoid(z)[2:5], np.log(pp.sigmoid(z[2:5]))) and pp.log_sigmoid(z)[0] == -800.0 and pp.softplus(z)[-1] == 800.0
    assert np.allclose(pp.softplus(z) - z, pp.softplus(-z))
    u = math.sqrt(2 / math.pi) * (z[1:6] + 0.044715 * z[1:6] ** 3)
    assert np.allclose(pp.gelu_tanh(z[1:6]), z[1:6] * pp.sigmoid(2 * u))      # the form the kernels take


def test_the_recurrences_are_decayed_sums_and_can_be_cut():
    g = np.random.default_rng(2)
    T, H, d, e = 12, 2, 4, 3
    q, k, v = g.standard_normal((T, H, d)), g.standard_normal((T, H, d)), g.standard_normal((T, H, e))
    dt, A, D = pp.softplus(g.standard_normal((T, H))), np.exp(g.standard_normal(H)), g.standard_normal(H)
    y, S = pp.ssd_recurrence(q, k, v, dt, A, D)
    want = D[:, None] * v
    for t in range(T):
        for j in range(t + 1):
            keep = np.exp(-A * dt[j + 1: t + 1].sum(axis=0)) * dt[j]
            want[t] += (keep * (q[t] * k[j]).sum(-1))[:, None] * v[j]
    assert np.allclose(y, want)
    y1, S1 = pp.ssd_recurrence(q[:5], k[:5], v[:5], dt[:5], A, D)
    y2, S2 = pp.ssd_recurrence(q[5:], k[5:], v[5:], dt[5:], A, D, S1)
    assert np.allclose(np.concatenate([y1, y2]), y) and np.allclose(S2, S)
    # mLSTM: the running maximum leaves the quotient as it is where the sum of keys decides, and floors it by e^-m elsewhere
    i, f = 3 * g.standard_normal((T, H)), pp.log_sigmoid(g.standard_normal((T, H)))
    o, st = pp.mlstm_recurrence(q, k, v, i, f)
    for t in range(T):
        num, den = np.zeros((H, e)), np.zeros(H)
        for j in range(t + 1):
            wgt = np.exp(f[j + 1: t + 1].sum(axis=0) + i[j]) * (q[t] * k[j]).sum(-1)
            num, den = num + wgt[:, None] * v[j], den + wgt
        m = np.log(np.maximum(1.0, 0.0)) + f[: t + 1].sum(axis=0)              # m in front of the first token is 0
        for j in range(t + 1):
            m = np.maximum(m, f[j + 1: t + 1].sum(axis=0) + i[j])
        want_t = num * np.exp(-m)[:, None] / (np.maximum(np.abs(den) * np.exp(-m), np.exp(-m)) + 1e-6)[:, None]
        assert np.allclose(o[t], want_t)
    o1, s1 = pp.mlstm_recurrence(q[:7], k[:7], v[:7], i[:7], f[:7])
    o2, s2 = pp.mlstm_recurrence(q[7:], k[7:], v[7:], i[7:], f[7:], s1)
    assert np.allclose(np.concatenate([o1, o2]), o) and all(np.allclose(a, b) for a, b in zip(s2, st))
    u, r, ii, lam = g.standard_normal((T, 5)), g.random((T, 5)), g.random((T, 5)), g.standard_normal(5)
    s, end = pp.lru_recurrence(u, r, ii, lam)
    a1, e1 = pp.lru_recurrence(u[:4], r[:4], ii[:4], lam)
    a2, e2 = pp.lru_recurrence(u[4:], r[4:], ii[4:], lam, e1)
    assert np.allclose(np.concatenate([a1, a2]), s) and np.allclose(e2, end)
    a0 = np.exp(-8 * r[0] * np.log1p(np.exp(lam)))
    assert np.allclose(s[0], np.sqrt(1 - a0 ** 2) * ii[0] * u[0])


def test_running_maxima_compose():
    """What the gates' kernel rests on: m -> max(f + m, i) twice is one such map with f1 + f2 and max(i1 + f2, i2)."""
    g = np.random.default_rng(3)
    f, i, m = g.standard_normal(50), g.standard_normal(50), 0.3
    A, B, x = 0.0, -np.inf, m
    for a, b in zip(f, i):
        x = max(a + x, b)
        A, B = A + a, max(B + a, b)
    assert abs(max(A + m, B) - x) < 1e-12


@pytest.mark.parametrize("make,branch,edge", [(pp.parallel_layer, "left", True), (pp.parallel_layer, "right", False), (pp.parallel2_layer, "left", False),
                                              (pp.parallel2_layer, "right", False), (pp.mamba2_layer, None, False)])
def test_what_the_edge_tests_rest_on(make, branch, edge):
    """With the other branch muted, a changed token inside the last position's chunk moves its plain logits and one in front of the
    chunk not at all; recurrences and causal attention carry every token."""
    cfg = pp.model([make()])
    w = pp.random_weights(cfg, 60)
    if branch:
        w[f"l0.mix.{'right' if branch == 'left' else 'left'}.out"] *= 0.0
    toks = list(np.random.default_rng(61).integers(0, cfg["vocab"], 58))      # chunks of 20: the last position's begins at 40
    ref = pp.forward(cfg, w, toks)[-1]
    for c, moves in ((40, True), (39, not edge), (30, not edge)):
        t = list(toks)
        t[c] = (t[c] + 1 + c) % cfg["vocab"]
        moved = np.abs(pp.forward(cfg, w, t)[-1] - ref).max()
        assert (moved > 1e-7 * ref.std()) == moves and (moves or moved == 0.0), (make.__name__, branch, c, moved)
