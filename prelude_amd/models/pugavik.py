"""Pugavik: from its typed configuration to a model specification.

A decoder whose layers are listed one by one in the configuration.  The embedding is the token's row times a constant, in
32-bit: it is the stream.  A layer has one layer norm (``layer_norm``); its mixer and its dense feed-forward (``plain_mlp``,
GELU in its tanh form) both read that norm's output and are added to the stream together.  They stand side by side in one
``parallel_mixers``: one product makes what both want of their input, one product adds up both outputs, and the add into
the stream waits for the next norm (the ``prenorm_mixer_only`` block).  A layer without a feed-forward is the mixer alone.
The mixer is

* ``attention``: grouped-query attention under a sliding window whose heads' scores are mixed by a matrix, with biases,
  queries and keys normed per head, rotation in pairs, values over their own root mean square and a sink
  (``talking_heads_attention``);
* ``gla``: gated linear attention with a decay per key channel (``gated_linear_attention``);
* ``latent_attention``: attention through a latent with a shared rotated key part, queries straight from the input
  (``latent_attention`` with ``q_rank`` 0).

The layers ``loop.start .. loop.stop - 1`` run ``loop.times`` times in a row on the same tensors, each pass with caches and
state of its own (one run per pass in the order); in front of a pass the embedding is added to the stream once more (not
in front of the first) and then the pass's vector.
Tensor names: ``embed``, ``loop.step``, ``l<i>.norm1``, ``l<i>.norm1.b``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``,
``final.norm.b``, ``head``.
"""
from __future__ import annotations

from ..config.model_config import PugavikConfig
from ..config.registry import Architecture, register_architecture
from .spec import LayerSpec, ModelSpec, PartSpec, RunSpec

# no longest position is part of the design (angles are computed from the position, there is no table); the engine's
# bookkeeping wants a bound, and positions are 32-bit integers
MAX_POSITIONS = 1 << 24


def _position(positions, dims: int, base: float):
    if not dims:
        return None
    name = f"rot{dims}@{base!r}"
    positions.setdefault(name, PartSpec("rotary_frequencies", dict(rotary_dim=dims, theta=base)))
    return name


def _mixer(cfg: PugavikConfig, lc, positions):
    """(kind, parameters, tensor names) of a layer's mixer; the names are the checkpoint's behind ``l<i>.mix.``."""
    h, m = cfg.width, lc.mixer
    if lc.type == "attention":
        return "talking_heads_attention", dict(
            hidden_size=h, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim, scale=m.scale,
            norm_eps=cfg.norm_eps, window=m.window, position=_position(positions, m.rot_dims, m.rot_base), rotary_dim=m.rot_dims,
            bias=True, qk_norm=True, value_norm=True, sink="learned"), \
            ("q", "q.b", "k", "k.b", "v", "v.b", "q.norm", "k.norm", "talk", "sink", "o")
    if lc.type == "gla":
        return "gated_linear_attention", dict(hidden_size=h, num_heads=m.heads, head_dim=m.dim, value_dim=m.vdim, tau=m.tau,
                                              norm_eps=cfg.norm_eps, rank=m.rank), \
            ("q", "k", "v", "g", "a1", "a2", "a2.b", "norm", "o")
    return "latent_attention", dict(
        hidden_size=h, num_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim, value_dim=m.vdim, kv_rank=m.kv_rank, q_rank=0,
        norm_eps=cfg.norm_eps, scale=m.scale, position=_position(positions, m.rot_dims, m.rot_base), rotary_dim=m.rot_dims), \
        ("q", "dkv", "dkv.norm", "uk", "uv", "o")


def _layer_spec(cfg: PugavikConfig, i: int, lc, positions) -> LayerSpec:
    h, p = cfg.width, f"l{i}."
    norm = PartSpec("layer_norm", dict(size=h, eps=cfg.norm_eps), {"weight": p + "norm1", "bias": p + "norm1.b"})
    kind, params, names = _mixer(cfg, lc, positions)
    if not lc.ff:
        mixer = PartSpec(kind, params, {n: f"{p}mix.{n}" for n in names})
    else:
        members = [dict(kind=kind, params=params),
                   dict(category="ffn", kind="plain_mlp", params=dict(hidden_size=h, intermediate_size=lc.ff, activation="gelu_tanh"))]
        weights = {f"0.{n}": f"{p}mix.{n}" for n in names}
        weights.update({"1.up": p + "mlp.up", "1.o": p + "mlp.down"})
        mixer = PartSpec("parallel_mixers", dict(hidden_size=h, members=members), weights)
    return LayerSpec("prenorm_mixer_only", {"input_norm": norm, "mixer": mixer})


def run_order(cfg: PugavikConfig):
    """The runs in order: (layer, the pass of the loop it opens or None)."""
    n = len(cfg.layers)
    if cfg.loop_stop <= cfg.loop_start:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(cfg.loop_start)]
    for t in range(cfg.loop_times):
        out += [(i, t if i == cfg.loop_start else None) for i in range(cfg.loop_start, cfg.loop_stop)]
    return out + [(i, None) for i in range(cfg.loop_stop, n)]


def pugavik_spec(cfg: PugavikConfig) -> ModelSpec:
    h = cfg.width
    positions = {}
    layers = [_layer_spec(cfg, i, lc, positions) for i, lc in enumerate(cfg.layers)]
    return ModelSpec(
        architecture="Pugavik", vocab_size=cfg.vocab, hidden_size=h, max_positions=MAX_POSITIONS, eos_token_ids=(),
        embedding=PartSpec("token_embedding", dict(vocab_size=cfg.vocab, hidden_size=h, scale=cfg.embed_scale), {"weight": "embed"}),
        layers=layers, order=[RunSpec(i, stream_row=t, add_embedding=bool(t)) for i, t in run_order(cfg)],
        stream_rows=("loop.step", cfg.loop_times) if cfg.has_loop else None,
        final_norm=PartSpec("layer_norm", dict(size=h, eps=cfg.norm_eps), {"weight": "final.norm", "bias": "final.norm.b"}),
        head=PartSpec("linear_head", dict(vocab_size=cfg.vocab, hidden_size=h), {"weight": "head"}),
        positions=positions)


PUGAVIK = register_architecture(Architecture(
    name="pugavik", architecture_aliases=("Pugavik",), model_type_aliases=("pugavik",),
    parse_config=PugavikConfig.from_dict, build_spec=pugavik_spec))
