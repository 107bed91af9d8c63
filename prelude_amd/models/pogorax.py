"""Pogorax: from its typed configuration to a model specification.

A decoder whose layers are listed one by one in the configuration.  The embedding is the token's row times a constant, in 32-bit: it
is the stream.  A layer norms the stream (RMS), runs its mixer, norms again and runs a dense gated feed-forward (``gated_mlp``, GELU in
its tanh form); one without a feed-forward is the mixer alone.  The mixer is

* ``mamba2``: Mamba-2's recurrence behind a short convolution (``mamba2``);
* ``parallel``: attention inside chunks of the sequence with a gate on its output (``windowed_attention`` with those parameters)
  beside the matrix memory of xLSTM (``mlstm``);
* ``parallel_2``: causal attention on rotated queries and keys, each over its own root mean square (``windowed_attention``), beside
  Griffin's recurrent block (``griffin_recurrence``).

Both of the latter are half the sum of their members' outputs, each brought to unit RMS over the model width and multiplied by a weight
of its own (``parallel_mixers`` with normed branches): norms, sum and the add into the stream wait for the norm behind.
Tensor names: ``embed``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*`` (``.left.*`` and ``.right.*`` in a parallel layer, their ``.out``
the branches' norm weights), ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from ..config.model_config import PogoraxConfig
from ..config.registry import Architecture, register_architecture
from .spec import LayerSpec, ModelSpec, PartSpec, RunSpec

BRANCH_SCALE = 0.5   # the design fixes this: half the sum of the two branches
# no longest position is part of the design (angles are computed from the position, there is no table); the engine's
# bookkeeping wants a bound, and positions are 32-bit integers
MAX_POSITIONS = 1 << 24


def _attention(cfg: PogoraxConfig, m, positions):
    """(parameters, tensor names) of a parallel layer's left member."""
    params = dict(hidden_size=cfg.width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim, scale=m.scale,
                  norm_eps=cfg.norm_eps)
    if m.chunk:
        return dict(params, chunk=m.chunk, output_gate=True), ("q", "k", "v", "g", "o")
    params["qk_norm"] = "unit"
    if m.rot_dims:
        name = f"rot{m.rot_dims}@{m.rot_base!r}"
        positions.setdefault(name, PartSpec("rotary_frequencies", dict(rotary_dim=m.rot_dims, theta=m.rot_base)))
        params.update(position=name, rotary_dim=m.rot_dims)
    return params, ("q", "k", "v", "o")


def _mixer(cfg: PogoraxConfig, lc, p: str, positions) -> PartSpec:
    h, m, eps = cfg.width, lc.mixer, cfg.norm_eps
    if lc.type == "mamba2":
        return PartSpec("mamba2", dict(hidden_size=h, num_heads=m.heads, value_dim=m.vdim, state_size=m.state, groups=m.groups, conv=m.conv,
                                       norm_eps=eps, norm_groups=m.norm_groups),
                        {n: f"{p}mix.{n}" for n in ("in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm", "o")})
    left, names = _attention(cfg, m.left, positions)
    r = m.right
    if lc.type == "parallel":
        right = dict(kind="mlstm", params=dict(hidden_size=h, num_heads=r.heads, head_dim=r.dim, value_dim=r.vdim, gate_cap=r.gate_cap, norm_eps=eps))
        own = ("q", "k", "v", "g", "i", "i.b", "f", "f.b", "norm", "o")
    else:
        right = dict(kind="griffin_recurrence", params=dict(hidden_size=h, width=r.width, blocks=r.blocks, conv=r.conv))
        own = ("y", "y.b", "x", "x.b", "conv", "conv.b", "ra", "ra.b", "ri", "ri.b", "lam", "o")
    weights = {f"0.{n}": f"{p}mix.left.{n}" for n in names + ("out",)}
    weights.update({f"1.{n}": f"{p}mix.right.{n}" for n in own + ("out",)})
    members = [dict(kind="windowed_attention", params=left, scale=BRANCH_SCALE), dict(right, scale=BRANCH_SCALE)]
    return PartSpec("parallel_mixers", dict(hidden_size=h, members=members, branch_norm_eps=eps), weights)


def _layer_spec(cfg: PogoraxConfig, i: int, lc, positions) -> LayerSpec:
    h, p = cfg.width, f"l{i}."
    norm = lambda name: PartSpec("rms_norm", dict(size=h, eps=cfg.norm_eps, residual_float32=True), {"weight": p + name})
    parts = {"input_norm": norm("norm1"), "mixer": _mixer(cfg, lc, p, positions)}
    if not lc.ff:
        return LayerSpec("prenorm_mixer_only", parts)
    parts["post_mixer_norm"] = norm("norm2")
    parts["ffn"] = PartSpec("gated_mlp", dict(hidden_size=h, intermediate_size=lc.ff, activation="gelu_tanh"),
                            {"gate_proj.weight": p + "mlp.gate", "up_proj.weight": p + "mlp.up", "down_proj.weight": p + "mlp.down"})
    return LayerSpec("prenorm", parts)


def pogorax_spec(cfg: PogoraxConfig) -> ModelSpec:
    h = cfg.width
    positions = {}
    layers = [_layer_spec(cfg, i, lc, positions) for i, lc in enumerate(cfg.layers)]
    return ModelSpec(
        architecture="Pogorax", vocab_size=cfg.vocab, hidden_size=h, max_positions=MAX_POSITIONS, eos_token_ids=(),
        embedding=PartSpec("token_embedding", dict(vocab_size=cfg.vocab, hidden_size=h, scale=cfg.embed_scale), {"weight": "embed"}),
        layers=layers, order=[RunSpec(i) for i in range(len(layers))],
        final_norm=PartSpec("rms_norm", dict(size=h, eps=cfg.norm_eps, residual_float32=True), {"weight": "final.norm"}),
        head=PartSpec("linear_head", dict(vocab_size=cfg.vocab, hidden_size=h), {"weight": "head"}), positions=positions)


POGORAX = register_architecture(Architecture(
    name="pogorax", architecture_aliases=("Pogorax",), model_type_aliases=("pogorax",),
    parse_config=PogoraxConfig.from_dict, build_spec=pogorax_spec))
