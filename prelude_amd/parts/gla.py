"""Gated linear attention: a recurrent mixer with a decay of its own per token, head and key channel.

With h the mixer's input: q = W_q h dim^(-1/2) and k = W_k h (heads of ``head_dim``), v = W_v h (heads of ``value_dim``), and
alpha = sigmoid(A_2 (A_1 h) + b)^(1 / tau), one number per head and key channel.  Per head

    S_t = diag(alpha_t) S_(t-1) + k_t v_t^T          S [head_dim, value_dim], from zero at a request's start
    o_t = S_t^T q_t

Every head's o over its own sqrt(mean(o^2) + eps), times a weight shared by the heads, times silu(W_g h); then the output
projection.  S is 32-bit and lives in a state slot of the request; decays, recurrence and norm are 32-bit.  Queries, keys,
values, the gate and A_1 h come from one product; A_2 is applied where the decays are made.
"""
from __future__ import annotations

from typing import Optional

import torch

from ..ops import kernels as K
from .base import MATRIX, NORM, VECTOR, Mixer, PartError, StateSpec, TensorReq, register_part


@register_part("mixer", "gated_linear_attention")
class GatedLinearAttention(Mixer):
    LAUNCHES = 5   # merged projection, decays, recurrence, norm and gate, output projection (portions: two passes more)
    GRAPH_SAFE_PORTIONS = True   # launches follow the step's shape alone; rows and state slots are read on the device

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, tau: float, norm_eps: float,
                 rank: Optional[int] = None):
        for name, v in (("hidden_size", hidden_size), ("num_heads", num_heads), ("head_dim", head_dim), ("value_dim", value_dim)):
            if int(v) <= 0:
                raise PartError(f"gated_linear_attention: {name} {v} must be positive")
        if head_dim > 256:
            raise PartError(f"gated_linear_attention: a key width of {head_dim} is more than the 256 the kernels take")
        if not tau > 0:
            raise PartError(f"gated_linear_attention: tau {tau} must be positive")
        self.hidden_size, self.num_heads = int(hidden_size), int(num_heads)
        self.head_dim, self.value_dim = int(head_dim), int(value_dim)
        self.tau, self.norm_eps = float(tau), float(norm_eps)
        # inner size of the decays' two-step projection; None: whatever the tensors have
        self.rank = int(rank) if rank else None
        self.w_in = self.w_o = self.a2 = self.a2_bias = self.out_norm = None

    @property
    def mixed_size(self) -> int:
        return self.num_heads * self.value_dim

    def cache_spec(self):
        return StateSpec((("s", (self.num_heads, self.head_dim, self.value_dim), torch.float32),))

    def tensors(self):
        h, qk, vv = self.hidden_size, self.num_heads * self.head_dim, self.mixed_size
        r = self.rank if self.rank else -1
        return {"q": TensorReq((qk, h), MATRIX), "k": TensorReq((qk, h), MATRIX), "v": TensorReq((vv, h), MATRIX),
                "g": TensorReq((vv, h), MATRIX), "a1": TensorReq((r, h), MATRIX), "a2": TensorReq((qk, r), MATRIX),
                "a2.b": TensorReq((qk,), VECTOR), "norm": TensorReq((self.value_dim,), NORM), "o": TensorReq((h, vv), MATRIX)}

    def input_rows(self, tensors) -> torch.Tensor:
        """The rows of the product of its input this mixer wants, [q | k | v | g | a1]; keeps its other tensors."""
        if tensors["a1"].shape[0] != tensors["a2"].shape[1]:
            raise PartError("gated_linear_attention: the two steps of the decays' projection disagree about their inner size")
        self.a2, self.a2_bias, self.out_norm = tensors["a2"].contiguous(), tensors["a2.b"], tensors["norm"]
        return torch.cat([tensors[n] for n in ("q", "k", "v", "g", "a1")], dim=0)

    def load(self, tensors, dtype, device):
        self.w_in = K.prepare_weight(self.input_rows(tensors).contiguous())
        self.w_o = K.prepare_weight(tensors["o"])

    def mix(self, x, p, off, step, cache, write_cache, out=None, out_scale=1.0):
        """From the product ``p`` of the mixer's input (this mixer's columns start at ``off``) to the normed, gated heads side
        by side [T, heads * value_dim], times ``out_scale``, into ``out`` when given."""
        if not write_cache:
            raise PartError("gated_linear_attention: a run cannot read another run's state; every run keeps its own")
        nh, d, e = self.num_heads, self.head_dim, self.value_dim
        k_off, v_off = off + nh * d, off + 2 * nh * d
        g_off = v_off + nh * e
        o = K.gated_linear_attention(p, off, k_off, v_off, g_off + nh * e, self.a2, self.a2_bias, self.tau, cache.tensors["s"], step,
                                     nh, d, e)
        return K.head_norm_gate(o, p[:, g_off: g_off + nh * e], self.out_norm, self.norm_eps, "silu", out, out_scale)

    def forward(self, x, step, cache, write_cache=True):
        p = K.linear(x, self.w_in)
        return K.linear(self.mix(x, p, 0, step, cache, write_cache), self.w_o, slices_ok=True)
