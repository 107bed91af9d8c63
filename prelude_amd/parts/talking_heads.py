"""Attention whose heads' scores are mixed before the softmax: score_h <- sum_g T[h, g] score_g with a learned T.

Queries, keys and values come from one product, optionally with biases; queries and keys are optionally brought to unit
RMS per head and multiplied by a weight all heads share, then their first ``rotary_dim`` dimensions are turned in pairs (2i
with 2i + 1) by position; values are optionally divided by their own root mean square per head (and cached so).  The mask is
a sliding window (0: none); the softmax may have a learned sink per head.

The mixing moves to the query side: with G key heads, head h's mixed score is one dot product of
q'_h = [sum_{g reads key head 0} T[h, g] q_g | .. | sum_{g reads key head G - 1} T[h, g] q_g] with all key heads of a token
side by side.  So the cache keeps one key of width G * head_dim a token, which every head reads, beside G value heads
(``SharedValueKVCacheSpec``), the queries are mixed once a token in 32-bit where they are normed and rotated, and what follows
is attention of ``num_heads`` heads over one key head.
"""
from __future__ import annotations

from typing import Optional

import torch

from ..ops import kernels as K
from .attention import SharedValueKVCacheSpec
from .base import MATRIX, NORM, VECTOR, Mixer, PartError, TensorReq, register_part


@register_part("mixer", "talking_heads_attention")
class TalkingHeadsAttention(Mixer):
    LAUNCHES = 5   # merged projection, norms + rotation + mixing + cache write, attention, its merge, output projection
    GRAPH_SAFE_PORTIONS = True

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int, scale: float,
                 norm_eps: float, window: int = 0, position: Optional[str] = None, rotary_dim: int = 0, bias: bool = False,
                 qk_norm: bool = False, value_norm: bool = False, sink: Optional[str] = None):
        if num_heads % num_kv_heads:
            raise PartError(f"talking_heads_attention: {num_heads} heads are not a multiple of {num_kv_heads} KV heads")
        if head_dim < 1 or num_kv_heads * head_dim > K.MASKED_MAX_KEY or not 1 <= value_dim <= K.MASKED_MAX_VALUE:
            raise PartError(f"talking_heads_attention: {num_kv_heads} keys of {head_dim} side by side (at most {K.MASKED_MAX_KEY}) or a "
                            f"value width of {value_dim} (at most {K.MASKED_MAX_VALUE}) is outside what the kernels take")
        if num_heads // num_kv_heads * (head_dim + num_heads) > K.TALKING_MAX_LDS or max(head_dim, value_dim) > K.TALKING_MAX_HEAD:
            raise PartError(f"talking_heads_attention: {num_heads} heads of {head_dim} do not fit the kernel that mixes them")
        if sink not in (None, "learned"):
            raise PartError(f"talking_heads_attention: sink {sink!r} is not one of None, 'learned'")
        self.hidden_size, self.num_heads, self.num_kv_heads = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.head_dim, self.value_dim, self.scale = int(head_dim), int(value_dim), float(scale)
        self.norm_eps, self.window, self.sink = float(norm_eps), int(window or 0), sink
        self.bias, self.qk_norm, self.value_norm = bool(bias), bool(qk_norm), bool(value_norm)
        self.position = position
        self.rotary_dim = int(rotary_dim or 0) if position else 0
        if self.rotary_dim % 2 or self.rotary_dim > self.head_dim:
            raise PartError(f"talking_heads_attention: {self.rotary_dim} rotated dimensions of a head of {self.head_dim}")
        self.rope = None
        self.w_in = self.w_o = self.biases = self.q_norm = self.k_norm = self.talk = self.sinks = None

    @property
    def nq(self) -> int:
        return self.num_heads * self.head_dim

    @property
    def nk(self) -> int:
        return self.num_kv_heads * self.head_dim

    @property
    def mixed_size(self) -> int:
        return self.num_heads * self.value_dim

    def cache_spec(self):
        return SharedValueKVCacheSpec(1, self.nk, self.window, self.value_dim, self.num_kv_heads)

    def bind(self, shared):
        if self.position is not None:
            if self.position not in shared:
                raise PartError(f"talking_heads_attention: the model has no position encoding named {self.position!r}")
            self.rope = shared[self.position]
            if getattr(self.rope, "rotary_dim", None) != self.rotary_dim or not hasattr(self.rope, "inv_freq"):
                raise PartError(f"talking_heads_attention: position encoding {self.position!r} must give the frequencies of "
                                f"{self.rotary_dim} rotated dimensions")

    def tensors(self):
        h, nv = self.hidden_size, self.num_kv_heads * self.value_dim
        t = {"q": TensorReq((self.nq, h), MATRIX), "k": TensorReq((self.nk, h), MATRIX), "v": TensorReq((nv, h), MATRIX),
             "o": TensorReq((h, self.mixed_size), MATRIX), "talk": TensorReq((self.num_heads, self.num_heads), VECTOR)}
        if self.bias:
            t.update({"q.b": TensorReq((self.nq,), VECTOR), "k.b": TensorReq((self.nk,), VECTOR), "v.b": TensorReq((nv,), VECTOR)})
        if self.qk_norm:
            t.update({"q.norm": TensorReq((self.head_dim,), NORM), "k.norm": TensorReq((self.head_dim,), NORM)})
        if self.sink:
            t["sink"] = TensorReq((self.num_heads,), VECTOR)
        return t

    def input_rows(self, tensors) -> torch.Tensor:
        """The rows of the product of its input this mixer wants, [q | k | v]; keeps its other tensors."""
        self.talk = tensors["talk"].contiguous()
        self.biases = tuple(tensors[n] for n in ("q.b", "k.b", "v.b")) if self.bias else None
        if self.qk_norm:
            self.q_norm, self.k_norm = tensors["q.norm"], tensors["k.norm"]
        self.sinks = tensors["sink"] if self.sink else None
        return torch.cat([tensors["q"], tensors["k"], tensors["v"]], dim=0)

    def load(self, tensors, dtype, device):
        self.w_in = K.prepare_weight(self.input_rows(tensors).contiguous())
        self.w_o = K.prepare_weight(tensors["o"])

    def on_matrix_cores(self, q, cache, out) -> bool:
        return (q.dtype == torch.bfloat16 and self.scale > 0 and K.attention_wide_supported(self.nk, self.value_dim, cache.k.shape[2])
                and (out is None or (out.stride(0) % 4 == 0 and out.data_ptr() % 8 == 0)))

    def mix(self, x, p, off, step, cache, write_cache, out=None, out_scale=1.0):
        """From the product ``p`` of its input (its columns start at ``off``) to the heads' outputs side by side
        [T, heads * value_dim], times ``out_scale``, into ``out`` when given."""
        if not write_cache:
            raise PartError("talking_heads_attention: reads no other layer's cache")
        g = step.kv[cache.group]
        q = K.talking_prepare(p, off, off + self.nq, off + self.nq + self.nk, self.biases, self.q_norm, self.k_norm,
                              self.rope.inv_freq if self.rope is not None else None, step.positions, self.talk, g.slots, cache.k,
                              cache.v, self.num_heads, self.num_kv_heads, self.head_dim, self.value_dim, self.rotary_dim,
                              self.value_norm, self.norm_eps)
        if self.on_matrix_cores(q, cache, out) and out_scale == 1.0:
            return K.attention_wide(q, cache.k, cache.v, g, step, self.window, self.scale, sink=self.sinks, out=out)
        return K.attention_masked(q, cache.k, cache.v, g, step, self.window, 0, self.scale, sink=self.sinks, out=out,
                                  out_scale=out_scale)

    def forward(self, x, step, cache, write_cache=True):
        p = K.linear(x, self.w_in)
        return K.linear(self.mix(x, p, 0, step, cache, write_cache), self.w_o, slices_ok=True)
