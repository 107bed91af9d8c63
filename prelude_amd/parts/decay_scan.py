"""Recurrent mixers whose state is a matrix per head that decays by one number a token: Mamba-2 and the matrix memory of xLSTM.

``mamba2``: with p = W_in h laid out as [z | x | B | C | dt] (inner = heads * ``value_dim`` columns of z and x, ``groups`` * ``state``
of B and C, one dt a head), [x | B | C] passes a causal convolution per channel with a bias and SiLU, s = softplus(dt + dt_bias), and
per head (head h reads group h / (heads / groups))

    S_t = exp(-exp(A_log) s) S_(t-1) + s B_t x_t^T,   y_t = S_t^T C_t + D x_t

y times silu(z), in ``norm_groups`` equal parts over their own sqrt(mean^2 + eps), times a weight; then the output projection.

``mlstm``: q = W_q h dim^(-1/2), k = W_k h (heads of ``head_dim``), v = W_v h (heads of ``value_dim``), log gates
i = c tanh((W_i h + b_i) / c) and f = log sigmoid(c tanh((W_f h + b_f) / c)), c = ``gate_cap``, one each a head.  With a running maximum
m_t = max(f + m_(t-1), i) that starts at zero,

    S_t = e^(f + m_(t-1) - m_t) S_(t-1) + e^(i - m_t) k v^T,   n_t likewise with k alone
    o_t = S_t^T q / (max(|n_t . q|, e^(-m_t)) + 1e-6)

Every head's o over its own sqrt(mean^2 + eps), times a weight of all heads' size, times sigmoid(W_g h); then the output projection.

Everything behind the projections and the convolution (whose result is kept in the engine's type) is 32-bit; S, n, m and the
convolution's last inputs live in a state slot of the request, zero at its start.
"""
from __future__ import annotations

import torch

from ..ops import kernels as K
from .base import MATRIX, NORM, VECTOR, Mixer, PartError, StateSpec, TensorReq, register_part

MAX_KEY = 256      # widest key of the kernels
MAX_TAPS = 17      # most taps of the convolution
MLSTM_FLOOR = 1e-6   # what the design adds to mLSTM's denominator


def _positive(kind: str, **sizes) -> None:
    for name, v in sizes.items():
        if int(v) <= 0:
            raise PartError(f"{kind}: {name} {v} must be positive")


@register_part("mixer", "mamba2")
class Mamba2(Mixer):
    LAUNCHES = 5   # merged projection, convolution, recurrence, gate and norm, output projection (portions: four more)
    GRAPH_SAFE_PORTIONS = True   # launches follow the step's shape alone; rows and state slots are read on the device

    def __init__(self, hidden_size: int, num_heads: int, value_dim: int, state_size: int, groups: int, conv: int, norm_eps: float,
                 norm_groups: int = 1):
        _positive("mamba2", hidden_size=hidden_size, num_heads=num_heads, value_dim=value_dim, state_size=state_size, groups=groups,
                  conv=conv, norm_groups=norm_groups)
        if num_heads % groups:
            raise PartError(f"mamba2: {num_heads} heads are not a multiple of {groups} groups")
        if num_heads * value_dim % norm_groups:
            raise PartError(f"mamba2: {norm_groups} norm groups do not divide an inner size of {num_heads * value_dim}")
        if state_size > MAX_KEY or conv > MAX_TAPS:
            raise PartError(f"mamba2: a state of {state_size} (at most {MAX_KEY}) or {conv} taps (at most {MAX_TAPS})")
        self.hidden_size, self.num_heads, self.value_dim, self.state_size = int(hidden_size), int(num_heads), int(value_dim), int(state_size)
        self.groups, self.conv, self.norm_eps, self.norm_groups = int(groups), int(conv), float(norm_eps), int(norm_groups)
        self.w_in = self.w_o = self.conv_weight = self.conv_bias = self.dt_bias = self.a_log = self.skip = self.out_norm = None

    @property
    def mixed_size(self) -> int:
        return self.num_heads * self.value_dim

    @property
    def channels(self) -> int:
        """Channels of the convolution, [x | B | C]."""
        return self.mixed_size + 2 * self.groups * self.state_size

    def cache_spec(self):
        state = (("s", (self.num_heads, self.state_size, self.value_dim), torch.float32),)
        if self.conv > 1:
            state += (("conv", (self.conv - 1, self.channels), torch.float32),)
        return StateSpec(state)

    def tensors(self):
        h, c, nh = self.hidden_size, self.channels, self.num_heads
        return {"in": TensorReq((self.mixed_size + c + nh, h), MATRIX), "conv": TensorReq((c, self.conv), VECTOR), "conv.b": TensorReq((c,), VECTOR),
                "dt_bias": TensorReq((nh,), VECTOR), "A_log": TensorReq((nh,), VECTOR), "D": TensorReq((nh,), VECTOR),
                "norm": TensorReq((self.mixed_size,), NORM), "o": TensorReq((h, self.mixed_size), MATRIX)}

    def input_rows(self, tensors) -> torch.Tensor:
        """The rows of the product of its input this mixer wants, [z | x | B | C | dt]; keeps its other tensors."""
        self.conv_weight = tensors["conv"].t().contiguous()   # [taps, channels]: a tap's weights side by side
        self.conv_bias, self.dt_bias, self.a_log = tensors["conv.b"], tensors["dt_bias"], tensors["A_log"]
        self.skip, self.out_norm = tensors["D"], tensors["norm"]
        return tensors["in"]

    def load(self, tensors, dtype, device):
        self.w_in = K.prepare_weight(K.pad_rows(self.input_rows(tensors)).contiguous())
        self.w_o = K.prepare_weight(tensors["o"])

    def mix(self, x, p, off, step, cache, write_cache, out=None, out_scale=1.0):
        """From the product ``p`` of its input (its columns start at ``off``) to the gated, normed heads side by side
        [T, heads * value_dim], times ``out_scale``, into ``out`` when given."""
        if not write_cache:
            raise PartError("mamba2: a run cannot read another run's state; every run keeps its own")
        inner, c, gn = self.mixed_size, self.channels, self.groups * self.state_size
        xbc = K.time_conv(p[:, off + inner: off + inner + c], self.conv_weight, cache.tensors.get("conv"), step, bias=self.conv_bias,
                          activation="silu")
        dt = p[:, off + inner + c: off + inner + c + self.num_heads]
        y = K.ssd_scan(xbc, inner + gn, inner, 0, dt, self.dt_bias, self.a_log, self.skip, cache.tensors["s"], step, self.num_heads,
                       self.groups, self.state_size, self.value_dim)
        return K.gated_group_norm(y.view(y.shape[0], inner), p[:, off: off + inner], self.out_norm, self.norm_groups, self.norm_eps, out,
                                  out_scale)

    def forward(self, x, step, cache, write_cache=True):
        p = K.linear(x, self.w_in)
        return K.linear(self.mix(x, p, 0, step, cache, write_cache), self.w_o, slices_ok=True)


@register_part("mixer", "mlstm")
class MLSTM(Mixer):
    LAUNCHES = 4   # merged projection, recurrence, norm and gate, output projection (portions: three more)
    GRAPH_SAFE_PORTIONS = True

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, gate_cap: float, norm_eps: float):
        _positive("mlstm", hidden_size=hidden_size, num_heads=num_heads, head_dim=head_dim, value_dim=value_dim)
        if head_dim > MAX_KEY:
            raise PartError(f"mlstm: a key width of {head_dim} is more than the {MAX_KEY} the kernels take")
        if not gate_cap > 0:
            raise PartError(f"mlstm: a gate cap of {gate_cap} is not positive")
        self.hidden_size, self.num_heads, self.head_dim, self.value_dim = int(hidden_size), int(num_heads), int(head_dim), int(value_dim)
        self.gate_cap, self.norm_eps = float(gate_cap), float(norm_eps)
        self.w_in = self.w_o = self.i_bias = self.f_bias = self.out_norm = None

    @property
    def mixed_size(self) -> int:
        return self.num_heads * self.value_dim

    def cache_spec(self):
        nh, d, e = self.num_heads, self.head_dim, self.value_dim
        return StateSpec((("s", (nh, d, e), torch.float32), ("n", (nh, d), torch.float32),
                          ("m", (nh, K.mlstm_max_copies(e)), torch.float32)))

    def tensors(self):
        h, qk, vv, nh = self.hidden_size, self.num_heads * self.head_dim, self.mixed_size, self.num_heads
        return {"q": TensorReq((qk, h), MATRIX), "k": TensorReq((qk, h), MATRIX), "v": TensorReq((vv, h), MATRIX), "g": TensorReq((vv, h), MATRIX),
                "i": TensorReq((nh, h), MATRIX), "i.b": TensorReq((nh,), VECTOR), "f": TensorReq((nh, h), MATRIX), "f.b": TensorReq((nh,), VECTOR),
                "norm": TensorReq((vv,), NORM), "o": TensorReq((h, vv), MATRIX)}

    def input_rows(self, tensors) -> torch.Tensor:
        """The rows of the product of its input this mixer wants, [q | k | v | g | i | f]; keeps its other tensors."""
        self.i_bias, self.f_bias, self.out_norm = tensors["i.b"], tensors["f.b"], tensors["norm"]
        return torch.cat([tensors[n] for n in ("q", "k", "v", "g", "i", "f")], dim=0)

    def load(self, tensors, dtype, device):
        self.w_in = K.prepare_weight(K.pad_rows(self.input_rows(tensors)).contiguous())
        self.w_o = K.prepare_weight(tensors["o"])

    def mix(self, x, p, off, step, cache, write_cache, out=None, out_scale=1.0):
        """As ``Mamba2.mix``."""
        if not write_cache:
            raise PartError("mlstm: a run cannot read another run's state; every run keeps its own")
        nh, d, e = self.num_heads, self.head_dim, self.value_dim
        v_off = off + 2 * nh * d
        g_off = v_off + nh * e
        i_off = g_off + nh * e
        t = cache.tensors
        o, den, floor = K.mlstm_scan(p, off, off + nh * d, v_off, i_off, i_off + nh, self.i_bias, self.f_bias, self.gate_cap, t["s"], t["n"], t["m"],
                                     step, nh, d, e, d ** -0.5)
        return K.head_norm_gate(o, p[:, g_off: g_off + nh * e], self.out_norm, self.norm_eps, "sigmoid", out, out_scale, den, floor, MLSTM_FLOOR)

    def forward(self, x, step, cache, write_cache=True):
        p = K.linear(x, self.w_in)
        return K.linear(self.mix(x, p, 0, step, cache, write_cache), self.w_o, slices_ok=True)
