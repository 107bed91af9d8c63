"""Griffin's recurrent block: two branches, one of them through a real-gated linear recurrent unit.

With h the mixer's input and ``width`` channels: y = act(W_y h + b_y), u = conv(W_x h + b_x), a causal convolution per channel with a
bias (zeros before the start, no activation).  u in ``blocks`` equal parts, in each r = sigmoid(A_r u + b_r) and i = sigmoid(A_i u + b_i),

    log a = -8 r softplus(lam),   S_t = a S_(t-1) + sqrt(1 - a^2) i u,   out = W_o (S * y)

with S zero at a request's start also for its first token.  Gates, decays and S are 32-bit; S and the convolution's last inputs live
in a state slot of the request.  The decay's factor of 8 softplus(lam), one a channel, is made once when the weights are loaded.
"""
from __future__ import annotations

import torch

from ..ops import kernels as K
from .base import MATRIX, VECTOR, Mixer, PartError, StateSpec, TensorReq, register_part
from .decay_scan import MAX_TAPS

DECAY_SHARPNESS = 8.0   # the design fixes this


@register_part("mixer", "griffin_recurrence")
class GriffinRecurrence(Mixer):
    LAUNCHES = 5   # merged projection, convolution, gates and single tokens, output projection (portions: carry and scan)
    GRAPH_SAFE_PORTIONS = True   # launches follow the step's shape alone; rows and state slots are read on the device

    def __init__(self, hidden_size: int, width: int, blocks: int, conv: int, activation: str = "gelu_tanh"):
        for name, v in (("hidden_size", hidden_size), ("width", width), ("blocks", blocks), ("conv", conv)):
            if int(v) <= 0:
                raise PartError(f"griffin_recurrence: {name} {v} must be positive")
        if width % blocks:
            raise PartError(f"griffin_recurrence: {blocks} blocks do not divide a width of {width}")
        if conv > MAX_TAPS:
            raise PartError(f"griffin_recurrence: {conv} taps are more than {MAX_TAPS}")
        if activation not in K.GATE_ACTIVATIONS:
            raise PartError(f"griffin_recurrence: activation {activation!r} is not one of {sorted(K.GATE_ACTIVATIONS)}")
        self.hidden_size, self.width, self.blocks, self.conv, self.activation = int(hidden_size), int(width), int(blocks), int(conv), activation
        self.w_in = self.w_o = self.x_bias = self.y_bias = self.conv_weight = self.conv_bias = None
        self.wr = self.wi = self.br = self.bi = self.rate = None

    @property
    def mixed_size(self) -> int:
        return self.width

    def cache_spec(self):
        state = (("s", (self.width,), torch.float32),)
        if self.conv > 1:
            state += (("conv", (self.conv - 1, self.width), torch.float32),)
        return StateSpec(state)

    def tensors(self):
        h, w, b = self.hidden_size, self.width, self.blocks
        t = {"y": TensorReq((w, h), MATRIX), "y.b": TensorReq((w,), VECTOR), "x": TensorReq((w, h), MATRIX), "x.b": TensorReq((w,), VECTOR),
             "conv": TensorReq((w, self.conv), VECTOR), "conv.b": TensorReq((w,), VECTOR), "lam": TensorReq((w,), VECTOR),
             "o": TensorReq((h, w), MATRIX)}
        for n in ("ra", "ri"):
            t[n], t[n + ".b"] = TensorReq((b, w // b, w // b), MATRIX), TensorReq((b, w // b), VECTOR)
        return t

    def input_rows(self, tensors) -> torch.Tensor:
        """The rows of the product of its input this mixer wants, [x | y]; keeps its other tensors."""
        self.x_bias, self.y_bias, self.conv_bias = tensors["x.b"], tensors["y.b"], tensors["conv.b"]
        self.conv_weight = tensors["conv"].t().contiguous()   # [taps, channels]: a tap's weights side by side
        self.wr, self.wi = tensors["ra"].contiguous(), tensors["ri"].contiguous()
        self.br, self.bi = tensors["ra.b"].reshape(-1).contiguous(), tensors["ri.b"].reshape(-1).contiguous()
        self.rate = (DECAY_SHARPNESS * torch.nn.functional.softplus(tensors["lam"].double(), threshold=80.0)).float()
        return torch.cat([tensors["x"], tensors["y"]], dim=0)

    def load(self, tensors, dtype, device):
        self.w_in = K.prepare_weight(self.input_rows(tensors).contiguous())
        self.w_o = K.prepare_weight(tensors["o"])

    def mix(self, x, p, off, step, cache, write_cache, out=None, out_scale=1.0):
        """From the product ``p`` of its input (its columns start at ``off``) to S * y [T, width], times ``out_scale``, into ``out`` when
        given."""
        if not write_cache:
            raise PartError("griffin_recurrence: a run cannot read another run's state; every run keeps its own")
        w = self.width
        u = K.time_conv(p[:, off: off + w], self.conv_weight, cache.tensors.get("conv"), step, in_bias=self.x_bias, bias=self.conv_bias)
        return K.lru_scan(u, self.wr, self.wi, self.br, self.bi, self.rate, cache.tensors["s"], p[:, off + w: off + 2 * w], self.y_bias, step,
                          out, out_scale, self.activation)

    def forward(self, x, step, cache, write_cache=True):
        p = K.linear(x, self.w_in)
        return K.linear(self.mix(x, p, 0, step, cache, write_cache), self.w_o, slices_ok=True)
