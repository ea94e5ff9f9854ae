"""Grouped-query attention whose queries, keys and values pass a short causal convolution over time instead of a
rotation, and whose output is gated:

    q | k | v = conv([Wq; Wk; Wv] x + b)              a convolution of a few taps per channel (`ShortConv`)
    q        *= 1 + coef ln(floor((p + 1) / every) + 1)              `temperature`: the only place positions enter
    s_j       = cap tanh(q . k_j scale / cap), j <= p                 `softcap`
    p_j       = exp(s_j) / (1 + sum exp(s))                           `sink_zero`: a sink whose score is 0, with no value
    y         = (concat(sum_j p_j v_j) * sigmoid(Wg x)) . Wo^T        `gate`

The convolution's last inputs are the request's state; keys are cached after it.  An execution that reads another
one's cache (the schedule's `cache_from`) is built with `own_keys` False: it has projections and a convolution for its
queries alone.

Everything after the convolution is `PagedAttention`'s.  Its matrix-core kernels take heads of a multiple of sixteen
numbers whose values are as wide as their keys; a bfloat16 run gives heads of other sizes the next such size when the
weights are bound: rows of zeros after each head's rows of every projection, gate and convolution, columns of zeros in
Wo.  Keys and values then end in zeros, which adds nothing to any score or result.
"""
from __future__ import annotations

from typing import List, Optional, Tuple

import torch

from .. import ops
from .attention import PagedAttention, pad_heads, padded_head
from .base import ParamSpec, StateNeed, register_part
from .dense_mlp import stack_rows
from .short_conv import ShortConv


class ConvAttention(PagedAttention):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int,
                 scale: Optional[float] = None, conv_taps: int = 0, qkv_bias: bool = True, own_keys: bool = True,
                 temperature: Optional[Tuple[float, float]] = None, softcap: float = 0.0, sink_zero: bool = True,
                 gate: bool = True, init_std: float = 0.02, pad: bool = True):
        """`conv_taps` 0: no convolution (one tap of weight one).  `pad` False: heads stay as they are."""
        # (the base's own checks of head sizes are about its step after the product, which is not used here)
        super().__init__(hidden_size, num_heads, num_kv_heads, 2, qkv_bias=False,
                         scale=float(scale) if scale is not None else head_dim ** -0.5, init_std=init_std, softcap=softcap)
        if not (0 < head_dim <= 256 and 0 < value_dim <= 256):
            raise ValueError(f"head_dim {head_dim} and value_dim {value_dim} must be between 1 and 256")
        if temperature is not None and float(temperature[1]) <= 0:
            raise ValueError("the temperature's step must be positive")
        self.key_size, self.value_size, self.qkv_bias = int(head_dim), int(value_dim), bool(qkv_bias)
        # as the kernels and the cache see them (a bfloat16 run widens them when the weights are bound)
        self.head_dim, self.value_dim = self.key_size, self.value_size
        self.taps, self.own_keys, self.pad = int(conv_taps), bool(own_keys), bool(pad)
        self.temperature = None if temperature is None else (float(temperature[0]), float(temperature[1]))
        self.sink_zero, self.has_gate = bool(sink_zero), bool(gate)
        self.names = ("q", "k", "v") if self.own_keys else ("q",)
        self.conv = self.w_in = None

    def _kv_heads(self) -> int:
        return self.num_kv_heads if self.own_keys else 0

    def state_need(self) -> StateNeed:
        channels = (self.num_heads + self._kv_heads()) * self.head_dim + self._kv_heads() * self.value_dim
        return StateNeed((max(1, max(0, self.taps - 1) * channels),), "float32")

    def _runs(self):
        """(name, heads, size in the checkpoint, size in the kernels) of the projections q, k, v."""
        rows = {"q": (self.num_heads, self.key_size, self.head_dim), "k": (self.num_kv_heads, self.key_size, self.head_dim),
                "v": (self.num_kv_heads, self.value_size, self.value_dim)}
        return [(n,) + rows[n] for n in self.names]

    def param_specs(self) -> List[ParamSpec]:
        W, s, O = self.hidden_size, self.init_std, self.num_heads * self.value_size
        specs = []
        for n, heads, size, _ in self._runs():
            specs.append(ParamSpec(f"{n}.weight", (heads * size, W), std=s))
            if self.qkv_bias:
                specs.append(ParamSpec(f"{n}.bias", (heads * size,), std=s))
            if self.taps:
                specs.append(ParamSpec(f"{n}.conv", (heads * size, self.taps), std=0.3))
        if self.has_gate:
            specs.append(ParamSpec("g.weight", (O, W), std=s))
        specs.append(ParamSpec("o.weight", (W, O), std=s))
        return specs

    def bind(self, tensors, rt) -> None:
        H, G = self.num_heads, self._kv_heads()
        if self.pad and rt.dtype == torch.bfloat16:
            self.head_dim = self.value_dim = padded_head(self.key_size, self.value_size)
        weights, biases, convs = [], [], {}
        for n, heads, size, to in self._runs():
            weights.append(pad_heads(tensors[f"{n}.weight"], heads, size, to))
            if self.qkv_bias:
                biases.append(pad_heads(tensors[f"{n}.bias"], heads, size, to))
            taps = tensors[f"{n}.conv"] if self.taps else torch.ones((heads * size, 1), dtype=torch.float32, device=rt.device)
            convs[f"{n}.conv"] = pad_heads(taps, heads, size, to)
        if self.has_gate:
            weights.append(pad_heads(tensors["g.weight"], H, self.value_size, self.value_dim))
        self.w_in = stack_rows(weights)
        self.w_out = pad_heads(tensors["o.weight"], H, self.value_size, self.value_dim, dim=1).contiguous()
        self.conv = ShortConv(H * self.head_dim, G * self.head_dim, G * self.value_dim, self.head_dim, self.value_dim,
                              max(1, self.taps))
        self.conv.bind(convs, names=self.names, bias=stack_rows(biases) if self.qkv_bias else None)
        if self.sink_zero:
            self.sink = torch.zeros(H, dtype=torch.float32, device=rt.device)

    def forward(self, ctx, x, cache):
        rt, T, H = ctx.rt, x.shape[0], self.num_heads
        proj = rt.linear(x, self.w_in)  # q | k | v | gate  (without keys of its own: q | gate)
        C = self.conv.channels
        q = rt.empty((T, H, self.head_dim))
        temperature = None if self.temperature is None else (ctx.positions,) + self.temperature
        if self.own_keys:
            self.conv.apply(ctx, proj, cache.state, q, cache.k, cache.v, slots=ctx.slots[cache.group],
                            temperature=temperature)
        else:
            self.conv.apply(ctx, proj, cache.state, q, q, q, temperature=temperature)  # (no k or v channels to write)
        gate = proj[:, C:] if self.has_gate else None
        out = rt.empty((T, H, self.value_dim))
        self.attend(ctx, q, cache, out, gate=gate)
        return rt.linear(out.view(T, self.out_dim), self.w_out)


register_part("mixer", "conv_attention", ConvAttention)
