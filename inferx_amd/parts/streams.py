"""Hyper-connections: a residual stream kept in several copies x_1 .. x_s (float32 [T, s, width]) in place of one.
Around every sublayer f three small learned tensors say what it reads and how its result comes back:

    u = sum_i a_i x_i;   y = f(norm(u));   x_j <- sum_i M[i, j] x_i + m b_j y      (all copies at once, from the old ones)

with a = `in`, b = `out`, M = `mix` (indexed [from, to]) and m a constant.  At the end of the model the stream is the sum
of the copies.

Nothing is formed between two sublayers: the result travels as a `StreamDelta`, and the next RMS norm brings it back
into the copies, forms what the next sublayer reads (at the end of the model the sum) and normalises that, in one
kernel.  The tensors are used as float32 in every run.
"""
from __future__ import annotations

from typing import List, Optional

import torch

from .. import ops
from .base import LazyDelta, ParamSpec, Part, register_part, resolve_delta


class HyperConnection(Part):
    """The three tensors of one sublayer."""

    graph_safe = True

    def __init__(self, streams: int, factor: float = 1.0):
        if not 1 <= streams <= ops.MAX_STREAMS:
            raise ValueError(f"{streams} streams: between 1 and {ops.MAX_STREAMS}")
        self.streams, self.factor = int(streams), float(factor)
        self.enter = self.mix = self.gain = None

    def param_specs(self) -> List[ParamSpec]:
        s = self.streams
        return [ParamSpec("in", (s,), std=0.3, mean=1.0 / s), ParamSpec("out", (s,), std=0.3, mean=1.0),
                ParamSpec("mix", (s, s), std=0.2, mean=1.0 / s)]

    def bind(self, tensors, rt) -> None:
        f32 = lambda name: tensors[name].to(torch.float32).contiguous()
        self.enter, self.mix, self.gain = f32("in"), f32("mix"), (f32("out") * self.factor).contiguous()


class StreamDelta(LazyDelta):
    """What stands between two sublayers: `result` (a tensor, a sum that is not formed yet, or None at the model's
    start) comes back through `left`, and `entered` says what is read next (None: the plain sum)."""

    def __init__(self, result, left: Optional[HyperConnection], entered: Optional[HyperConnection] = None):
        self.result, self.left, self.entered = result, left, entered

    def then(self, entered: HyperConnection) -> "StreamDelta":
        return StreamDelta(self.result, self.left, entered)

    def materialize(self, ctx):
        raise NotImplementedError("a stream of several copies goes on through a plain RMS norm only")

    def add_rmsnorm(self, ctx, h, weight, eps, rows, out) -> bool:
        y = None if self.result is None else resolve_delta(ctx, self.result)
        left, entered = self.left, self.entered
        ops.stream_norm(h, y, None if left is None else left.mix, None if left is None else left.gain,
                        None if entered is None else entered.enter, weight, out, eps, rows)
        return True


register_part("streams", "hyper_connection", HyperConnection)
