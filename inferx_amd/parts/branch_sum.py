"""What one or two branches leave for the residual stream, not added yet, and what the stream passes on its way into a
layer.

A `BranchSum` travels from a block to the norm that reads the stream next.  An RMS norm, or two of them over the same
stream, takes the whole sum in one kernel (`ops.branch_norm`): the branches' results, a last product's bias, the experts'
weighted sum with their shared expert, and at the start of a loop's pass the embedding once more and the pass's vector.
"""
from __future__ import annotations

from typing import List

import torch

from .. import ops
from .base import EmbeddedRows, LazyDelta, ParamSpec, StreamEntry, register_part
from .dense_mlp import BiasedDelta
from .moe import MoeSum


class BranchSum(LazyDelta):
    def __init__(self, *deltas):
        """`deltas`: branches' results (None, tensors or sums that are not formed yet)."""
        self.tensors, self.bias, self.experts, self.unformed = [], None, None, []
        self.again = self.step = None
        for d in deltas:
            self._take(d)

    @staticmethod
    def of(delta):
        """`delta` as a BranchSum, or None for a sum of another kind (which knows itself how to reach the stream)."""
        if isinstance(delta, BranchSum):
            return delta
        return BranchSum(delta) if delta is None or isinstance(delta, (torch.Tensor, BiasedDelta, MoeSum)) else None

    def _take(self, d) -> None:
        if d is None:
            return
        if isinstance(d, BranchSum):
            if d.again is not None or d.step is not None:
                raise ValueError("what enters a layer is added after its branches, not as one of them")
            self.tensors += d.tensors
            self.unformed += d.unformed
            for name in ("bias", "experts"):
                self._take_one(name, getattr(d, name), d)
        elif isinstance(d, BiasedDelta):
            self.tensors.append(d.tensor)
            self._take_one("bias", d.bias, d)
        elif isinstance(d, MoeSum):
            self._take_one("experts", d, d)
        elif isinstance(d, LazyDelta):
            self.unformed.append(d)
        else:
            self.tensors.append(d)

    def _take_one(self, name, value, delta) -> None:
        """The kernel knows one bias and one experts' sum."""
        if value is None:
            return
        if getattr(self, name) is not None:
            raise ValueError(f"two branches with {'biases' if name == 'bias' else 'experts'} in one sum")
        setattr(self, name, value)

    def entered(self, again, step) -> "BranchSum":
        """The same sum with the embedding's result (`EmbeddedRows` or a tensor, or None) and a vector added after it."""
        out = BranchSum(self)
        out.again, out.step = again, step
        return out

    def _shape(self):
        for t in self.tensors:
            return tuple(t.shape)
        if self.experts is not None:
            return self.experts.topk_w.shape[0], self.experts.width
        if isinstance(self.again, EmbeddedRows):
            return self.again.ids.numel(), self.again.table.shape[1]
        return None if self.again is None else tuple(self.again.shape)

    def form(self, ctx, h, norms=(), eps: float = 0.0, rows=None) -> None:
        """h += the sum, and the norms' results ((weight, out) each).  With `rows` only those rows are normalised (the
        model's last norm: nobody reads the stream after it, so whether h is updated does not matter)."""
        tensors = self.tensors + [d.materialize(ctx) for d in self.unformed]
        kind = norms[0][1].dtype if norms else (self.experts.y.dtype if self.experts is not None else
                                                (tensors[0].dtype if tensors else None))
        together = [t for t in tensors if t.dtype == kind][:2]
        for t in tensors:  # (more than two, or of another type than the norms' results)
            if not any(t is u for u in together):
                ops.branch_norm(h, t)
        a, b = (together + [None, None])[:2]
        m, again = self.experts, self.again
        if again is not None:
            again = (again.table, again.ids, again.scale) if isinstance(again, EmbeddedRows) else (again, None, 1.0)
        ops.branch_norm(h, a, b, self.bias, None if m is None else (m.y, m.dest, m.topk_w, m.shared, m.gate), again, self.step,
                        norms, eps, rows)

    def materialize(self, ctx):
        shape = self._shape()
        if shape is None:
            if not self.unformed:  # (a vector alone, for every token)
                return None if self.step is None else self.step.to(torch.float32).expand(ctx.num_tokens, -1).contiguous()
            total = self.unformed[0].materialize(ctx).to(torch.float32, copy=True)
            BranchSum(*self.unformed[1:]).entered(None, self.step).form(ctx, total)
            return total
        total = torch.zeros(shape, dtype=torch.float32, device=ctx.rt.device)
        self.form(ctx, total)
        return total

    def add_rmsnorm(self, ctx, h, weight, eps, rows, out) -> bool:
        self.form(ctx, h, [(weight, out)], eps, rows)
        return True


class LoopEntry(StreamEntry):
    """What is added to the stream before pass `index` of a stretch of layers that runs `times` times: row `index` of a
    learned table, and with `embedding` the embedding's result once more."""

    graph_safe = True

    def __init__(self, width: int, times: int, index: int, embedding: bool, init_std: float = 0.02):
        if not 0 <= index < times:
            raise ValueError(f"pass {index} of {times}")
        self.width, self.times, self.index = int(width), int(times), int(index)
        self.needs_embedding, self.init_std = bool(embedding), float(init_std)
        self.step = None

    def param_specs(self) -> List[ParamSpec]:
        return [ParamSpec("steps", (self.times, self.width), std=self.init_std)]

    def bind(self, tensors, rt) -> None:
        self.step = tensors["steps"][self.index].clone()  # (a buffer of its own: the kernel wants its start aligned)

    def forward(self, ctx, pending, again):
        return BranchSum(pending).entered(again if self.needs_embedding else None, self.step)


register_part("entry", "loop", LoopEntry)
