"""The two ends of a model: token ids -> residual stream, and wanted rows -> logits.

h[t] = table[id_t] * scale (reference: EmbeddingKernel, src/backends/cuda/ops/layers.cu:465-481, no scale there);
logits = x . W^T in float32 for the wanted rows only (reference: src/model/qwen2.cc:1059-1066 computes all rows
and picks afterwards; a tied head aliases the table, :1335-1336: here the head's tensor simply carries the
embedding's checkpoint name, so both parts are handed the same tensor).
"""
from __future__ import annotations

from typing import List, Optional

import torch

from .. import ops
from .base import EmbeddedRows, Embedding, Head, ParamSpec, register_part


class TokenEmbedding(Embedding):
    """Options: an RMS norm of the row (`norm_eps` not None; its tensor `norm.weight` plus `norm_offset`), and `streams` s:
    the stream is made in s equal copies, float32 [T, s, hidden] (see streams.py)."""

    graph_safe = True

    def __init__(self, vocab_size: int, hidden_size: int, scale: float = 1.0, init_std: float = 0.02,
                 norm_eps: Optional[float] = None, norm_offset: float = 0.0, streams: Optional[int] = None):
        self.vocab_size, self.hidden_size = int(vocab_size), int(hidden_size)
        self.scale, self.init_std = float(scale), float(init_std)
        self.norm_eps, self.norm_offset = None if norm_eps is None else float(norm_eps), float(norm_offset)
        self.streams = None if streams is None else int(streams)
        self.weight = self.norm_weight = None

    def param_specs(self) -> List[ParamSpec]:
        specs = [ParamSpec("weight", (self.vocab_size, self.hidden_size), std=self.init_std)]
        if self.norm_eps is not None:
            specs.append(ParamSpec("norm.weight", (self.hidden_size,), std=0.1, mean=1.0 - self.norm_offset))
        return specs

    def bind(self, tensors, rt) -> None:
        self.weight = tensors["weight"].contiguous()
        if self.norm_eps is not None:
            self.norm_weight = (tensors["norm.weight"].to(torch.float32) + self.norm_offset).contiguous()

    def forward(self, ctx):
        if self.norm_eps is not None or self.streams is not None:
            h = ctx.rt.empty((ctx.num_tokens, self.streams or 1, self.hidden_size), torch.float32)
            ops.embed_norm(h, self.weight, ctx.token_ids, self.norm_weight, self.norm_eps or 0.0, self.scale)
            return h if self.streams is not None else h.squeeze(1)
        h = ctx.rt.empty((ctx.num_tokens, self.hidden_size), torch.float32)
        ops.embed(h, self.weight, ctx.token_ids, self.scale)
        return h

    def again(self, ctx, h):
        if self.norm_eps is not None or self.streams is not None:
            return super().again(ctx, h)
        return EmbeddedRows(self.weight, ctx.token_ids, self.scale)


class LinearHead(Head):
    graph_safe = True

    def __init__(self, vocab_size: int, hidden_size: int, init_std: float = 0.02, scale: float = 1.0):
        self.vocab_size, self.hidden_size, self.init_std = int(vocab_size), int(hidden_size), float(init_std)
        self.scale = float(scale)  # logits = x . W^T * scale, the product in float32
        self.weight = None

    def param_specs(self) -> List[ParamSpec]:
        return [ParamSpec("weight", (self.vocab_size, self.hidden_size), std=self.init_std)]

    def bind(self, tensors, rt) -> None:
        self.weight = tensors["weight"].contiguous()

    def forward(self, ctx, x):
        logits = ctx.rt.linear_f32(x, self.weight)
        return logits if self.scale == 1.0 else logits.mul_(self.scale)


register_part("embedding", "token_embedding", TokenEmbedding)
register_part("head", "linear_head", LinearHead)
