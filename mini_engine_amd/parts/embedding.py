"""Token embedding and output head (reference layers/embed_head.py:5-23)."""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import Head, Norm, ParamSpec, Part


class TokenEmbedding(Part):
    def __init__(self, vocab_size: int, hidden_size: int, scale: float | None = None, norm: Norm | None = None):
        """`scale`: the rows are multiplied by it and come back in float32 (they start the 32-bit stream unrounded). `norm`: the
        rows pass it (one kernel with the lookup) and come back in float32; the two exclude each other."""
        super().__init__()
        if norm is not None and (scale is not None or not hasattr(norm, "row_norm")):
            raise ValueError("a norm on the embedding's rows comes without a scale and runs inside the lookup's kernel (`row_norm`)")
        if norm is not None:
            self.add_child("norm", norm)
        else:
            self.norm = None
        self.vocab_size = vocab_size
        self.hidden_size = hidden_size
        self.scale = None if scale is None else float(scale)
        self.add_param("weight", ParamSpec((vocab_size, hidden_size), init="matrix", dtype="compute"))

    def forward(self, token_ids: torch.Tensor) -> torch.Tensor:
        if self.norm is not None:
            return ops.stream_mix_norm(self.weight, 1, [], None, None, None, self.norm.row_norm(), torch.float32, rows=token_ids, keep=False)[1]
        return ops.gather_rows(self.weight, token_ids) if self.scale is None else ops.gather_rows(self.weight, token_ids, scale=self.scale)


class LMHead(Head):
    """logits = x . W^T in float32. When tied, W is the embedding matrix itself: the same
    tensor, not a copy (reference models/qwen3.py:107-109)."""

    def __init__(self, vocab_size: int, hidden_size: int, tied_to: TokenEmbedding | None = None, softcap: float | None = None):
        """`softcap`: the logits are bent into (-softcap, softcap): z <- softcap * tanh(z / softcap)."""
        super().__init__()
        self.vocab_size = vocab_size
        self.hidden_size = hidden_size
        self.tied_to = tied_to
        self.softcap = None if softcap is None else float(softcap)
        if tied_to is None:
            self.add_param("weight", ParamSpec((vocab_size, hidden_size), init="matrix", dtype="compute"))

    def matrix(self) -> torch.Tensor:
        return self.tied_to.weight if self.tied_to is not None else self.weight

    def forward(self, x: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
        """`out`: a float32 [rows, vocab] tensor to write the logits into (a step with a fixed layout
        keeps one)."""
        z = ops.linear(x, self.matrix(), torch.float32, out=out)
        return z if self.softcap is None else ops.softcap_(z, self.softcap)
