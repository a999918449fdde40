"""Token embedding and output head."""
from __future__ import annotations

from typing import Dict

import torch

from ..csrc import ops
from ..errors import ConfigError
from ..weights.loader import WeightSpec
from .base import Part, register_part
from .linear import linear


class Embedding(Part):
    """x[t, :] = float(table[ids[t], :]) * scale, nothing added; scale 1 unless a design names one
    (reference: engine/kernels/embedding_lookup.cu:16-31).  ``positions`` N: a learned vector for each of the first N
    positions of a sequence (``positions`` [N, hidden]) joins the token's before the scale; there are no others, so a
    request cannot grow beyond N tokens."""
    category = "embedding"
    graph_safe = True     # launches kernels only: may run inside a captured graph

    def __init__(self, vocab_size: int, hidden_size: int, scale: float = 1.0, positions: int = 0):
        self.vocab_size, self.hidden_size, self.scale = int(vocab_size), int(hidden_size), float(scale)
        if positions < 0:
            raise ConfigError(f"embedding: {positions} positions")
        self.position_limit = int(positions)      # (0: positions are not looked up here, nothing bounds them)
        self.table = self.places = None

    def weight_specs(self) -> Dict[str, WeightSpec]:
        out = {"weight": WeightSpec((self.vocab_size, self.hidden_size), kind="table")}
        if self.position_limit:
            out["positions"] = WeightSpec((self.position_limit, self.hidden_size), kind="table")
        return out

    def bind(self, tensors, rt) -> None:
        self.table = tensors["weight"]
        if self.position_limit:             # (one kernel reads both: where only one is kept in 32-bit, both are)
            dt = torch.float32 if torch.float32 in (self.table.dtype, tensors["positions"].dtype) else self.table.dtype
            self.table, self.places = self.table.to(dt), tensors["positions"].to(dt).contiguous()

    def forward(self, ctx) -> torch.Tensor:
        if self.places is not None:
            return ops.embed_placed(self.table, self.places, ctx.token_ids, ctx.positions, factor=self.scale)
        return ops.embed_gather(self.table, ctx.token_ids, factor=self.scale)

    def add_to(self, x: torch.Tensor, ctx) -> torch.Tensor:
        """x += the embedding of the step's tokens, in place on the float32 stream."""
        if self.places is not None:
            return ops.embed_placed(self.table, self.places, ctx.token_ids, ctx.positions, factor=self.scale, add_to=x)
        return ops.embed_add(self.table, ctx.token_ids, x, factor=self.scale)

    def beside(self, x: torch.Tensor, ctx, out_dtype: torch.dtype) -> torch.Tensor:
        """[T, 2 H] in ``out_dtype``: the stream's rows, each followed by the embedding of the row's token."""
        if self.places is not None:
            raise ConfigError("embedding: learned positions do not stand beside the stream")
        return ops.embed_beside(x, self.table, ctx.token_ids, out_dtype, factor=self.scale)


class LMHead(Part):
    """logits = h W^T in float32 (reference: engine/src/model.cpp:612-615).  If
    ``tied_to`` names the embedding table's tensor and the file has no weight
    of the head's own, the table is used.  ``softcap`` c: logits = c tanh(logits / c) (0: as they are)."""
    category = "head"
    graph_safe = True     # launches kernels only: may run inside a captured graph

    def __init__(self, vocab_size: int, hidden_size: int, tied_to=None, softcap: float = 0.0):
        self.vocab_size, self.hidden_size, self.tied_to = int(vocab_size), int(hidden_size), tied_to
        self.softcap = float(softcap)
        if self.softcap < 0:
            raise ConfigError(f"output head: softcap {softcap} must not be negative")
        self.weight = None

    def weight_specs(self) -> Dict[str, WeightSpec]:
        return {"weight": WeightSpec((self.vocab_size, self.hidden_size), optional=self.tied_to is not None)}

    def bind(self, tensors, rt) -> None:
        self.weight = ops.StreamedWeight(tensors["weight"])

    accepts_lazy_norm = True

    def forward(self, h) -> torch.Tensor:
        logits = linear(h, self.weight, out_dtype=torch.float32)
        return ops.softcap(logits, self.softcap) if self.softcap else logits


register_part("embedding", "embedding", Embedding)
register_part("head", "lm_head", LMHead)
