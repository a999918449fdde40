"""The weighted sum of two mixers of one input."""
from __future__ import annotations

from typing import Dict

import torch

from ..cache.specs import Bundle
from ..csrc import ops
from ..errors import ConfigError
from ..weights.loader import WeightSpec
from .base import Part, build_part, register_part
from .linear import linear


class Parallel(Part):
    """x += left_scale * left(h) + right_scale * right(h).  One input, so the two input products are one, and
    both mixers end in a product that adds to the stream, so these are one as well: a row holds the left one's heads, then the
    right one's, each already times its mixer's scale (in float32, before they are rounded), and an output bias joins
    the product times the scale.  The layer keeps both mixers' caches.  Tensors carry ``left.`` or ``right.`` before their names.

    A mixer that can stand here says ``stands_beside`` and has
      input_names()   the tensors whose rows, one after the other, make its input product
      bind_heads(tensors, rt)   everything else it binds, but for its output matrix ``o``; ``o_b`` is its output bias or None
      heads_width     the columns its heads leave
      run_heads(x, ctx, cache, writes, out, factor)   its heads, times factor, from the input product's float32 rows into out"""
    category = "mixer"
    graph_safe = True     # launches kernels only: may run inside a captured graph
    adds_one_product = True   # the output is one last product through linear(): a block may hand it ops.Fresh
    accepts_lazy_norm = True  # (one product reads the norm)

    def __init__(self, left, right, left_scale: float = 1.0, right_scale: float = 1.0):
        self.sides = {"left": build_part("mixer", left), "right": build_part("mixer", right)}
        self.scales = {"left": float(left_scale), "right": float(right_scale)}
        for name, side in self.sides.items():
            if not getattr(side, "stands_beside", False):
                raise ConfigError(f"parallel mixer: the {name} one ({type(side).__name__}) cannot stand beside another")
        if len({side.hidden_size for side in self.sides.values()}) != 1:
            raise ConfigError("parallel mixer: both mixers read and write one stream, their widths must agree")
        self.hidden_size = self.sides["left"].hidden_size

    def children(self):
        return list(self.sides.values())

    def cache_spec(self):
        return Bundle(tuple((name, side.cache_spec()) for name, side in self.sides.items()))

    def weight_specs(self) -> Dict[str, WeightSpec]:
        return {f"{name}.{local}": spec for name, side in self.sides.items() for local, spec in side.weight_specs().items()}

    def step_work(self, batch, rows: int, elem: int):
        works = [side.step_work(batch, rows, elem) for side in self.sides.values()]      # (the tensors are the sides')
        return sum(w[0] for w in works), sum(w[1] for w in works)

    def working_bytes_per_row(self, elem: int) -> float:
        """The sides' own, the input product's rows being float32."""
        return sum(side.working_bytes_per_row(elem) + (4 - elem) * sum(spec.shape[0] for local, spec in side.weight_specs().items()
                                                                      if local in side.input_names()) for side in self.sides.values())

    def bind(self, tensors, rt) -> None:
        mine = {name: {local: tensors[f"{name}.{local}"] for local in side.weight_specs()} for name, side in self.sides.items()}
        inputs = {name: [mine[name][n] for n in side.input_names()] for name, side in self.sides.items()}
        self.rows = {name: sum(t.shape[0] for t in parts) for name, parts in inputs.items()}
        self.w_in = ops.StreamedWeight(torch.cat(inputs["left"] + inputs["right"], dim=0).contiguous())
        self.w_o = ops.StreamedWeight(torch.cat([mine[name]["o"] for name in self.sides], dim=1).contiguous())
        self.o_b = None
        for name, side in self.sides.items():
            side.bind_heads(mine[name], rt)
            if side.o_b is not None:
                scaled = side.o_b * self.scales[name]
                self.o_b = scaled if self.o_b is None else self.o_b + scaled
        self.act_dtype = rt.act_dtype

    def wants_prepared_norm(self, n_rows: int) -> bool:
        """Whether the first product is better served by a norm that the product before prepared than by fusing the
        norm or running it: the weight's own plan says (ops.LinearPlan.wants_prepared)."""
        return self.act_dtype == torch.bfloat16 and self.w_in.plan.wants_prepared(n_rows)

    def forward(self, h, ctx, cache, residual, writes: bool = True) -> None:
        x = linear(h, self.w_in, out_dtype=torch.float32)
        left, right = self.sides["left"], self.sides["right"]
        o = torch.empty((x.shape[0], left.heads_width + right.heads_width), dtype=self.act_dtype, device=x.device)
        left.run_heads(x[:, :self.rows["left"]], ctx, cache.left, writes, out=o[:, :left.heads_width], factor=self.scales["left"])
        right.run_heads(x[:, self.rows["left"]:], ctx, cache.right, writes, out=o[:, left.heads_width:], factor=self.scales["right"])
        linear(o, self.w_o, accumulate_into=residual, ctx=ctx, bias=self.o_b)


register_part("mixer", "parallel", Parallel)
