"""What the stream goes through between layers, before a call of the model's schedule."""

from __future__ import annotations

from typing import Dict

import torch

from .. import ops
from .base import Entrance, HiddenState, ParamDecl, register_part
from .linear import Linear


@register_part("entrance", "origin_mix")
class OriginMix(Entrance):
    """x <- W [x; x0] + step[number], x0 the embedding's output: the entrance of pass ``number`` of layers that run
    ``numbers`` times with the same weights.

    The product reads rows [x; x0] in the compute type.  Their second half is written when the step begins, their first by
    the kernel that folds the pending output in (its norm, the float32 sum, one rounding), which also sets the stream
    to step[number]; the product stays pending as a delta on it, unrounded: float32, whole or in partial sums."""

    graph_safe = True

    def __init__(self, hidden_size: int, numbers: int):
        if numbers < 1:
            raise ValueError(f"origin mix: {numbers} passes")
        self.hidden_size, self.numbers = hidden_size, int(numbers)
        self.linear = Linear(2 * hidden_size, hidden_size)
        self.step = None

    def param_decls(self) -> Dict[str, ParamDecl]:
        return {"weight": ParamDecl((self.hidden_size, 2 * self.hidden_size)),
                "step": ParamDecl((self.numbers, self.hidden_size), "vector", "bias")}

    weight = property(lambda s: s.linear.weight, lambda s, t: setattr(s.linear, "weight", t))

    def prepare(self, device, compute_dtype) -> None:
        self.linear.prepare(bool(self.options.get("weight_copies", True)))

    def release_optional_memory(self) -> int:
        return self.linear.drop_copy()

    def begin(self, hidden: HiddenState, ctx) -> None:
        x0 = hidden.residual
        rows = torch.empty((x0.shape[0], 2 * self.hidden_size), dtype=ctx.compute_dtype, device=x0.device)
        ops.round_columns(x0, rows[:, self.hidden_size:])
        ctx.memo[id(self)] = rows

    def forward(self, hidden: HiddenState, ctx, number: int) -> None:
        if hidden.delta2 is not None or hidden.delta_bias is not None or hidden.delta_scale != 1.0:
            raise RuntimeError("origin mix: a second pending delta, a pending bias or a factor is not taken")
        rows = ctx.memo[id(self)]
        post = hidden.delta_norm
        ops.stream_out(hidden.residual, hidden.delta, None if post is None else post.weight, 0.0 if post is None else post.eps,
                       rows[:, :self.hidden_size], self.step[number])
        hidden.delta, hidden.delta_norm = self.linear.for_stream(rows, ctx), None
