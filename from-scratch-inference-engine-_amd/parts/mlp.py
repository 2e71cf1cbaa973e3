"""Dense feed-forwards, with and without a gate."""

from __future__ import annotations

import math
from typing import Dict, Optional

import torch

from .. import ops
from .base import FeedForward, ParamDecl, register_part
from ..ops.functions import GEMM_MFMA_SKINNY_BEST_M
from .linear import Linear


@register_part("feed_forward", "gated")
@register_part("feed_forward", "swiglu")
class SwiGLU(FeedForward):
    """down(act(gate(x)) * up(x)), no biases, act = SiLU (src/model/model.cpp:134-138) unless ``activation``
    names another one the kernels know ("gelu_tanh", "relu") or is an ``ops.GateAct`` with constants of its own
    ("clipped": gate and up value cut off at a limit, g sigmoid(slope g) (u + 1)).  gate and up are one
    matrix [2I, H] with their rows interleaved (gate_0, up_0, gate_1, up_1, ...): x is read once,
    and the lane that holds gate_j also holds up_j, so that for a few rows (decoding) SiLU*up
    happens in the product's epilogue and the [T, 2I] intermediate never reaches memory."""

    graph_safe = True

    def __init__(self, hidden_size: int, intermediate_size: int, activation="silu"):
        self.activation = activation
        self._gate_act = ops.gate_act(activation)  # refuses a name the kernels do not know
        self.hidden_size = hidden_size
        self.intermediate_size = intermediate_size
        self.gate_up = Linear(hidden_size, 2 * intermediate_size)
        self.down = Linear(intermediate_size, hidden_size)

    def param_decls(self) -> Dict[str, ParamDecl]:
        return {"gate_up_weight": ParamDecl((2 * self.intermediate_size, self.hidden_size), layout="interleave"),
                "down_weight": ParamDecl((self.hidden_size, self.intermediate_size))}

    @property
    def gate_up_weight(self):
        return self.gate_up.weight

    @gate_up_weight.setter
    def gate_up_weight(self, t):
        self.gate_up.weight = t

    @property
    def down_weight(self):
        return self.down.weight

    @down_weight.setter
    def down_weight(self, t):
        self.down.weight = t

    def prepare(self, device, compute_dtype) -> None:
        copies = bool(self.options.get("weight_copies", True))
        self.gate_up.prepare(copies)
        self.down.prepare(copies)

    def release_optional_memory(self) -> int:
        return self.gate_up.drop_copy() + self.down.drop_copy()

    # rows up to which silu(gate) * up comes from the product that shares x through LDS when the weight
    # has a fragment-ordered copy (beyond: the library's product and a kernel for SiLU*up)
    streamed_swiglu_max_rows = 128

    def forward(self, x: torch.Tensor, ctx) -> torch.Tensor:
        m = x.shape[0]
        if (x.dtype == torch.bfloat16 and self.gate_up.streamed is not None and 0 < m <= self.streamed_swiglu_max_rows
                and self.gate_up.wide_takes(m, 1, gate_up=True)):
            # from the fragment-ordered copy at any number of rows up to 64, and up to 128 where the
            # kernel has the launch shape for it: SiLU*up in the product's epilogue
            act = ops.gemm_mfma_wide_swiglu(x, self.gate_up.streamed, act=self._gate_act)
        elif (x.dtype == torch.bfloat16 and 3 <= m <= GEMM_MFMA_SKINNY_BEST_M and self.hidden_size % 128 == 0
                and self.gate_up.out_features % 4 == 0 and self.gate_up.out_features // 64 >= ops.compute_units()):
            # three rows and more of a matrix that gives every compute unit a workgroup: the kernel that
            # shares x through LDS (one or two rows, and small matrices, are faster in the other)
            act = ops.gemm_mfma_wide_swiglu(x, self.gate_up.weight, act=self._gate_act)
        elif x.dtype == torch.bfloat16 and m <= GEMM_MFMA_SKINNY_BEST_M and self.hidden_size % 8 == 0:
            act = ops.gemm_mfma_skinny_gated(x, self.gate_up.weight, self._gate_act)
        else:
            act = ops.swiglu(self.gate_up(x), act=self._gate_act)
        return self.down.for_residual(act, ctx)


def _softplus(v: float) -> float:
    return max(v, 0.0) + math.log1p(math.exp(-abs(v)))


@register_part("feed_forward", "plain")
class PlainFeedForward(FeedForward):
    """down(act(up(x) + b_up)) + b_down without a gate.  act = xIELU with two learned numbers (p, q) (parameter ``act``):
    softplus(p) z^2 + z / 2 above zero, (1/2 + softplus(q)) (exp(z) - 1 - z) + z / 2 below it; the softpluses are taken
    once, when the weights are loaded.

    Bias and activation happen in the first product's epilogue for the rows that the engine's own products take, in the
    kernel that adds up its partial sums, or in one pass of their own behind the library's product.
    ``defer_bias=True``: the second bias is not added here but left in ``residual_bias`` for the norm that adds this
    part's output to the stream (``HiddenState.delta_bias``), so that the second product may leave partial sums."""

    graph_safe = True

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "xielu", bias: bool = True,
                 defer_bias: bool = False):
        if activation != "xielu":
            raise ValueError(f"feed-forward: unknown activation '{activation}' (xielu)")
        self.hidden_size, self.intermediate_size = hidden_size, intermediate_size
        self.has_bias, self.defer_bias = bool(bias), bool(defer_bias) and bool(bias)
        self.up = Linear(hidden_size, intermediate_size, bias=self.has_bias)
        self.down = Linear(intermediate_size, hidden_size, bias=self.has_bias and not self.defer_bias)
        self.act: Optional[torch.Tensor] = None
        self._act: Optional[ops.PointAct] = None

    def param_decls(self) -> Dict[str, ParamDecl]:
        decls = {"up_weight": ParamDecl((self.intermediate_size, self.hidden_size)),
                 "down_weight": ParamDecl((self.hidden_size, self.intermediate_size)),
                 "act": ParamDecl((2,), "vector", "bias")}
        if self.has_bias:
            decls["up_bias"] = ParamDecl((self.intermediate_size,), "vector", "bias")
            decls["down_bias"] = ParamDecl((self.hidden_size,), "vector", "bias")
        return decls

    up_weight = property(lambda s: s.up.weight, lambda s, t: setattr(s.up, "weight", t))
    up_bias = property(lambda s: s.up.bias, lambda s, t: setattr(s.up, "bias", t))
    down_weight = property(lambda s: s.down.weight, lambda s, t: setattr(s.down, "weight", t))

    @property
    def down_bias(self) -> Optional[torch.Tensor]:
        return self.residual_bias if self.defer_bias else self.down.bias

    @down_bias.setter
    def down_bias(self, t) -> None:
        if self.defer_bias:
            self.residual_bias = t
        else:
            self.down.bias = t

    def prepare(self, device, compute_dtype) -> None:
        p, q = (float(v) for v in self.act.double().cpu())
        self._act = ops.PointAct("xielu", _softplus(p), 0.5 + _softplus(q))
        copies = bool(self.options.get("weight_copies", True))
        self.up.prepare(copies)
        self.down.prepare(copies)

    def release_optional_memory(self) -> int:
        return self.up.drop_copy() + self.down.drop_copy()

    def _activated(self, x: torch.Tensor) -> torch.Tensor:
        m, up = x.shape[0], self.up
        if x.dtype == torch.bfloat16 and m > 0:
            if (up.streamed is not None and ops.gemm_mfma_wide_act_takes(m, up.streamed)
                    and (m <= 48 or self.intermediate_size <= 32 * ops.compute_units())):
                # (a full fourth tile of x keeps a unit busy by itself: with more than a workgroup a unit the product in
                # slices of K, 64 rows of N = 14336, K = 4096 30.7 us against 34.1)
                return ops.gemm_mfma_wide_act(x, up.streamed, up.bias, self._act)
            if m <= GEMM_MFMA_SKINNY_BEST_M and self.hidden_size % 8 == 0:
                return ops.gemm_mfma_skinny_act(x, up.weight, up.bias, self._act)
            sums = up.partial_sums(x) if self.intermediate_size % 4 == 0 else None
            if sums is not None:
                return ops.sum_round(sums, up.bias, self._act)
        y = up(x, skip_bias=True)
        return ops.bias_act(y, up.bias, self._act, out=y)

    def forward(self, x: torch.Tensor, ctx) -> torch.Tensor:
        return self.down.for_residual(self._activated(x), ctx)
