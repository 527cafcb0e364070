"""Gated feed-forward: down(act(gate x) * up x), act silu (SwiGLU) or the tanh form of gelu.

Reference: csrc/layers/mlp/mlp.cpp:7-38; gate and up are the two halves (gate first) of one fused
projection: csrc/layers/linear/fused_linear.cpp:152-158,177-180.
"""
from __future__ import annotations

from typing import Dict

import torch

from .. import kernels
from .base import BuildContext, DeferredNorm, FeedForward, Param, join_name
from .linear import FusedLinear, Linear
from .registry import register_feed_forward


@register_feed_forward("swiglu")
class SwiGLU(FeedForward):
    records_mixed_steps = True

    def __init__(self, hidden_size: int, intermediate_size: int, bias: bool, ctx: BuildContext,
                 names=("gate_proj", "up_proj", "down_proj"), suffix: str = "weight", activation: str = "silu", whole_output: bool = False):
        self.whole_output = bool(whole_output)     # one [T, hidden] tensor in the activations' dtype, never float32 parts
        kernels.glu_code(activation)
        self.activation = activation
        self.gate_up = FusedLinear(hidden_size, [intermediate_size, intermediate_size], [names[0], names[1]],
                                   bias, ctx, suffix=suffix)
        self.down = Linear(intermediate_size, hidden_size, names[2], bias, ctx, suffix=suffix)

    def named_parameters(self) -> Dict[str, Param]:
        out = dict(self.gate_up.named_parameters())
        out.update(self.down.named_parameters())
        return out

    def takes_deferred(self, rows: int) -> bool:
        return kernels.gateup_resident_ok(rows, self.gate_up.weight)

    def forward(self, x, batch) -> torch.Tensor:
        if isinstance(x, DeferredNorm):   # the norm's division happens in the gate/up kernel's epilogue
            act = kernels.gateup_swiglu_gemm(x.x, self.gate_up.weight, self.gate_up.bias, row_ss=x.sumsq, eps=x.eps,
                                             act=self.activation)
            return self.down.forward(act, allow_parts=not self.whole_output)
        frag = (lambda: self.gate_up.frag_weight("gate_up8")) if kernels.frag_weight_ok(self.gate_up.weight) else None
        act = kernels.gateup_swiglu_gemm(x, self.gate_up.weight, self.gate_up.bias, frag_w=frag, act=self.activation)   # few rows: activation in the epilogue
        if act is not None:
            return self.down.forward(act, allow_parts=not self.whole_output)
        gu = self.gate_up.forward(x)
        if self.down.bias is None and self.activation == "silu" and not self.whole_output:
            fused = kernels.swiglu_gemm(gu, self.down.weight)   # few rows: activation inside the product
            if fused is not None:
                return fused
        return self.down.forward(kernels.swiglu(gu, self.activation), allow_parts=not self.whole_output)


@register_feed_forward("gated_mlp")
class GatedMLP(SwiGLU):
    """The same with the gate's activation named (`activation`: "silu" or "gelu_tanh")."""

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str, bias: bool, ctx: BuildContext, **names):
        super().__init__(hidden_size, intermediate_size, bias, ctx, activation=activation, **names)


@register_feed_forward("activation_mlp")
class ActivationMLP(FeedForward):
    """down(act(up x)) with one of the kernels' activations (`relu2`: the square of relu, `gelu_tanh`, `silu`, ...).
    `whole_output`: the result comes as one [T, hidden] tensor in the activations' dtype, for an arrangement that norms
    it before it is added.  `defer_bias`: the down projection's bias is left to the residual sum (`deferred_bias`), so that the
    product itself may come in parts."""
    records_mixed_steps = True

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str, bias: bool, ctx: BuildContext,
                 names=("up_proj", "down_proj"), suffix: str = "weight", whole_output: bool = False, bias_suffix: str = "bias",
                 defer_bias: bool = False):
        kernels.activation_code(activation)
        self.activation = activation
        self.whole_output = bool(whole_output)
        defer = bool(bias and defer_bias)
        self.up = Linear(hidden_size, intermediate_size, names[0], bias, ctx, suffix=suffix, bias_suffix=bias_suffix)
        self.down = Linear(intermediate_size, hidden_size, names[1], bias and not defer, ctx, suffix=suffix, bias_suffix=bias_suffix)
        self.deferred_name = join_name(names[1], bias_suffix)
        self.deferred_bias = torch.empty((int(hidden_size),), dtype=ctx.dtype, device=ctx.device) if defer else None

    def named_parameters(self) -> Dict[str, Param]:
        out = dict(self.up.named_parameters())
        out.update(self.down.named_parameters())
        if self.deferred_bias is not None:
            out[self.deferred_name] = Param(self.deferred_bias)
        return out

    def forward(self, x, batch) -> torch.Tensor:
        frag = self.up.frag_weight if kernels.frag_weight_ok(self.up.weight) and x.shape[0] <= kernels.TALL_MAX_ROWS else None
        act = kernels.linear_activation(x, self.up.weight, self.up.bias, self.activation, frag_w=frag)
        return self.down.forward(act, allow_parts=not self.whole_output)
