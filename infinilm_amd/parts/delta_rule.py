"""The gated delta rule: a linear attention whose state forgets by a decay computed from the input and is corrected by what
it already holds under a token's key.

  projections without bias: kv_heads query and key heads of dim entries, heads value heads of vdim entries (consecutive
        value heads share a query/key head)
  a short causal convolution per channel of q, k and v (`conv_taps` inputs, the last the token's own, zeros before a
        sequence's start; no bias), then silu
  every query and key head divided by its length (the root of its sum of squares + unit_eps), queries by sqrt(dim) too
  per value head a strength beta_t in (0, 1), sigmoid of its projection, and a decay g_t: log g_t = -exp(A_log)
        softplus(projection + dt_bias)
  per value head a matrix M [dim, vdim], zero before a sequence's start; with the vectors of token t as rows
        D_t = g_t M_{t-1},   c_t = beta_t (v_t - k_t D_t),   M_t = D_t + outer(k_t, c_t),   y_t = q_t M_t
  y_t divided by its root mean square, times norm [vdim] and silu of a gate's projection, per head; then the output product.

Two states a request, float32 rows of the cache manager's pools: the convolution's last conv_taps - 1 inputs, and M as
[heads, vdim, dim].  Everything between the projections is float32 whatever the activations' dtype.
"""
from __future__ import annotations

from typing import Dict, Sequence

import torch

from .. import kernels
from ..cache.needs import FixedState
from .base import BuildContext, Mixer, Param
from .linear import FusedLinear, Linear
from .registry import register_mixer


@register_mixer("gated_delta_rule")
class GatedDeltaRule(Mixer):
    records_mixed_steps = True   # every index comes from the batch's device tensors

    def __init__(self, hidden_size: int, heads: int, kv_heads: int, dim: int, vdim: int, conv_taps: int, eps: float, ctx: BuildContext,
                 unit_eps: float = 1e-6, names: Sequence[str] = ("q", "k", "v", "g", "b", "a", "o", "A_log", "dt_bias", "norm", "conv"),
                 suffix: str = ""):
        self.H, self.G, self.dk, self.dv = int(heads), int(kv_heads), int(dim), int(vdim)
        if self.G <= 0 or self.H % self.G:
            raise ValueError(f"{heads} heads do not divide into {kv_heads} query/key heads")
        if self.dk > kernels.DELTA_MAX_KEY_DIM:
            raise ValueError(f"key size {self.dk} is above the recurrence kernel's {kernels.DELTA_MAX_KEY_DIM}")
        self.taps = int(conv_taps)
        if not 0 <= self.taps <= kernels.CONV_MAX_TAPS:
            raise ValueError(f"{self.taps} taps: the convolution kernel takes up to {kernels.CONV_MAX_TAPS}")
        self.eps, self.unit_eps, self.dtype = float(eps), float(unit_eps), ctx.dtype
        self.names = tuple(names)
        qn, kn, vn, gn, bn, an, on = self.names[:7]
        H, G, dk, dv = self.H, self.G, self.dk, self.dv
        hp = -(-H // 8) * 8                                   # (the per-head rows filled up, so that rows stay 16-byte aligned)
        self.C = 2 * G * dk + H * dv
        self.b_off, self.a_off = self.C + H * dv, self.C + H * dv + hp
        self.proj = FusedLinear(hidden_size, [G * dk, G * dk, H * dv, H * dv, hp, hp], [qn, kn, vn, gn, bn, an], False, ctx, suffix=suffix,
                                out_heads=[None, None, None, None, (1, H, hp), (1, H, hp)])
        self.o_proj = Linear(H * dv, hidden_size, on, False, ctx, suffix=suffix)
        dev = ctx.device
        # taps as rows over all channels: a step's kernel reads a tap of neighbouring channels in one piece
        self.conv_w = torch.empty((self.taps, self.C), dtype=ctx.dtype, device=dev) if self.taps else None
        self.a_log, self.dt_bias = (torch.empty((H,), dtype=torch.float32, device=dev) for _ in range(2))
        self.norm_w = torch.empty((dv,), dtype=ctx.dtype, device=dev)

    def named_parameters(self) -> Dict[str, Param]:
        qn, kn, vn, gn, bn, an, on, ln, dn, nn, cn = self.names
        out = dict(self.proj.named_parameters())
        out.update(self.o_proj.named_parameters())
        if self.taps:
            c = 0
            for name, size in zip((qn, kn, vn), self.proj.out_sizes):
                out[f"{name}.{cn}"] = Param(self.conv_w[:, c:c + size].t())
                c += size
        out[ln], out[dn] = Param(self.a_log), Param(self.dt_bias)
        out[nn] = Param(self.norm_w, neutral=1.0)
        return out

    def cache_need(self):
        return (FixedState((max(self.taps - 1, 0), self.C), torch.float32), FixedState((self.H, self.dv, self.dk), torch.float32))

    def forward(self, x, batch, view):
        conv, state = view
        u = self.proj.forward(x)                                  # [T, q | k | v | g | b | a]
        R = state.state_in.numel()
        rows, gates = kernels.conv_delta_inputs(u, self.conv_w, conv.pool, conv.state_in, conv.state_out, batch.seg_of_token, batch.seg_offsets, R,
                                                self.H, self.G, self.dk, self.dv, self.b_off, self.a_off, self.a_log, self.dt_bias,
                                                float(self.dk) ** -0.5, self.unit_eps, max_len=batch.max_q_len)
        y = kernels.delta_rule(rows, gates, self.H, self.G, self.dk, self.dv, state.pool, state.state_in, state.state_out, batch.seg_offsets, R,
                               self.norm_w, u[:, self.C:self.C + self.H * self.dv], self.eps, self.dtype, max_len=batch.max_q_len)
        return self.o_proj.forward(y, allow_parts=True)
