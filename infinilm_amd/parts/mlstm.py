"""The matrix memory of an mLSTM (xLSTM): a linear attention whose state is written and forgotten through exponential gates.

  projections without bias: query and key heads of dim entries, value heads of vdim entries; queries by 1 / sqrt(dim)
  two numbers a head and token, each squeezed to within +-cap by z -> cap tanh(z / cap) after its bias: i (the logarithm of how
        strongly the token is written) and, through log sigmoid, f (the logarithm of what stays of the past)
  a matrix S [dim, vdim], a vector n [dim] and a number m, all zero before a sequence's start; with vectors as rows
        m' = max(f + m, i),   keep = e^(f + m - m'),   put = e^(i - m')
        S' = keep S + put outer(k, v),   n' = keep n + put k,   y = q S' / (max(|q . n'|, e^-m') + 1e-6)
  y of every head by its root mean square, times norm [heads vdim] and the sigmoid of a gate's projection; then the output product.

Two states a request, float32 rows of the cache manager's pools: S with n as one row more, [heads, vdim + 1, dim], and m [heads].
Everything between the projections is float32 whatever the activations' dtype.
"""
from __future__ import annotations

from typing import Dict, Sequence

import torch

from .. import kernels
from ..cache.needs import FixedState
from .base import BuildContext, Mixer, Param, join_name
from .linear import FusedLinear, Linear
from .registry import register_mixer


@register_mixer("mlstm")
class MLSTM(Mixer):
    records_mixed_steps = True   # every index comes from the batch's device tensors

    def __init__(self, hidden_size: int, heads: int, dim: int, vdim: int, gate_cap: float, eps: float, ctx: BuildContext,
                 names: Sequence[str] = ("q", "k", "v", "g", "i", "f", "o", "norm"), suffix: str = "", bias_suffix: str = "bias"):
        self.H, self.dk, self.dv = int(heads), int(dim), int(vdim)
        if self.dk > kernels.MLSTM_MAX_KEY_DIM:
            raise ValueError(f"key size {self.dk} is above the recurrence kernel's {kernels.MLSTM_MAX_KEY_DIM}")
        self.cap, self.eps, self.dtype = float(gate_cap), float(eps), ctx.dtype
        if self.cap <= 0:
            raise ValueError(f"the gates' cap {gate_cap} must be positive")
        self.names, self.bias_suffix = tuple(names), bias_suffix
        qn, kn, vn, gn, i_n, fn, on, _ = self.names
        H, dk, dv = self.H, self.dk, self.dv
        # (q, k, v, g rows and the per-head rows filled up, so that rows stay 16-byte aligned)
        used = H * (2 * dk + 2 * dv)
        hp = -(-(used + H) // 8) * 8 - used
        self.g_off, self.i_off, self.f_off = H * (2 * dk + dv), used, used + hp
        fp = -(-H // 8) * 8
        self.proj = FusedLinear(hidden_size, [H * dk, H * dk, H * dv, H * dv, hp, fp], [qn, kn, vn, gn, i_n, fn], False, ctx, suffix=suffix,
                                out_heads=[None, None, None, None, (1, H, hp), (1, H, fp)])
        self.o_proj = Linear(H * dv, hidden_size, on, False, ctx, suffix=suffix)
        self.bias_i, self.bias_f = (torch.empty((H,), dtype=torch.float32, device=ctx.device) for _ in range(2))
        self.norm_w = torch.empty((H * dv,), dtype=ctx.dtype, device=ctx.device)

    def named_parameters(self) -> Dict[str, Param]:
        i_n, fn, nn = self.names[4], self.names[5], self.names[7]
        out = dict(self.proj.named_parameters())
        out.update(self.o_proj.named_parameters())
        out[join_name(i_n, self.bias_suffix)] = Param(self.bias_i)
        out[join_name(fn, self.bias_suffix)] = Param(self.bias_f)
        out[nn] = Param(self.norm_w, neutral=1.0)
        return out

    def cache_need(self):
        return (FixedState((self.H, self.dv + 1, self.dk), torch.float32), FixedState((self.H,), torch.float32))

    def forward(self, x, batch, view):
        state, top = view
        u = self.proj.forward(x)                                  # [T, q | k | v | g | i | f]
        y = kernels.mlstm(u, self.bias_i, self.bias_f, self.i_off, self.f_off, self.g_off, self.H, self.dk, self.dv, self.cap, state.pool, top.pool,
                          state.state_in, state.state_out, batch.seg_offsets, state.state_in.numel(), self.norm_w, self.eps, self.dtype,
                          max_len=batch.max_q_len)
        return self.o_proj.forward(y, allow_parts=True)
