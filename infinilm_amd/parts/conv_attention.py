"""Grouped-query attention with short convolutions, norms over whole rows and masks by chunks.

  projections without bias: heads query heads and kv_heads key heads of dim entries, kv_heads value heads of vdim entries
  a short causal convolution per channel of q, k and v right after the projection (`conv_taps` inputs, the last the token's
        own, zeros before a sequence's start; no bias; 0: none), whose last conv_taps - 1 inputs are state of the request
  q and k RMS-normed over all rows of all heads at once, with weights of that size (`row_norm`)
  the first `rotary_dim` entries of every q and k head turned in the pairs (2i, 2i + 1) by position x frequency_i
  softmax(scale q k^T) v over what the token sees: all keys up to its own, the last `window`, or (`chunk`) those of its own
        chunk of positions, chunks counted from the sequence's start; query head h reads key/value head h // (heads / kv_heads)
  W_o on the heads side by side.

Scores, softmax weights, norms and angles are float32 whatever the activations' dtype.  A layer with `own_kv` false has no key
and value tensors: its run borrows the cache entry another layer's run writes (`LayerRun.borrows`) and attends over it with
its own queries and its own mask.  `cache_window` / `cache_chunks`: what the cache keeps for all the layers that read an
entry (0 and (): every position)."""
from __future__ import annotations

from typing import Dict, Optional, Sequence, Tuple

import torch

from .. import kernels
from ..cache.manager import KVView, Lent
from ..cache.needs import FixedState, PagedKV
from .base import BuildContext, Mixer, Param
from .linear import FusedLinear, Linear
from .registry import register_mixer
from .rotary import pair_frequencies


@register_mixer("conv_attention")
class ConvAttention(Mixer):
    records_mixed_steps = True

    def __init__(self, hidden_size: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, eps: float, ctx: BuildContext,
                 window: int = 0, chunk: int = 0, cache_window: int = 0, cache_chunks: Tuple[int, ...] = (), conv_taps: int = 0,
                 rotary_dim: int = 0, theta: float = 1.0, own_kv: bool = True, row_norm: bool = True,
                 names: Sequence[str] = ("q", "k", "v", "o", "conv", "norm"), suffix: str = ""):
        self.H, self.G, self.dim, self.vdim = int(heads), int(kv_heads), int(dim), int(vdim)
        if self.G <= 0 or self.H % self.G:
            raise ValueError(f"{heads} query heads do not divide into {kv_heads} groups")
        self.scale, self.eps = float(scale), float(eps)
        self.window, self.chunk = int(window), int(chunk)
        self.cache_window, self.cache_chunks = int(cache_window), tuple(int(c) for c in cache_chunks)
        if self.window and self.chunk:
            raise ValueError("a mask by a window or by chunks, not both")
        if (self.cache_window and not 0 < self.window <= self.cache_window) or (self.cache_chunks and self.chunk not in self.cache_chunks):
            raise ValueError("the cache does not keep what this layer's mask shows it")
        self.taps = int(conv_taps)
        if not 0 <= self.taps <= kernels.CONV_MAX_TAPS:
            raise ValueError(f"{self.taps} taps: the convolution kernel takes up to {kernels.CONV_MAX_TAPS}")
        self.rd = int(rotary_dim)
        if self.rd % 2 or not 0 <= self.rd <= self.dim:
            raise ValueError(f"rotary_dim {rotary_dim} must be even and at most the head size {dim}")
        self.own_kv = bool(own_kv)
        self.d = -(-max(self.dim, self.vdim) // 16) * 16             # the cache's head size
        self.names = tuple(names)
        qn, kn, vn, on = self.names[:4]
        sizes, self.proj_names = [self.H * self.dim], [qn]
        if self.own_kv:
            sizes += [self.G * self.dim, self.G * self.vdim]
            self.proj_names += [kn, vn]
        self.C = sum(sizes)
        dev = ctx.device
        self.qkv = FusedLinear(hidden_size, sizes, self.proj_names, False, ctx, suffix=suffix)
        self.o_proj = Linear(self.H * self.d, hidden_size, on, False, ctx, suffix=suffix, in_heads=(self.H, self.vdim, self.d))
        # taps as rows over all channels (see GatedDeltaRule)
        self.conv_w = torch.empty((self.taps, self.C), dtype=ctx.dtype, device=dev) if self.taps else None
        self.q_norm = torch.empty((self.H * self.dim,), dtype=ctx.dtype, device=dev) if row_norm else None
        self.k_norm = torch.empty((self.G * self.dim,), dtype=ctx.dtype, device=dev) if row_norm and self.own_kv else None
        self.freq = pair_frequencies(self.rd, theta, dev)

    def named_parameters(self) -> Dict[str, Param]:
        qn, kn, vn, on, cn, nn = self.names
        out = dict(self.qkv.named_parameters())
        out.update(self.o_proj.named_parameters())
        if self.taps:
            c = 0
            for name, size in zip(self.proj_names, self.qkv.out_sizes):
                out[f"{name}.{cn}"] = Param(self.conv_w[:, c:c + size].t())
                c += size
        if self.q_norm is not None:
            out[f"{qn}.{nn}"] = Param(self.q_norm, neutral=1.0)
        if self.k_norm is not None:
            out[f"{kn}.{nn}"] = Param(self.k_norm, neutral=1.0)
        return out

    def _kv_need(self) -> PagedKV:
        return PagedKV(self.G, self.d, self.cache_window, chunks=self.cache_chunks)

    def borrowed_need(self) -> Optional[PagedKV]:
        """What a layer without keys and values of its own reads of the cache entry it borrows."""
        return None if self.own_kv else self._kv_need()

    def cache_need(self):
        state = FixedState((self.taps - 1, self.C), torch.float32) if self.taps > 1 else None
        if not self.own_kv:
            return state
        return self._kv_need() if state is None else (self._kv_need(), state)

    def forward(self, x, batch, view):
        lent = None
        if isinstance(view, Lent):
            view, lent = view.own, view.lent
        members = view if isinstance(view, tuple) else (view,)
        conv = next((m for m in members if m is not None and not isinstance(m, KVView)), None)
        holder = members if self.own_kv else (lent if isinstance(lent, tuple) else (lent,))
        kv = next((m for m in holder if isinstance(m, KVView)), None)
        if kv is None:
            raise RuntimeError("the attention got no keys and values to attend over")
        u = self.qkv.forward(x)                                   # [T, q | k | v]
        q = kernels.conv_norm_rope_kvwrite(u, self.conv_w, conv.pool if conv is not None else None, conv.state_in if conv is not None else None,
                                           conv.state_out if conv is not None else None, batch.seg_of_token, batch.seg_offsets,
                                           batch.state_in.numel(), batch.positions, self.freq, self.q_norm, self.k_norm, kv.k, kv.v,
                                           kv.slots if self.own_kv else None, self.H, self.G, self.dim, self.vdim, self.rd, self.eps,
                                           own_kv=self.own_kv, max_len=batch.max_q_len)
        o = kernels.paged_attention(q, kv.k, kv.v, kv.block_tables, batch.seg_of_token, batch.positions, self.H, self.G, self.d, self.scale,
                                    self.window, batch.max_total_len, batch.att_tiles, batch.att_single_rows, float_weights=True,
                                    chunk=self.chunk)
        return self.o_proj.forward(o, allow_parts=True)
