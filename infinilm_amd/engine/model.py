"""The generic causal language model: embedding, layers run in the order the description gives,
final norm, output head at the wanted rows.  It is built from a `ModelSpec` alone; the embedding and
the head are parts chosen by kind like the layers' (`parts/ends.py`).

Reference for the flow: csrc/models/minicpm4/minicpm4_for_causal_lm.cpp:89-101 (model loop),
:123-127 (head); gathering the wanted rows before the head follows the generic template
csrc/layers/causal_lm_templates/text_causal_lm.hpp:59-75 rather than MiniCPM4's own class, which
computes logits at every position.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from ..cache.manager import Lent
from ..config.spec import ModelSpec, PartSpec
from ..parts import BuildContext, HyperStreams, Param, ResidualStream, build_block
from ..parts.base import join_name
from ..parts.linear import Linear
from ..parts.registry import build_embedding, build_head, build_norm


class CausalLM:
    def __init__(self, spec: ModelSpec, dtype: torch.dtype, device):
        spec.validate()
        self.spec = spec
        self.dtype = dtype
        self.device = torch.device(device)
        ctx = BuildContext(dtype=dtype, device=self.device)
        self.embedding = build_embedding(PartSpec(spec.embed_kind, dict(spec.embed_params, vocab_size=spec.vocab_size,
                                                                         hidden_size=spec.hidden_size, scale=spec.embed_scale)), ctx)
        self.blocks = [build_block(ls, ctx) for ls in spec.layers]
        self.final_norm = build_norm(spec.final_norm, ctx)
        self.output_head = build_head(PartSpec(spec.head.kind, dict(spec.head.params, vocab_size=spec.vocab_size,
                                                                    hidden_size=spec.hidden_size, scale=spec.head.scale)), ctx)
        if spec.head.always_tied:
            self.output_head.tie(self.embedding.table)
        self.run_vectors = None
        if spec.run_vectors is not None:
            self.run_vectors = torch.empty((int(spec.run_vectors[1]), spec.hidden_size), dtype=dtype, device=self.device)
        self.run_projection = None
        if spec.run_projection is not None:
            self.run_projection = Linear(2 * spec.hidden_size, spec.hidden_size, spec.run_projection, False, ctx, suffix="")
        # tensors of the model that several layers read (a table of which every layer takes its own columns): made here, loaded
        # under their own names, handed to every block that asks for them
        self.shared_tensors = {name: torch.empty(tuple(shape), dtype=dtype, device=self.device)
                               for name, shape in (spec.shared_tensors or {}).items()}
        for b in self.blocks:
            if hasattr(b, "bind_shared"):
                b.bind_shared(self.shared_tensors)
        self._keeps_embedding = any(r.start is not None and (r.start.embedding != 0.0 or r.start.project_embedding) for r in spec.order)
        # cache entry -> what its writer's mixer needs
        self.cache_needs: List = [None] * spec.num_cache_entries()
        for run in spec.order:
            if run.cache is not None and run.writes_cache:
                self.cache_needs[run.cache] = self.blocks[run.layer].cache_need()
        for run in spec.order:
            if run.cache is not None and not run.writes_cache:
                need = self.blocks[run.layer].cache_need()
                if need != self.cache_needs[run.cache]:
                    raise ValueError(f"layer {run.layer} reads cache entry {run.cache}, whose writer keeps "
                                     f"{self.cache_needs[run.cache]}, but needs {need}")
        for run in spec.order:
            if run.borrows is not None:
                want = getattr(self.blocks[run.layer].mixer, "borrowed_need", lambda: None)()
                held = self.cache_needs[run.borrows]
                if want is None or want not in (held if isinstance(held, (tuple, list)) else (held,)):
                    raise ValueError(f"layer {run.layer} borrows cache entry {run.borrows}, which keeps {held}, but reads {want}")

    # ---- tensors by checkpoint name ---------------------------------------------------------
    @property
    def embed(self) -> torch.Tensor:
        """The embedding's table."""
        return self.embedding.table

    @property
    def head(self) -> torch.Tensor:
        """The head's matrix (the embedding's table itself when the head is tied)."""
        return self.output_head.weight

    @property
    def head_is_tied(self) -> bool:
        return self.output_head.tied

    def named_parameters(self) -> Dict[str, Param]:
        out: Dict[str, Param] = {}
        for name, p in self.embedding.named_parameters().items():
            out[join_name(self.spec.embed_name, name)] = p
        for b in self.blocks:
            out.update(b.named_parameters())
        for name, p in self.final_norm.named_parameters().items():
            out[join_name(self.spec.final_norm_name, name)] = p
        if self.run_vectors is not None:
            out[self.spec.run_vectors[0]] = Param(self.run_vectors)
        if self.run_projection is not None:
            out.update(self.run_projection.named_parameters())
        for name, t in self.shared_tensors.items():
            out[name] = Param(t)
        if not self.spec.head.always_tied:
            for name, p in self.output_head.named_parameters().items():
                out[join_name(self.spec.head.name, name)] = p
        return out

    def tie_head_to_embedding(self) -> None:
        """The head reads the embedding table itself (one tensor, no copy); the embedding's scale
        is applied at lookup, so the table the head sees is the unscaled one
        (python/infinilm/modeling_utils.py:342-351)."""
        self.output_head.tie(self.embedding.table)

    def weight_bytes(self) -> int:
        seen = {}
        for p in self.named_parameters().values():
            t = p.tensor
            seen[t.untyped_storage().data_ptr() if t.device.type != "meta" else id(t)] = t.untyped_storage().nbytes()
        return sum(seen.values())

    # ---- forward ------------------------------------------------------------------------------
    def _embed(self, batch) -> torch.Tensor:
        if getattr(self.embedding, "takes_positions", False):
            return self.embedding.forward(batch.token_ids, batch.positions)
        return self.embedding.forward(batch.token_ids)

    def forward(self, batch, cache) -> torch.Tensor:
        """float32 logits [len(batch.want_rows), vocab] for the tokens of `batch`."""
        embedded = self._embed(batch)
        stream = HyperStreams(embedded, self.spec.streams) if self.spec.streams else ResidualStream(embedded)
        taps = batch.taps
        if taps is not None:
            taps["embed"] = embedded.clone()
        # the embedding's output once more for the runs that add it again (the stream itself is summed into in place)
        first = self._embed(batch) if self._keeps_embedding else None
        for i, run in enumerate(self.spec.order):
            if run.start is not None:
                if run.start.embedding != 0.0:
                    stream.push_more(first, run.start.embedding)
                if run.start.vector_row is not None:
                    stream.push_more(self.run_vectors[run.start.vector_row], 1.0)
                if run.start.project_embedding:
                    stream.project_beside(first, self.run_projection, self.dtype)
            view = cache.view(run.cache, batch, run.writes_cache) if run.cache is not None else None
            if run.borrows is not None:
                view = Lent(view, cache.view(run.borrows, batch, False))
            self.blocks[run.layer].forward(stream, batch, view)
            if taps is not None:
                taps[f"run{i}"] = stream.snapshot()
        if batch.num_wanted == 0:
            return torch.empty((0, self.spec.vocab_size), dtype=torch.float32, device=self.device)
        if not batch.wants_all_rows:
            stream = stream.gather(batch.want_rows)
        x = self.final_norm.forward(stream)
        return self.output_head.forward(x)
