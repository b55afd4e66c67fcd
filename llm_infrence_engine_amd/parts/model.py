"""A model assembled from a ``ModelSpec``: embedding, layers in the order the spec gives, final norm, head.

The same layer may run more than once and a run may read an earlier run's cache; each run that keeps a
cache of its own is one entry of the cache manager's groups.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch

from ..config.spec import ModelSpec
from ..weights.reader import CheckpointReader, place
from ..weights.spec import TensorSpec
from . import (attention, blocks, delta, ends, experts, feed_forward, filters, latent, linear_attention, mingru,  # noqa: F401
               norms, pooled_attention, positions, scan, side, side_by_side, streams)      # (register the built-in parts)
from .base import KVView, Runtime, StateView, StepContext, build_part, part_class, weakest


@dataclass
class RunCache:
    """What one run of a layer was given by the cache manager for this step."""

    kv: Optional[KVView] = None
    state: Optional[StateView] = None


class Model:
    def __init__(self, spec: ModelSpec):
        self.spec = spec
        self.embedding = build_part("embedding", spec.embedding)
        self.layers = []
        for ls in spec.layers:
            self.layers.append(part_class("block", ls.block).build(ls.parts))
        self.final_norm = build_part("norm", spec.final_norm)
        self.head = build_part("head", spec.head)
        self.pass_entry = build_part("pass_entry", spec.pass_entry) if spec.pass_entry is not None else None
        self.rt: Optional[Runtime] = None

    # ------------------------------------------------------------------ weights
    def _parts(self):
        return [self.embedding, *([self.pass_entry] if self.pass_entry is not None else []), *self.layers, self.final_norm,
                self.head]

    def tensor_specs(self) -> List[TensorSpec]:
        """Every tensor the model wants, each name once (a tied head names the embedding's)."""
        seen, out = set(), []
        for p in self._parts():
            for s in p.tensor_specs():
                if s.name not in seen:
                    seen.add(s.name)
                    out.append(s)
        return out

    def ignorable_tensors(self) -> List[str]:
        return list(getattr(self.head, "ignorable", lambda: [])()) + list(self.spec.ignorable)

    def load(self, reader: CheckpointReader, rt: Runtime) -> "Model":
        reader.check(self.tensor_specs(), self.ignorable_tensors())
        placed: Dict[str, torch.Tensor] = {}

        def get(spec: TensorSpec) -> torch.Tensor:
            if spec.name not in placed:
                placed[spec.name] = place(reader.get(spec.name), spec, rt.dtype, rt.device)
            return placed[spec.name]

        for p in self._parts():
            p.load(get, rt)
        self.rt = rt
        reader.close()
        return self

    # ------------------------------------------------------------------ cache needs, run by run
    def run_needs(self):
        """For every entry of the order: (CacheNeed or None, StateNeed(s) or None, cache_of)."""
        return [(self.layers[run.layer].cache_need(), self.layers[run.layer].state_need(), run.cache_of)
                for run in self.spec.order]

    def graph_safe(self):
        """Which steps of this model may be captured into graphs: True (all), "decode" (steps of single tokens)
        or False (none); the weakest answer of its parts (see ``Part.graph_safe``)."""
        return weakest([b.graph_safe() for b in self.layers] +
                       [p.graph_safe for p in (self.embedding, self.final_norm, self.head)] +
                       ([self.pass_entry.graph_safe] if self.pass_entry is not None else []))

    # ------------------------------------------------------------------ one step
    def forward(self, ctx: StepContext, caches: List[RunCache]) -> torch.Tensor:
        """Float logits [M, V] at ``ctx.logit_rows``.  Runs only the step's tokens, from the cache."""
        x, pending = self.forward_hidden(ctx, caches)
        return self.head_logits(x, pending, ctx.logit_rows)

    def forward_hidden(self, ctx: StepContext, caches: List[RunCache]):
        """Embedding and all runs of the order: the float residual stream ([N, H], or [N, S, H] where the model has S
        copies of it) and what the last run has still to write into it (an addend, a write that the final norm carries out
        itself, or None)."""
        x = self.embedding.forward(ctx)
        kept = x.clone() if self.pass_entry is not None and self.pass_entry.keeps_embedding else None
        pending = None
        for i, run in enumerate(self.spec.order):
            if run.opens_pass is not None:
                if pending is not None:      # the pass's addends go into the sum itself
                    from ..kernels import ops

                    pending.add_into(x) if hasattr(pending, "add_into") else ops.residual_add(x, pending)
                    pending = None
                new = self.pass_entry.forward(x, kept, run.opens_pass)
                x = x if new is None else new
            c = caches[i]
            pending = self._settled(x, pending, self.layers[run.layer])
            pending = self.layers[run.layer].forward(x, pending, ctx, c.kv, c.state)
        return x, self._settled(x, pending, self.final_norm)

    @staticmethod
    def _settled(x, pending, reader):
        """``pending`` as ``reader`` (a block or the final norm) takes it: a write that is more than an addend is carried out
        now if the reader does not do that itself."""
        if hasattr(pending, "add_into") and not reader.settles_writes:
            pending.add_into(x)
            return None
        return pending

    def head_logits(self, x: torch.Tensor, pending: Optional[torch.Tensor], rows: torch.Tensor) -> torch.Tensor:
        """Final norm and head on the rows ``rows`` (int32) of what ``forward_hidden`` returned; x is left as it is."""
        if rows.numel() == 0:
            return torch.empty(0, self.spec.vocab_size, dtype=torch.float32, device=x.device)
        norm = self.final_norm.lazy if self.head.accepts_lazy_norm else self.final_norm.forward
        return self.head.forward(norm(x, delta=pending, rows=rows, write_back=False))
