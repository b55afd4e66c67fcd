"""A feed-forward made of routed experts.

Router logits z = W_router h in float; scores s = softmax(z) over all the router's outputs; the ``top`` outputs with the
largest s + correction are chosen (``correction``: a stored vector that steers the choice and nothing else; False: there is
none) and weigh in with their s as it is.  ``scores`` "sigmoid": s is every logit's own sigmoid.  ``activation`` "swiglu":
an expert is down(silu(gate(h)) * up(h)) with a third matrix ``gate``.  ``weight_on`` "input": the weight multiplies what
the expert reads instead of what it returns, out = sum expert(s h) (both first products are linear, so the kernel applies
s to their results, in float, before the activation).  The first ``experts`` outputs are small feed-forwards down(act(up(h))) without biases; the last
``identity`` outputs are experts without tensors whose output is h itself.  ``shared_ff``: one more expert of that size
that every token runs, weighted by sigmoid(W_sg h), one number per token, or (``shared_gate`` False) as it is.
``activation`` "clamped_glu" with ``limit`` and ``alpha``: g = min(gate(h), limit), u = clamp(up(h), -limit, limit), an expert
is down(g sigmoid(alpha g) (u + 1)); the shared expert is of the same form with ``shared_limit``.  ``groups`` (count, keep):
the outputs form ``count`` equal groups of neighbours, a group counts as its largest s + correction (``group_top`` 2: as the sum
of its two largest), and only outputs of the ``keep`` best groups can be chosen.  ``normalise``: the chosen weights are divided by
their sum (+ 1e-20); ``weight_scale`` multiplies them.

Nothing here waits for the device: the tokens' choices are grouped by expert into tiles on the device, and the experts'
products run tile by tile over a launch whose size depends on the sizes alone, so a step can be captured."""
from __future__ import annotations

from typing import Optional

import torch

from ..kernels import linear, ops
from ..weights.spec import TensorSpec
from .base import FeedForward, register_part
from .feed_forward import ClampedGLU


class RoutedExperts(FeedForward):
    def __init__(self, prefix: str, hidden_size: int, expert_ff: int, experts: int, top: int, identity: int = 0,
                 shared_ff: int = 0, activation: str = "gelu", scores: str = "softmax", correction: bool = True,
                 weight_on: str = "output", groups=None, normalise: bool = False, limit: Optional[float] = None,
                 alpha: float = 1.702, shared_limit: Optional[float] = None, shared_gate: bool = True, group_top: int = 1,
                 weight_scale: float = 1.0):
        if activation not in ("gelu", "swiglu", "clamped_glu"):
            raise ValueError(f"no activation {activation!r} for routed experts; there are 'gelu', 'swiglu' and 'clamped_glu'")
        if activation == "clamped_glu" and (limit is None or (shared_ff and shared_limit is None)):
            raise ValueError("clamped experts need a limit (a shared one its own)")
        if activation == "swiglu" and shared_ff:
            raise ValueError("there is no shared expert of the 'swiglu' form")
        if scores not in ("softmax", "sigmoid") or weight_on not in ("output", "input"):
            raise ValueError("scores are 'softmax' or 'sigmoid'; the weight lies on the expert's 'output' or 'input'")
        if weight_on == "input" and (activation != "swiglu" or identity or shared_ff):
            raise ValueError("a weight on the expert's input comes with 'swiglu' experts alone")
        if experts <= 0 or identity < 0 or not 0 < top <= experts + identity:
            raise ValueError(f"{top} of {experts} + {identity} experts cannot be chosen")
        if experts + identity > ops.ROUTE_MAX_OUTPUTS or top > ops.ROUTE_MAX_TOP:
            raise ValueError(f"the router kernel takes up to {ops.ROUTE_MAX_OUTPUTS} outputs and a top of {ops.ROUTE_MAX_TOP}")
        self.prefix, self.hidden_size, self.expert_ff = prefix, hidden_size, expert_ff
        self.experts, self.identity, self.top, self.shared_ff = experts, identity, top, shared_ff
        self.activation, self.scores, self.has_correction, self.weight_on = activation, scores, bool(correction), weight_on
        self.groups, self.normalise = (tuple(groups) if groups is not None else None), bool(normalise)
        self.group_top, self.weight_scale = int(group_top), float(weight_scale)
        if self.group_top not in (1, 2):
            raise ValueError(f"a group counts as its best output or as its two best ones' sum, not as its {group_top} best")
        if self.groups is not None:
            count, keep = self.groups
            n_out = experts + identity
            if count <= 0 or n_out % count or not 0 < keep <= count or top > keep * (n_out // count):
                raise ValueError(f"{top} of {n_out} outputs cannot be chosen within {keep} of {count} equal groups")
        self.limit, self.alpha, self.shared_gate = limit, float(alpha), bool(shared_gate) and bool(shared_ff)
        self.gated = activation in ("swiglu", "clamped_glu")
        # the shared expert: a feed-forward of its own, under this one's tensor names
        self.shared = ClampedGLU(prefix + "shared.", hidden_size, shared_ff, shared_limit, alpha) \
            if shared_ff and activation == "clamped_glu" else None

    def tensor_specs(self):
        p, W, F = self.prefix, self.hidden_size, self.expert_ff
        specs = []
        for e in range(self.experts):
            if self.gated:
                specs.append(TensorSpec(f"{p}e{e}.gate", (F, W)))
            specs += [TensorSpec(f"{p}e{e}.up", (F, W)), TensorSpec(f"{p}e{e}.down", (W, F))]
        n_out = self.experts + self.identity
        specs.append(TensorSpec(p + "router", (n_out, W)))
        if self.has_correction:
            specs.append(TensorSpec(p + "correction", (n_out,), "bias"))
        if self.shared is not None:
            specs += self.shared.tensor_specs()
        elif self.shared_ff:
            specs += [TensorSpec(p + "shared.up", (self.shared_ff, W)), TensorSpec(p + "shared.down", (W, self.shared_ff))]
        if self.shared_gate:
            specs.append(TensorSpec(p + "shared.sg", (1, W)))
        return specs

    def load(self, get, rt):
        self.rt = rt
        t = {s.name[len(self.prefix):]: get(s) for s in self.tensor_specs()}
        if self.gated:      # gate and up rows interleaved, expert by expert: [E, 2F, W]
            self.w_up = torch.stack([linear.interleave_rows(t[f"e{e}.gate"], t[f"e{e}.up"]) for e in range(self.experts)]).contiguous()
        else:
            self.w_up = torch.stack([t[f"e{e}.up"] for e in range(self.experts)]).contiguous()       # [E, F, W]
        self.w_down = torch.stack([t[f"e{e}.down"] for e in range(self.experts)]).contiguous()   # [E, W, F]
        # the router and the shared expert's gate read the same h: one product, float out
        self.w_router = linear.prepare_weight(torch.cat([t["router"]] + ([t["shared.sg"]] if self.shared_gate else []), dim=0))
        self.correction = t["correction"] if self.has_correction else None
        if self.shared is not None:
            self.shared.load(get, rt)
        elif self.shared_ff:
            self.w_shared_up, self.w_shared_down = linear.prepare_weight(t["shared.up"]), linear.prepare_weight(t["shared.down"])

    def _chosen(self, h):
        """(ids [N, top], weights float [N, top] or None, the chosen experts' rows float [N * top, W], router's logits)."""
        N, W, E = h.shape[0], self.hidden_size, self.experts
        logits = linear.linear(h, self.w_router, out_dtype=torch.float32)
        ids, weights = ops.moe_route(logits, self.correction, self.top, E + self.identity, self.scores, self.groups, self.normalise,
                                     self.group_top, self.weight_scale)
        rows, tile_expert = ops.moe_align(ids, E, ops.moe_tile_choice(ids.numel(), E, (W, self.expert_ff), h.dtype))
        mid = None
        if self.activation == "clamped_glu" and h.dtype == torch.bfloat16 and W % 32 == 0:
            try:            # on the matrix cores the gate is the product's epilogue
                mid = ops.grouped_gemm(h, self.w_up, rows, tile_expert, self.rt.empty(rows.numel(), self.expert_ff),
                                       gather_div=self.top, act="clamped_glu", limit=self.limit, alpha=self.alpha)
            except ops.UnsupportedShape:
                mid = None
        if mid is not None:
            pass
        elif self.gated:
            gu = ops.grouped_gemm(h, self.w_up, rows, tile_expert, self.rt.empty(rows.numel(), 2 * self.expert_ff),
                                  gather_div=self.top)
            mid = self.rt.empty(rows.numel(), self.expert_ff)
            on_input = self.weight_on == "input"
            if self.activation == "clamped_glu":
                ops.clamped_glu(gu, mid, self.limit, self.alpha, rows)
            else:
                ops.scaled_swiglu(gu, mid, weights.view(-1) if on_input else None, rows)
            if on_input:
                weights = None
        else:
            mid = ops.grouped_gemm(h, self.w_up, rows, tile_expert, self.rt.empty(rows.numel(), self.expert_ff),
                                   gather_div=self.top, act=self.activation)
        part = ops.grouped_gemm(mid, self.w_down, rows, tile_expert,
                                torch.empty((N * self.top, W), dtype=torch.float32, device=h.device), scatter=True)
        return ids, weights, part, logits

    def _shared(self, h, ctx):
        if self.shared is not None:
            return self.shared.forward(h, ctx)
        u = linear.linear(h, self.w_shared_up)
        return linear.linear(ops.gelu(u, torch.empty_like(u)), self.w_shared_down)

    def forward(self, h, ctx):
        ids, weights, part, logits = self._chosen(h)
        shared = self._shared(h, ctx) if self.shared_ff else None
        gate = logits[:, self.experts + self.identity] if self.shared_gate else None
        out = torch.empty((h.shape[0], self.hidden_size), dtype=torch.float32, device=h.device)
        return ops.moe_combine(part, ids, weights, h, self.experts, out, shared, gate)

    def forward_deferred(self, h, ctx):
        """The weighted sum over the chosen experts' rows, and the shared expert's addition, left to the caller's kernel."""
        if self.identity or self.shared_gate or self.weight_on == "input":
            return self.forward(h, ctx)
        _, weights, part, _ = self._chosen(h)
        return (self._shared(h, ctx) if self.shared_ff else None), part, weights


register_part("feed_forward", "routed_experts", RoutedExperts)
