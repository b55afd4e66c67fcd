"""A residual stream made of several copies, and the arrangement of layers that read and write it.

The stream is X [tokens, S, width] (float), every copy equal to the embedding's output at the start.  A sublayer has a
*link* to the streams, three small stored tensors: a [S] (``in``), b [S] (``out``) and M [S, S] (``mix``, indexed [from, to]),
and with them

    u = sum_s a[s] X[s];   y = sublayer(norm(u));   X[t] <- sum_s M[s, t] X[s] + b[t] y   (all t from the old X)

in place of a residual sum.  The last line of a sublayer and the first of the next one are one pass over X
(``ops.streams_step``): a layer hands its last write on as ``pending``, the next reader carries it out.  A model ends with
``summed_streams``, the norm of the plain sum of the streams."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Optional

import torch

from ..kernels import ops
from ..weights.spec import TensorSpec
from .base import Block, Norm, Part, build_part, register_part


@dataclass
class StreamsWrite:
    """A write into the streams that is still to be carried out: ``y`` a sublayer's output (as ``ops.streams_step`` takes
    it), ``link`` the sublayer's own."""

    y: Any
    link: "StreamLink"

    def args(self):
        return self.y, self.link.mix, self.link.b

    def add_into(self, x: torch.Tensor) -> None:
        ops.streams_step(x, write=self.args())


class StreamLink(Part):
    """``streams`` numbers a and b and a square matrix M of one sublayer (tensors ``in``, ``out``, ``mix``), kept in float."""

    def __init__(self, prefix: str, streams: int, names=("in", "out", "mix")):
        if not 0 < streams <= ops.STREAMS_MAX:
            raise ValueError(f"{streams} streams: there are 1 to {ops.STREAMS_MAX}")
        self.prefix, self.streams, self.names = prefix, streams, tuple(names)

    def tensor_specs(self):
        a, b, m = (self.prefix + n for n in self.names)
        S = self.streams
        return [TensorSpec(a, (S,), "norm"), TensorSpec(b, (S,), "norm"), TensorSpec(m, (S, S), "mixing")]

    def load(self, get, rt):
        self.rt = rt
        self.a, self.b, self.mix = (get(s) for s in self.tensor_specs())

    def read(self, x: torch.Tensor, norm: Norm, pending: Optional[StreamsWrite]) -> torch.Tensor:
        """norm(u) of the streams after the pending write, which is kept in x: one pass."""
        out = self.rt.empty(x.shape[0], x.shape[2])
        return ops.streams_step(x, write=pending.args() if pending is not None else None,
                                read=(self.a, norm.statistic, norm.weight, norm.bias, norm.eps, out))


class HyperConnectedPreNorm(Block):
    """The usual two sublayers, mixer and feed-forward with a norm before each, on several streams: every sublayer reads its
    input from the streams and writes its result to them through a link of its own.  Without a feed-forward the layer has one
    sublayer."""

    takes = {"position": "position", "mixer_norm": "norm", "mixer": "mixer", "mixer_link": "stream_link",
             "feed_forward_norm": "norm", "feed_forward": "feed_forward", "feed_forward_link": "stream_link"}
    optional = ("position", "feed_forward_norm", "feed_forward", "feed_forward_link")
    settles_writes = True

    def __init__(self, **built):
        super().__init__(**built)
        for name in ("mixer_norm", "feed_forward_norm"):
            norm = self.built[name]
            if norm is not None and getattr(norm, "statistic", None) is None:
                raise ValueError(f"{name}: {type(norm).__name__} cannot be taken of a sum of streams on the way (no statistic)")
        if self.feed_forward is not None and (self.feed_forward_norm is None or self.feed_forward_link is None):
            raise ValueError("a feed-forward on streams comes with a norm and a link")

    def forward(self, x, pending, ctx, kv, state):
        h = self.mixer_link.read(x, self.mixer_norm, pending)
        pending = StreamsWrite(self.mixer.forward(h, ctx, kv, state), self.mixer_link)
        if self.feed_forward is None:
            return pending
        h = self.feed_forward_link.read(x, self.feed_forward_norm, pending)
        return StreamsWrite(self.feed_forward.forward_deferred(h, ctx), self.feed_forward_link)


class SummedStreams(Norm):
    """A norm (``norm``: its ``PartSpec``, or a built one's) of the sum of the streams, for a model's end."""

    settles_writes = True

    def __init__(self, prefix: str, streams: int, norm):
        self.streams = streams
        self.norm = build_part("norm", norm)
        if getattr(self.norm, "statistic", None) is None:
            raise ValueError(f"the norm {norm.kind!r} cannot be taken of a sum of streams on the way (no statistic)")

    def tensor_specs(self):
        return self.norm.tensor_specs()

    def load(self, get, rt):
        self.rt = rt
        self.norm.load(get, rt)
        self.ones = torch.ones(self.streams, dtype=torch.float32, device=rt.device)

    def forward(self, x, delta=None, rows=None, write_back=True):
        n = x.shape[0] if rows is None else rows.numel()
        m = self.norm
        return ops.streams_step(x, write=delta.args() if delta is not None else None,
                                read=(self.ones, m.statistic, m.weight, m.bias, m.eps, self.rt.empty(n, x.shape[2])),
                                rows=rows, write_back=write_back)


register_part("stream_link", "stream_link", StreamLink)
register_part("block", "hyper_connected_pre_norm", HyperConnectedPreNorm)
register_part("norm", "summed_streams", SummedStreams)
