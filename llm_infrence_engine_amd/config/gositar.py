"""Typed configuration of the Gositar decoder and its translation into a ``ModelSpec``.

config.json: ``architecture`` "Gositar", ``vocab``, ``width``, ``streams``, ``norm.eps`` and ``layers`` (one entry per layer:
``type`` "latent_attention" or "latent_attention_2"; ``mixer``, its sizes and constants; ``mlp``: a feed-forward, or null for
a layer without one).

mixer: {"heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot": {"base", "dims", "scaling": {"factor", "original",
       "fast", "slow"} or absent}}
mlp:   {"kind": "dense", "ff"}, or {"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "top", "groups":
       {"count", "keep"} or absent}, "shared": {"ff", "limit"} or absent}

Fixed by the design and therefore constants here: the residual stream has ``streams`` copies that every sublayer reads and
writes through a link of its own (``l<i>.hc1.*``, ``l<i>.hc2.*``), with a layer norm (weight, no bias) before the sublayer; both
mixers are causal attention through a latent with queries straight from the input; "latent_attention" rotates neighbouring
entries and has one output gate per head, "latent_attention_2" rotates half-split pairs and has no gate; the dense
feed-forward is down(relu(up)^2); routed experts have softmax scores, a correction that steers the choice, weights normalised
over the chosen ones, the clamped gated form, and an ungated shared expert; the head is a matrix of its own; tensors are named
``embed``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

import copy
import json
from dataclasses import dataclass
from typing import Tuple

from .gidurax import _need
from .registry import ConfigError, register_architecture
from .spec import ModelSpec, PartSpec, Run, layer

# type -> (how rotated entries are paired, the output gate)
MIXERS = {"latent_attention": ("neighbours", "head"), "latent_attention_2": ("half", False)}
GLU_ALPHA = 1.702      # the experts' g * sigmoid(alpha g)


@dataclass(frozen=True)
class GositarConfig:
    vocab: int
    width: int
    streams: int
    norm_eps: float
    layers: Tuple[dict, ...]          # as config.json gives them (checked in __post_init__, never changed afterwards)

    architecture = "Gositar"

    def __hash__(self):
        return hash(json.dumps(self.to_dict(), sort_keys=True))

    def __post_init__(self):
        if self.vocab <= 0 or self.width <= 0 or self.streams <= 0:
            raise ConfigError("vocab, width and streams must be positive")
        if not self.norm_eps >= 0:
            raise ConfigError(f"norm.eps must be >= 0, got {self.norm_eps}")
        if not self.layers:
            raise ConfigError("config.json: 'layers' is empty")
        for i, entry in enumerate(self.layers):
            where = f"layers[{i}]"
            kind = entry.get("type") if isinstance(entry, dict) else None
            if kind not in MIXERS:
                raise ConfigError(f"config.json: {where}.type is {kind!r}; this design has {', '.join(MIXERS)}")
            m = entry.get("mixer")
            for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"):
                _need(m, k, where + ".mixer")
            _need(m, "scale", where + ".mixer", float)
            rot = m.get("rot")
            _need(rot, "base", where + ".mixer.rot", float)
            dims = _need(rot, "dims", where + ".mixer.rot")
            if dims % 2 or dims > m["rot_dim"]:
                raise ConfigError(f"config.json: {where}.mixer.rot.dims = {dims} must be even and at most rot_dim")
            if rot.get("scaling") is not None:
                for k in ("factor", "original", "fast", "slow"):
                    if not _need(rot["scaling"], k, where + ".mixer.rot.scaling", float) > 0:
                        raise ConfigError(f"config.json: {where}.mixer.rot.scaling.{k} must be positive")
            if entry.get("mlp") is not None:
                self._check_mlp(entry["mlp"], where + ".mlp")

    @staticmethod
    def _check_mlp(mlp: dict, where: str) -> None:
        if mlp.get("kind") == "dense":
            _need(mlp, "ff", where)
        elif mlp.get("kind") == "moe":
            for name in ("expert", "shared"):
                if name == "expert" or mlp.get("shared") is not None:
                    _need(mlp.get(name), "ff", f"{where}.{name}")
                    _need(mlp.get(name), "limit", f"{where}.{name}", float)
            r = mlp.get("router")
            experts, top = _need(r, "experts", where + ".router"), _need(r, "top", where + ".router")
            if top > experts:
                raise ConfigError(f"config.json: {where}.router: top {top} exceeds the experts there are")
            if r.get("groups") is not None:
                count = _need(r["groups"], "count", where + ".router.groups")
                keep = _need(r["groups"], "keep", where + ".router.groups")
                if experts % count or keep > count or top > keep * (experts // count):
                    raise ConfigError(f"config.json: {where}.router: {top} of {experts} experts within {keep} of {count} "
                                      f"equal groups cannot be chosen")
        else:
            raise ConfigError(f"config.json: {where}.kind is {mlp.get('kind')!r}; this design has 'dense' and 'moe'")

    # ------------------------------------------------------------------ config.json
    @classmethod
    def from_dict(cls, d: dict) -> "GositarConfig":
        layers = d.get("layers")
        if not isinstance(layers, list):
            raise ConfigError("config.json lacks the list 'layers'")
        return cls(vocab=_need(d, "vocab", "config"), width=_need(d, "width", "config"), streams=_need(d, "streams", "config"),
                   norm_eps=_need(d.get("norm"), "eps", "norm", float), layers=tuple(copy.deepcopy(e) for e in layers))

    def to_dict(self) -> dict:
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "streams": self.streams,
                "norm": {"eps": self.norm_eps}, "layers": [copy.deepcopy(e) for e in self.layers]}

    # ------------------------------------------------------------------ derived sizes
    @property
    def num_params(self) -> int:
        from ..parts.model import Model

        total = 0
        for s in Model(self.to_spec()).tensor_specs():
            n = 1
            for d in s.shape:
                n *= d
            total += n
        return total

    # ------------------------------------------------------------------ the model as data
    def _norm(self, prefix: str, name: str) -> PartSpec:
        return PartSpec("layer_norm", prefix, {"size": self.width, "eps": self.norm_eps, "name": name})

    def _link(self, prefix: str) -> PartSpec:
        return PartSpec("stream_link", prefix, {"streams": self.streams})

    def _mixer(self, i: int, entry: dict) -> Tuple[PartSpec, PartSpec]:
        """(mixer PartSpec, position PartSpec) of layer i."""
        m, rot = entry["mixer"], entry["mixer"]["rot"]
        pairing, gate = MIXERS[entry["type"]]
        mixer = PartSpec("latent_attention", f"l{i}.mix.", {
            "hidden_size": self.width, "heads": m["heads"], "dim": m["dim"], "rot_dim": m["rot_dim"], "vdim": m["vdim"],
            "q_rank": None, "kv_rank": m["kv_rank"], "scale": float(m["scale"]), "eps": self.norm_eps, "window": None,
            "sink": False, "output_gate": gate})
        scaling = tuple(sorted(rot["scaling"].items())) if rot.get("scaling") is not None else None
        position = PartSpec("rotary_pairs", "", {"width": m["rot_dim"], "dims": rot["dims"], "theta": float(rot["base"]),
                                                 "pairing": pairing, "scaling": scaling})
        return mixer, position

    def _feed_forward(self, i: int, mlp: dict) -> PartSpec:
        p, W = f"l{i}.mlp.", self.width
        if mlp["kind"] == "dense":
            return PartSpec("dense_act", p, {"hidden_size": W, "intermediate_size": mlp["ff"], "activation": "relu2"})
        r, shared = mlp["router"], mlp.get("shared")
        groups = (r["groups"]["count"], r["groups"]["keep"]) if r.get("groups") is not None else None
        return PartSpec("routed_experts", p, {
            "hidden_size": W, "expert_ff": mlp["expert"]["ff"], "experts": r["experts"], "top": r["top"], "groups": groups,
            "normalise": True, "activation": "clamped_glu", "limit": float(mlp["expert"]["limit"]), "alpha": GLU_ALPHA,
            "shared_ff": shared["ff"] if shared is not None else 0,
            "shared_limit": float(shared["limit"]) if shared is not None else None, "shared_gate": False})

    def to_spec(self) -> ModelSpec:
        W = self.width
        layers, ignorable = [], []
        for i, entry in enumerate(self.layers):
            p, mlp = f"l{i}.", entry.get("mlp")
            mixer, position = self._mixer(i, entry)
            second = mlp is not None
            layers.append(layer(
                "hyper_connected_pre_norm", position=position, mixer_norm=self._norm(p, "norm1"), mixer=mixer,
                mixer_link=self._link(p + "hc1."),
                feed_forward_norm=self._norm(p, "norm2") if second else None,
                feed_forward=self._feed_forward(i, mlp) if second else None,
                feed_forward_link=self._link(p + "hc2.") if second else None))
            if not second:     # a layer with one sublayer has no use for the second's norm and link, if a checkpoint has them
                ignorable += [p + "norm2"] + [p + "hc2." + n for n in ("in", "out", "mix")]
        return ModelSpec(
            architecture=self.architecture, hidden_size=W, vocab_size=self.vocab,
            embedding=PartSpec("token_embedding", "", {"vocab_size": self.vocab, "hidden_size": W, "name": "embed",
                                                       "streams": self.streams}),
            layers=tuple(layers), order=tuple(Run(i) for i in range(len(layers))),
            final_norm=PartSpec("summed_streams", "", {"streams": self.streams, "norm": self._norm("final.", "norm")}),
            head=PartSpec("lm_head", "", {"hidden_size": W, "vocab_size": self.vocab, "tied_to": None, "name": "head"}),
            ignorable=tuple(ignorable),
        )


register_architecture(GositarConfig.architecture, GositarConfig, model_type="gositar")
