"""Typed configuration of the Kisusun decoder and its translation into a ``ModelSpec``.

config.json: ``architecture`` "Kisusun", ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_scale`` and ``layers``
(one entry per layer: ``type`` "attention"; ``mixer``, its sizes and constants; ``mlp``: a feed-forward, or null for a layer
without one).

mixer: {"heads", "kv_heads", "dim", "vdim", "scale", "softcap" or absent, "rot": {"base", "dims", "scaling": {"factor"} or
       absent} or absent, "mask": {"size"} or absent (all keys), "v_mix": true, false or absent}
mlp:   {"kind": "dense", "ff"}, or {"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "top", "scale", "groups":
       {"count", "keep"} or absent}, "shared": {"ff", "limit"} or absent}

Fixed by the design and therefore constants here: sublayers read the residual stream as it is, and their results pass an RMS
norm on the way into it; queries and keys are RMS-normalised over the whole projection, before the rotation of half-split pairs
with frequencies divided by one factor; a one is added to the softmax's denominator; every entry of the concatenated heads is
gated by a sigmoid of its own; layers with ``v_mix`` blend their values with the first such layer's; the dense feed-forward is
gated with silu; experts are of the clamped gated form, scored by sigmoids, chosen inside the best groups (a group counts as
the sum of its two best), weighted by score times ``router.scale``, beside an ungated shared expert; the head is the embedding
table; tensors are named ``embed``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``.
"""
from __future__ import annotations

import copy
import json
from dataclasses import dataclass
from typing import Optional, Tuple

from .gidurax import _need
from .registry import ConfigError, register_architecture
from .spec import ModelSpec, PartSpec, Run, layer

MIXERS = ("attention",)
GLU_ALPHA = 1.702      # the experts' g * sigmoid(alpha g)
GROUP_TOP = 2          # a group of experts counts as the sum of so many best scores


@dataclass(frozen=True)
class KisusunConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    logit_scale: float
    layers: Tuple[dict, ...]          # as config.json gives them (checked in __post_init__, never changed afterwards)

    architecture = "Kisusun"

    def __hash__(self):
        return hash(json.dumps(self.to_dict(), sort_keys=True))

    def __post_init__(self):
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError("vocab and width must be positive")
        if not self.norm_eps >= 0:
            raise ConfigError(f"norm.eps must be >= 0, got {self.norm_eps}")
        if not self.layers:
            raise ConfigError("config.json: 'layers' is empty")
        first = None       # (place, values a token) of the first layer that blends its values
        for i, entry in enumerate(self.layers):
            where = f"layers[{i}]"
            kind = entry.get("type") if isinstance(entry, dict) else None
            if kind not in MIXERS:
                raise ConfigError(f"config.json: {where}.type is {kind!r}; this design has {', '.join(MIXERS)}")
            m = entry.get("mixer")
            for k in ("heads", "kv_heads", "dim", "vdim"):
                _need(m, k, where + ".mixer")
            if not _need(m, "scale", where + ".mixer", float) > 0:
                raise ConfigError(f"config.json: {where}.mixer.scale must be positive")
            if m["heads"] % m["kv_heads"]:
                raise ConfigError(f"config.json: {where}.mixer: {m['heads']} heads cannot share {m['kv_heads']} kv_heads")
            if m.get("softcap") is not None and not _need(m, "softcap", where + ".mixer", float) > 0:
                raise ConfigError(f"config.json: {where}.mixer.softcap must be positive")
            rot = m.get("rot")
            if rot is not None:
                _need(rot, "base", where + ".mixer.rot", float)
                dims = _need(rot, "dims", where + ".mixer.rot", positive=False)
                if dims % 2 or dims > m["dim"]:
                    raise ConfigError(f"config.json: {where}.mixer.rot.dims = {dims} must be even and at most dim")
                if rot.get("scaling") is not None and not _need(rot["scaling"], "factor", where + ".mixer.rot.scaling", float) > 0:
                    raise ConfigError(f"config.json: {where}.mixer.rot.scaling.factor must be positive")
            if m.get("mask") is not None:
                _need(m["mask"], "size", where + ".mixer.mask")
            if m.get("v_mix"):
                size = m["kv_heads"] * m["vdim"]
                if first is None:
                    first = (i, size)
                elif size != first[1]:
                    raise ConfigError(f"config.json: {where}.mixer: {size} values a token cannot be blended with the "
                                      f"{first[1]} of layers[{first[0]}]")
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
            _need(r, "scale", where + ".router", float)
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
    def from_dict(cls, d: dict) -> "KisusunConfig":
        layers = d.get("layers")
        if not isinstance(layers, list):
            raise ConfigError("config.json lacks the list 'layers'")
        return cls(vocab=_need(d, "vocab", "config"), width=_need(d, "width", "config"),
                   norm_eps=_need(d.get("norm"), "eps", "norm", float),
                   embedding_scale=_need(d.get("embedding"), "scale", "embedding", float),
                   logit_scale=_need(d, "logit_scale", "config", float), layers=tuple(copy.deepcopy(e) for e in layers))

    def to_dict(self) -> dict:
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "embedding": {"scale": self.embedding_scale}, "logit_scale": self.logit_scale,
                "layers": [copy.deepcopy(e) for e in self.layers]}

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
    def _norm(self, prefix: str, name: str, gain: float = 1.0) -> PartSpec:
        return PartSpec("rms_norm", prefix, {"size": self.width, "eps": self.norm_eps, "name": name, "gain": gain})

    def _mixer(self, i: int, m: dict, value_blend: Optional[str]) -> Tuple[PartSpec, PartSpec]:
        """(mixer PartSpec, position PartSpec) of layer i."""
        p, rot = f"l{i}.mix.", m.get("rot") or {}
        position = PartSpec("qk_norm_rotary_half", p, {
            "head_dim": m["dim"], "eps": self.norm_eps, "over": "projection", "heads": (m["heads"], m["kv_heads"]),
            "dims": int(rot.get("dims", 0)), "base": float(rot.get("base", 10000.0)),
            "scaling": (("factor", float(rot["scaling"]["factor"])),) if rot.get("scaling") is not None else None})
        mixer = PartSpec("gqa_attention", p, {
            "hidden_size": self.width, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "value_dim": m["vdim"], "scale": float(m["scale"]), "qkv_bias": False, "out_bias": False, "sink": "zero",
            "softcap": float(m["softcap"]) if m.get("softcap") is not None else None,
            "window": m["mask"]["size"] if m.get("mask") is not None else None, "gate": "entry", "value_blend": value_blend,
            "names": {"q": "q", "k": "k", "v": "v", "o": "o", "gate": "g", "blend": "vmix"}})
        return mixer, position

    def _feed_forward(self, i: int, mlp: dict) -> PartSpec:
        p, W = f"l{i}.mlp.", self.width
        if mlp["kind"] == "dense":
            return PartSpec("gated_glu", p, {"hidden_size": W, "intermediate_size": mlp["ff"], "activation": "silu"})
        r, shared = mlp["router"], mlp.get("shared")
        groups = (r["groups"]["count"], r["groups"]["keep"]) if r.get("groups") is not None else None
        return PartSpec("routed_experts", p, {
            "hidden_size": W, "expert_ff": mlp["expert"]["ff"], "experts": r["experts"], "top": r["top"], "groups": groups,
            "group_top": GROUP_TOP, "scores": "sigmoid", "correction": False, "weight_scale": float(r["scale"]),
            "activation": "clamped_glu", "limit": float(mlp["expert"]["limit"]), "alpha": GLU_ALPHA,
            "shared_ff": shared["ff"] if shared is not None else 0,
            "shared_limit": float(shared["limit"]) if shared is not None else None, "shared_gate": False})

    def to_spec(self) -> ModelSpec:
        W = self.width
        layers, ignorable = [], []
        first = next((i for i, e in enumerate(self.layers) if e["mixer"].get("v_mix")), None)
        for i, entry in enumerate(self.layers):
            p, m, mlp = f"l{i}.", entry["mixer"], entry.get("mlp")
            blend = None if not m.get("v_mix") else ("first" if i == first else "blend")
            mixer, position = self._mixer(i, m, blend)
            layers.append(layer(
                "post_norm_residual", position=position, mixer=mixer, mixer_post_norm=self._norm(p, "norm1"),
                feed_forward=self._feed_forward(i, mlp) if mlp is not None else None,
                feed_forward_post_norm=self._norm(p, "norm2") if mlp is not None else None))
            # what a layer has no use for, if a checkpoint has it
            if blend != "blend":
                ignorable.append(p + "mix.vmix")
            if mlp is None:
                ignorable.append(p + "norm2")
        return ModelSpec(
            architecture=self.architecture, hidden_size=W, vocab_size=self.vocab,
            embedding=PartSpec("token_embedding", "", {"vocab_size": self.vocab, "hidden_size": W, "name": "embed",
                                                       "scale": self.embedding_scale}),
            layers=tuple(layers), order=tuple(Run(i) for i in range(len(layers))),
            final_norm=self._norm("final.", "norm", gain=self.logit_scale),
            head=PartSpec("lm_head", "", {"hidden_size": W, "vocab_size": self.vocab, "tied_to": "embed", "name": "head"}),
            ignorable=tuple(ignorable),
        )


register_architecture(KisusunConfig.architecture, KisusunConfig, model_type="kisusun")
