"""Typed configuration of the Dazapel decoder, read from config.json keys.

A Dazapel model is a list of layers with an RMS norm before and after every sublayer, whose
contribution to the stream is multiplied by `residual_mult`.  A span of layers may run several
times in a row with the same weights (`loop`); before each pass a learned vector of that pass
is added to the stream.  The head is the embedding table.  config.json:

    architecture    "Dazapel"
    vocab, width    sizes of the table and of the stream
    norm.eps        eps of every RMS norm
    residual_mult   multiplier of every sublayer's contribution
    loop            null, or {start, stop, times}: layers start .. stop - 1 run `times` times
    layers[i]       type     "attention"
                    mixer    heads, kv_heads, dim, vdim, scale, mask {size, keep_first},
                             rot {base, dims, scaling {factor, original, fast, slow}}
                    mlp      null, or {kind: "moe", expert {ff, limit},
                             router {experts, top, scale, groups {count, keep}},
                             shared {ff, limit}}

The mixer is grouped-query attention with biased projections, a rotation of the first rot.dims
elements of a head whose frequencies may be stretched, queries and keys brought to unit RMS
after it, a sliding window that keeps the sequence's first tokens visible, and a sigmoid gate on
every element of the heads (`parts.attention.Attention` with those options).  The feed-forward
is a mixture of experts with sigmoid scores chosen within groups, renormalised and scaled
weights, clamped-swish experts and an expert that every token takes (`parts.moe.RoutedMLP`).
Checkpoint names: `embed`, `loop.step`, `l<i>.norm1|norm1b|norm2|norm2b`, `l<i>.mix.*`,
`l<i>.mlp.*`, `final.norm`.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple

from .specs import (AttentionSpec, GatedMLPSpec, LayerSpec, LoopSpec, ModelSpec, NormSpec,
                    PositionSpec, RoutedMLPSpec, YarnScaling, default_schedule, looped_schedule)

ARCHITECTURE = "Dazapel"
SWISH_ALPHA = 1.702            # a constant the design fixes: the swish's slope
MAX_POSITIONS = 1 << 30        # no table of positions: a sequence is as long as the cache allows


class DazapelConfigError(ValueError):
    pass


def _int(source: Mapping[str, Any], key: str, where: str, least: int = 1) -> int:
    if key not in source:
        raise DazapelConfigError(f"config.json: {where} lacks '{key}'")
    value = source[key]
    if isinstance(value, bool) or not isinstance(value, (int, float)) or int(value) != value \
            or value < least or value > 2**31 - 1:
        raise DazapelConfigError(f"config.json: {where}.{key} must be an integer of at least "
                                 f"{least}, got {value!r}")
    return int(value)


def _number(source: Mapping[str, Any], key: str, where: str, above: Optional[float] = 0.0) -> float:
    if key not in source:
        raise DazapelConfigError(f"config.json: {where} lacks '{key}'")
    value = source[key]
    if isinstance(value, bool) or not isinstance(value, (int, float)) or not math.isfinite(value) \
            or (above is not None and value <= above):
        raise DazapelConfigError(f"config.json: {where}.{key} must be a number"
                                 + ("" if above is None else f" above {above:g}")
                                 + f", got {value!r}")
    return float(value)


def _object(source: Mapping[str, Any], key: str, where: str) -> Mapping[str, Any]:
    value = source.get(key)
    if not isinstance(value, dict):
        raise DazapelConfigError(f"config.json: {where} lacks the object '{key}'")
    return value


def _optional_object(source, key, where):
    value = source.get(key)
    if value is not None and not isinstance(value, dict):
        raise DazapelConfigError(f"config.json: {where}.{key} must be an object or null")
    return value


def _known_keys(source: Mapping[str, Any], known, where: str) -> None:
    """Options this decoder does not implement are refused, never ignored."""
    extra = sorted(set(source) - set(known))
    if extra:
        raise DazapelConfigError(f"config.json: {where} has keys this decoder does not know: {extra}")


@dataclass(frozen=True)
class DazapelRotation:
    base: float
    dims: int
    scaling: Optional[YarnScaling]           # None: the frequencies as they are

    @classmethod
    def from_dict(cls, source, where):
        _known_keys(source, ("base", "dims", "scaling"), where)
        scaling = _optional_object(source, "scaling", where)
        if scaling is not None:
            _known_keys(scaling, ("factor", "original", "fast", "slow"), where + ".scaling")
            scaling = YarnScaling(**{key: _number(scaling, key, where + ".scaling")
                                     for key in ("factor", "original", "fast", "slow")})
        made = cls(base=_number(source, "base", where), dims=_int(source, "dims", where, least=2),
                   scaling=scaling)
        if made.scaling is not None and made.base == 1.0:
            raise DazapelConfigError(f"config.json: {where}: a base of 1 has no wavelengths to stretch")
        return made

    def to_dict(self):
        out = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = {"factor": self.scaling.factor, "fast": self.scaling.fast,
                              "original": self.scaling.original, "slow": self.scaling.slow}
        return out


@dataclass(frozen=True)
class DazapelAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int]                    # mask.size; None: every earlier position
    keep_first: int                          # mask.keep_first
    rot: Optional[DazapelRotation]           # None: no rotation

    type = "attention"

    @classmethod
    def from_dict(cls, source, where):
        _known_keys(source, ("heads", "kv_heads", "dim", "vdim", "scale", "mask", "rot"), where)
        window, keep_first = None, 0
        mask = _optional_object(source, "mask", where)
        if mask is not None:
            _known_keys(mask, ("size", "keep_first"), where + ".mask")
            if mask.get("size") is not None:
                window = _int(mask, "size", where + ".mask")
            if mask.get("keep_first") is not None:
                keep_first = _int(mask, "keep_first", where + ".mask", least=0)
        rot = _optional_object(source, "rot", where)
        made = cls(heads=_int(source, "heads", where), kv_heads=_int(source, "kv_heads", where),
                   dim=_int(source, "dim", where), vdim=_int(source, "vdim", where),
                   scale=_number(source, "scale", where), window=window, keep_first=keep_first,
                   rot=None if rot is None else DazapelRotation.from_dict(rot, where + ".rot"))
        if made.heads % made.kv_heads:
            raise DazapelConfigError(f"config.json: {where}.heads must be a multiple of kv_heads")
        if made.rot is not None and (made.rot.dims % 2 or made.rot.dims > made.dim):
            raise DazapelConfigError(f"config.json: {where}.rot.dims must be even and at most dim")
        return made

    def to_dict(self):
        out = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
               "scale": self.scale, "vdim": self.vdim}
        if self.window is not None or self.keep_first:
            out["mask"] = {"keep_first": self.keep_first}
            if self.window is not None:
                out["mask"]["size"] = self.window
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out


MIXERS = {"attention": DazapelAttention}


@dataclass(frozen=True)
class DazapelExpert:
    ff: int
    limit: float

    @classmethod
    def from_dict(cls, source, where):
        _known_keys(source, ("ff", "limit"), where)
        return cls(ff=_int(source, "ff", where), limit=_number(source, "limit", where))

    def to_dict(self):
        return {"ff": self.ff, "limit": self.limit}


@dataclass(frozen=True)
class DazapelExperts:
    expert: DazapelExpert
    experts: int
    top: int
    scale: float
    groups: int
    keep: int                                # groups that take part
    shared: Optional[DazapelExpert]          # None: no expert that every token takes

    kind = "moe"

    @classmethod
    def from_dict(cls, mlp, where):
        if mlp.get("kind") != "moe":
            raise DazapelConfigError(f"config.json: {where}.kind must be 'moe', got {mlp.get('kind')!r}")
        _known_keys(mlp, ("kind", "expert", "router", "shared"), where)
        router = _object(mlp, "router", where)
        _known_keys(router, ("experts", "top", "scale", "groups"), where + ".router")
        groups = _optional_object(router, "groups", where + ".router")
        count = keep = 1
        if groups is not None:
            _known_keys(groups, ("count", "keep"), where + ".router.groups")
            count = _int(groups, "count", where + ".router.groups")
            keep = _int(groups, "keep", where + ".router.groups")
        shared = _optional_object(mlp, "shared", where)
        made = cls(expert=DazapelExpert.from_dict(_object(mlp, "expert", where), where + ".expert"),
                   experts=_int(router, "experts", where + ".router"),
                   top=_int(router, "top", where + ".router"),
                   scale=_number(router, "scale", where + ".router", above=None),
                   groups=count, keep=keep,
                   shared=None if shared is None
                   else DazapelExpert.from_dict(shared, where + ".shared"))
        if made.experts % count or keep > count:
            raise DazapelConfigError(f"config.json: {where}.router.groups: {count} groups of which "
                                     f"{keep} are kept do not fit {made.experts} experts")
        if made.top > made.experts // count * keep:
            raise DazapelConfigError(f"config.json: {where}.router.top is above the experts of the "
                                     "kept groups")
        return made

    def to_dict(self):
        out = {"expert": self.expert.to_dict(), "kind": "moe",
               "router": {"experts": self.experts, "groups": {"count": self.groups, "keep": self.keep},
                          "scale": self.scale, "top": self.top}}
        if self.shared is not None:
            out["shared"] = self.shared.to_dict()
        return out


@dataclass(frozen=True)
class DazapelLayer:
    mixer: DazapelAttention
    mlp: Optional[DazapelExperts]            # None: the layer has no feed-forward

    @classmethod
    def from_dict(cls, source, where):
        if not isinstance(source, dict):
            raise DazapelConfigError(f"config.json: {where} must be an object")
        _known_keys(source, ("type", "mixer", "mlp"), where)
        kind = source.get("type")
        if kind not in MIXERS:
            raise DazapelConfigError(f"config.json: {where}.type must be one of {sorted(MIXERS)}, "
                                     f"got {kind!r}")
        mlp = _optional_object(source, "mlp", where)
        return cls(mixer=MIXERS[kind].from_dict(_object(source, "mixer", where), where + ".mixer"),
                   mlp=None if mlp is None else DazapelExperts.from_dict(mlp, where + ".mlp"))

    def to_dict(self):
        return {"mixer": self.mixer.to_dict(),
                "mlp": None if self.mlp is None else self.mlp.to_dict(),
                "type": self.mixer.type}


@dataclass(frozen=True)
class DazapelConfig:
    vocab: int
    width: int
    norm_eps: float
    residual_mult: float
    layers: Tuple[DazapelLayer, ...]
    loop: Optional[Tuple[int, int, int]] = None      # (start, stop, times)

    architecture = ARCHITECTURE

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "DazapelConfig":
        # (keys of the top level that the decoder does not know are a file's own notes; inside
        # a layer an unknown key would change what is computed, and is refused)
        norm = _object(source, "norm", "the top level")
        _known_keys(norm, ("eps",), "norm")
        layers = source.get("layers")
        if not isinstance(layers, list) or not layers:
            raise DazapelConfigError("config.json: 'layers' must be a list of at least one layer")
        loop = _optional_object(source, "loop", "the top level")
        span = None
        if loop is not None:
            _known_keys(loop, ("start", "stop", "times"), "loop")
            span = (_int(loop, "start", "loop", least=0), _int(loop, "stop", "loop"),
                    _int(loop, "times", "loop"))
            if not span[0] < span[1] <= len(layers):
                raise DazapelConfigError(f"config.json: loop.start < loop.stop <= {len(layers)} "
                                         f"must hold, got {span[0]} and {span[1]}")
        return cls(vocab=_int(source, "vocab", "the top level"),
                   width=_int(source, "width", "the top level"),
                   norm_eps=_number(norm, "eps", "norm"),
                   residual_mult=_number(source, "residual_mult", "the top level", above=None),
                   layers=tuple(DazapelLayer.from_dict(layer, f"layers[{index}]")
                                for index, layer in enumerate(layers)),
                   loop=span)

    def to_dict(self) -> dict:
        """config.json content that `from_dict` reads back to an equal object."""
        return {"architecture": ARCHITECTURE, "layers": [layer.to_dict() for layer in self.layers],
                "loop": None if self.loop is None else
                {"start": self.loop[0], "stop": self.loop[1], "times": self.loop[2]},
                "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult,
                "vocab": self.vocab, "width": self.width}

    # ------------------------------------------------------------------
    def _mixer_spec(self, mixer: DazapelAttention) -> AttentionSpec:
        position = PositionSpec(kind="none") if mixer.rot is None else \
            PositionSpec(kind="rope_half", theta=mixer.rot.base, dim=mixer.rot.dims,
                         scaling=mixer.rot.scaling)
        return AttentionSpec(n_heads=mixer.heads, n_kv_heads=mixer.kv_heads, head_dim=mixer.dim,
                             value_dim=mixer.vdim, qkv_bias=True, o_bias=True, scale=mixer.scale,
                             window=mixer.window, keep_first=mixer.keep_first, position=position,
                             qk_unit_norm=True, qk_norm_eps=self.norm_eps, output_gate=True)

    @staticmethod
    def _feed_forward_spec(mlp: Optional[DazapelExperts]) -> Optional[RoutedMLPSpec]:
        if mlp is None:
            return None
        swish = dict(activation="clamped_swish", alpha=SWISH_ALPHA)
        shared = None if mlp.shared is None else \
            GatedMLPSpec(intermediate_size=mlp.shared.ff, limit=mlp.shared.limit, bias=False, **swish)
        return RoutedMLPSpec(n_experts=mlp.experts, top=mlp.top, intermediate_size=mlp.expert.ff,
                             scoring="sigmoid", weight_scale=mlp.scale, group_count=mlp.groups,
                             group_keep=mlp.keep, limit=mlp.expert.limit, shared=shared, **swish)

    def model_spec(self) -> ModelSpec:
        norm = NormSpec(kind="rmsnorm", eps=self.norm_eps)
        layers = tuple(LayerSpec(block="sandwich", norm=norm, mixer=self._mixer_spec(layer.mixer),
                                 feed_forward=self._feed_forward_spec(layer.mlp),
                                 residual_scale=self.residual_mult, defer_output=True)
                       for layer in self.layers)
        loop = None if self.loop is None else LoopSpec(*self.loop, remix=False)
        schedule = (default_schedule(len(layers)) if loop is None
                    else looped_schedule(len(layers), loop))
        spec = ModelSpec(architecture=ARCHITECTURE, vocab_size=self.vocab, hidden_size=self.width,
                         layers=layers, schedule=schedule, final_norm=norm,
                         tie_word_embeddings=True, max_position_embeddings=MAX_POSITIONS,
                         bos_token_id=None, eos_token_id=None, loop=loop)
        spec.validate()
        return spec

    # ------------------------------------------------------------------
    _MIXER_NAMES = {"q_proj.weight": "q", "q_proj.bias": "q.b", "k_proj.weight": "k",
                    "k_proj.bias": "k.b", "v_proj.weight": "v", "v_proj.bias": "v.b",
                    "gate_proj.weight": "g", "o_proj.weight": "o", "o_proj.bias": "o.b"}
    _EXPERT_NAMES = {"gate_proj.weight": "gate", "up_proj.weight": "up", "down_proj.weight": "down"}

    def checkpoint_name(self, parameter: str) -> str:
        """Name of a model parameter in the checkpoint."""
        top = {"embed.weight": "embed", "final_norm.weight": "final.norm", "head.weight": "head",
               "head.bias": "head.b", "loop.step": "loop.step"}
        if parameter in top:
            return top[parameter]
        parts = parameter.split(".", 3)
        if parts[0] == "layers" and len(parts) == 4 and parts[1].isdigit() \
                and int(parts[1]) < len(self.layers):
            index, part, rest = int(parts[1]), parts[2], parts[3]
            if part in ("norm1", "norm1b", "norm2", "norm2b") and rest == "weight":
                return f"l{index}.{part}"
            if part == "mixer" and rest in self._MIXER_NAMES:
                return f"l{index}.mix.{self._MIXER_NAMES[rest]}"
            if part == "ffn":
                if rest == "router.weight":
                    return f"l{index}.mlp.router"
                which, _, matrix = rest.partition(".")
                if which == "shared" and matrix in self._EXPERT_NAMES:
                    return f"l{index}.mlp.shared.{self._EXPERT_NAMES[matrix]}"
                expert, _, matrix = matrix.partition(".")    # experts.<e>.<gate|up|down>_proj.weight
                if which == "experts" and expert.isdigit() and matrix in self._EXPERT_NAMES:
                    return f"l{index}.mlp.e{expert}.{self._EXPERT_NAMES[matrix]}"
        raise KeyError(f"Dazapel has no checkpoint tensor for parameter '{parameter}'")
