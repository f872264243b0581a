"""Typed configuration of the Lemotar decoder, read from config.json keys.

A Lemotar model is a list of layers whose norms sit on the sum of the scaled stream and a
sublayer's output, x <- norm1(alpha x + mixer(x)); x <- norm2(alpha x + ff(x)), every norm's
weight stored around zero.  The embedding rows are multiplied by a constant; the model ends with
a norm of the same kind and a head of its own.  config.json:

    architecture     "Lemotar"
    vocab, width     sizes of the table and of the stream
    norm.eps         eps of every norm
    embedding.scale  multiplier of the embedding rows
    postln_alpha     the stream's multiplier where a sublayer's output joins it
    layers[i]        type     "parallel" | "latent_attention"
                     mixer    parallel: left  {heads, kv_heads, dim, vdim, scale, softcap, mask
                                               {size}, rot {base, dims}}
                                        right {heads, kv_heads, dim, vdim, conv}
                              latent_attention: heads, dim, rot_dim, vdim, kv_rank, scale, mask
                                        {size}, rot {base, dims, scaling {factor, original, fast,
                                        slow}}, kv_from
                     mlp      null, or {kind: "dense", ff}

Mixers: `parallel` is window attention whose values are its keys as projected, with a norm over
the whole query and key projections, a rotation of neighbouring pairs, capped scores and a one in
the softmax's denominator (`parts.attention.Attention`), beside the gated delta rule with a decay
per key channel and low-rank decay and gate (`parts.delta.GatedDelta`), joined by
`parts.parallel.ParallelMixer`; `latent_attention` caches one latent and one rotated key part a
position (`parts.latent.LatentAttention`), or reads those of an earlier layer (`kv_from`).
The two ranks are told by the checkpoint's tensors alone (`sized_by`).  Checkpoint names:
`embed`, `l<i>.norm1|norm2`, `l<i>.mix.*`, `l<i>.mlp.gate|up|down`, `final.norm`, `head`.
"""
from __future__ import annotations

import dataclasses
import math
from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple

from .specs import (AttentionSpec, GatedDeltaSpec, GatedMLPSpec, LatentAttentionSpec, LayerSpec,
                    ModelSpec, NormSpec, ParallelSpec, PositionSpec, ScheduleEntry, YarnScaling)

ARCHITECTURE = "Lemotar"
MAX_POSITIONS = 1 << 30        # no table of positions: a sequence is as long as the cache allows
UNIT_EPS = 1e-6                # queries and keys of the delta rule: x / sqrt(sum(x^2) + UNIT_EPS)
WEIGHT_OFFSET = 1.0            # the layers' and the final norm's weights are stored less this


class LemotarConfigError(ValueError):
    pass


def _int(source: Mapping[str, Any], key: str, where: str, least: int = 1) -> int:
    if key not in source:
        raise LemotarConfigError(f"config.json: {where} lacks '{key}'")
    value = source[key]
    if isinstance(value, bool) or not isinstance(value, (int, float)) or int(value) != value \
            or value < least or value > 2**31 - 1:
        raise LemotarConfigError(f"config.json: {where}.{key} must be an integer of at least "
                                 f"{least}, got {value!r}")
    return int(value)


def _number(source: Mapping[str, Any], key: str, where: str, positive: bool = True) -> float:
    if key not in source:
        raise LemotarConfigError(f"config.json: {where} lacks '{key}'")
    value = source[key]
    if isinstance(value, bool) or not isinstance(value, (int, float)) or not math.isfinite(value) \
            or (positive and value <= 0):
        raise LemotarConfigError(f"config.json: {where}.{key} must be a "
                                 f"{'positive ' if positive else ''}number, got {value!r}")
    return float(value)


def _object(source: Mapping[str, Any], key: str, where: str) -> Mapping[str, Any]:
    value = source.get(key)
    if not isinstance(value, dict):
        raise LemotarConfigError(f"config.json: {where} lacks the object '{key}'")
    return value


def _optional_object(source, key, where):
    value = source.get(key)
    if value is not None and not isinstance(value, dict):
        raise LemotarConfigError(f"config.json: {where}.{key} must be an object")
    return value


def _known_keys(source: Mapping[str, Any], known, where: str) -> None:
    """Options this decoder does not implement are refused, never ignored."""
    extra = sorted(set(source) - set(known))
    if extra:
        raise LemotarConfigError(f"config.json: {where} has keys this decoder does not know: {extra}")


def _window(source, where) -> Optional[int]:
    mask = _optional_object(source, "mask", where)
    if mask is None or mask.get("size") is None:
        return None
    _known_keys(mask, ("size",), where + ".mask")
    return _int(mask, "size", where + ".mask")


@dataclass(frozen=True)
class LemotarRotation:
    base: float
    dims: int
    scaling: Optional[YarnScaling] = None

    @classmethod
    def from_dict(cls, source, key, where, widest, scaled):
        rot = _optional_object(source, key, where)
        if rot is None:
            return None
        where = f"{where}.{key}"
        _known_keys(rot, ("base", "dims", "scaling") if scaled else ("base", "dims"), where)
        dims = _int(rot, "dims", where, least=2)
        if dims % 2 or dims > widest:
            raise LemotarConfigError(f"config.json: {where}.dims must be even and at most {widest}")
        made = None
        scaling = _optional_object(rot, "scaling", where) if scaled else None
        if scaling is not None:
            inner = where + ".scaling"
            _known_keys(scaling, ("factor", "original", "fast", "slow"), inner)
            made = YarnScaling(**{name: _number(scaling, name, inner)
                                  for name in ("factor", "original", "fast", "slow")})
        return cls(base=_number(rot, "base", where), dims=dims, scaling=made)

    def to_dict(self):
        out = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = dataclasses.asdict(self.scaling)
        return out


@dataclass(frozen=True)
class LemotarSoftmax:
    """The softmax half of a parallel mixer."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: Optional[float]                 # None: scores as they are
    window: Optional[int]                    # mask.size; None: every earlier position
    rot: Optional[LemotarRotation]

    @classmethod
    def from_dict(cls, source, where):
        _known_keys(source, ("heads", "kv_heads", "dim", "vdim", "scale", "softcap", "mask", "rot"),
                    where)
        dim = _int(source, "dim", where)
        made = cls(heads=_int(source, "heads", where), kv_heads=_int(source, "kv_heads", where),
                   dim=dim, vdim=_int(source, "vdim", where), scale=_number(source, "scale", where),
                   softcap=(None if source.get("softcap") is None
                            else _number(source, "softcap", where)),
                   window=_window(source, where),
                   rot=LemotarRotation.from_dict(source, "rot", where, dim, scaled=False))
        if made.heads % made.kv_heads:
            raise LemotarConfigError(f"config.json: {where}.heads must be a multiple of kv_heads")
        if made.vdim != made.dim:
            raise LemotarConfigError(f"config.json: {where}.vdim must be dim: the values are the keys")
        return made

    def to_dict(self):
        out = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
               "scale": self.scale, "vdim": self.vdim}
        if self.softcap is not None:
            out["softcap"] = self.softcap
        if self.window is not None:
            out["mask"] = {"size": self.window}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class LemotarDelta:
    """The recurrent half of a parallel mixer.  The two ranks are not keys of config.json: None
    stands for one head's key or value size until a checkpoint tells them."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: Optional[int] = None
    gate_rank: Optional[int] = None

    @classmethod
    def from_dict(cls, source, where):
        _known_keys(source, ("heads", "kv_heads", "dim", "vdim", "conv"), where)
        made = cls(**{name: _int(source, name, where)
                      for name in ("heads", "kv_heads", "dim", "vdim", "conv")})
        if made.heads % made.kv_heads:
            raise LemotarConfigError(f"config.json: {where}.heads must be a multiple of kv_heads")
        return made

    def to_dict(self):
        return {"conv": self.conv, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                "vdim": self.vdim}


@dataclass(frozen=True)
class LemotarParallel:
    left: LemotarSoftmax
    right: LemotarDelta

    type = "parallel"

    @classmethod
    def from_dict(cls, source, where):
        _known_keys(source, ("left", "right"), where)
        return cls(left=LemotarSoftmax.from_dict(_object(source, "left", where), where + ".left"),
                   right=LemotarDelta.from_dict(_object(source, "right", where), where + ".right"))

    def to_dict(self):
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


@dataclass(frozen=True)
class LemotarLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: Optional[int]
    rot: Optional[LemotarRotation]
    kv_from: Optional[int]                   # the layer whose latents this one reads

    type = "latent_attention"

    @classmethod
    def from_dict(cls, source, where):
        _known_keys(source, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "mask", "rot",
                             "kv_from"), where)
        rot_dim = _int(source, "rot_dim", where, least=0)
        made = cls(heads=_int(source, "heads", where), dim=_int(source, "dim", where),
                   rot_dim=rot_dim, vdim=_int(source, "vdim", where),
                   kv_rank=_int(source, "kv_rank", where), scale=_number(source, "scale", where),
                   window=_window(source, where),
                   rot=LemotarRotation.from_dict(source, "rot", where, rot_dim, scaled=True)
                   if rot_dim else None,
                   kv_from=(None if source.get("kv_from") is None
                            else _int(source, "kv_from", where, least=0)))
        if rot_dim and (made.rot is None or made.rot.dims != rot_dim):
            raise LemotarConfigError(f"config.json: {where}.rot.dims must be rot_dim")
        return made

    def to_dict(self):
        out = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank,
               "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


MIXERS = {"parallel": LemotarParallel, "latent_attention": LemotarLatent}


@dataclass(frozen=True)
class LemotarLayer:
    mixer: object                # one of the two mixer configurations
    ff: Optional[int]            # hidden size of the feed-forward; None: the layer has none

    @classmethod
    def from_dict(cls, source, where):
        if not isinstance(source, dict):
            raise LemotarConfigError(f"config.json: {where} must be an object")
        _known_keys(source, ("type", "mixer", "mlp"), where)
        kind = source.get("type")
        if kind not in MIXERS:
            raise LemotarConfigError(f"config.json: {where}.type must be one of {sorted(MIXERS)}, "
                                     f"got {kind!r}")
        mixer = MIXERS[kind].from_dict(_object(source, "mixer", where), where + ".mixer")
        mlp = _optional_object(source, "mlp", where)
        if mlp is None:
            return cls(mixer=mixer, ff=None)
        _known_keys(mlp, ("kind", "ff"), where + ".mlp")
        if mlp.get("kind") != "dense":
            raise LemotarConfigError(f"config.json: {where}.mlp.kind must be 'dense', "
                                     f"got {mlp.get('kind')!r}")
        return cls(mixer=mixer, ff=_int(mlp, "ff", where + ".mlp"))

    def to_dict(self):
        return {"mixer": self.mixer.to_dict(),
                "mlp": None if self.ff is None else {"ff": self.ff, "kind": "dense"},
                "type": self.mixer.type}


@dataclass(frozen=True)
class LemotarConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    alpha: float
    layers: Tuple[LemotarLayer, ...]

    architecture = ARCHITECTURE

    @classmethod
    def from_dict(cls, source: Mapping[str, Any]) -> "LemotarConfig":
        # (keys of the top level that the decoder does not know are a file's own notes; inside
        # a layer an unknown key would change what is computed, and is refused)
        norm = _object(source, "norm", "the top level")
        _known_keys(norm, ("eps",), "norm")
        embedding = _object(source, "embedding", "the top level")
        _known_keys(embedding, ("scale",), "embedding")
        layers = source.get("layers")
        if not isinstance(layers, list) or not layers:
            raise LemotarConfigError("config.json: 'layers' must be a list of at least one layer")
        config = cls(vocab=_int(source, "vocab", "the top level"),
                     width=_int(source, "width", "the top level"),
                     norm_eps=_number(norm, "eps", "norm"),
                     embedding_scale=_number(embedding, "scale", "embedding", positive=False),
                     alpha=_number(source, "postln_alpha", "the top level", positive=False),
                     layers=tuple(LemotarLayer.from_dict(layer, f"layers[{index}]")
                                  for index, layer in enumerate(layers)))
        for index, layer in enumerate(config.layers):
            mixer = layer.mixer
            source_index = getattr(mixer, "kv_from", None)
            if source_index is None:
                continue
            where = f"layers[{index}].mixer.kv_from"
            if source_index >= index:
                raise LemotarConfigError(f"config.json: {where} must name an earlier layer")
            other = config.layers[source_index].mixer
            if not isinstance(other, LemotarLatent) or other.kv_from is not None:
                raise LemotarConfigError(f"config.json: {where} must name a latent_attention layer "
                                         "with latents of its own")
            if (other.kv_rank, other.rot_dim, other.rot) != (mixer.kv_rank, mixer.rot_dim, mixer.rot):
                raise LemotarConfigError(f"config.json: {where}: the two layers' latents or "
                                         "rotations differ")
        return config

    def to_dict(self) -> dict:
        """config.json content that `from_dict` reads back to an equal object (but for ranks that
        a checkpoint has told)."""
        return {"architecture": ARCHITECTURE, "embedding": {"scale": self.embedding_scale},
                "layers": [layer.to_dict() for layer in self.layers],
                "norm": {"eps": self.norm_eps}, "postln_alpha": self.alpha, "vocab": self.vocab,
                "width": self.width}

    def sized_by(self, shapes: Mapping[str, Tuple[int, ...]]) -> "LemotarConfig":
        """This configuration with the ranks of the low-rank decay and gate as a checkpoint's
        tensors (name -> shape) tell them."""
        layers = []
        for index, layer in enumerate(self.layers):
            if isinstance(layer.mixer, LemotarParallel):
                ranks = {}
                for field, name in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    shape = shapes.get(f"l{index}.mix.right.{name}")
                    if shape is not None and len(shape) == 2:
                        ranks[field] = int(shape[0])
                right = dataclasses.replace(layer.mixer.right, **ranks)
                layer = dataclasses.replace(layer, mixer=dataclasses.replace(layer.mixer, right=right))
            layers.append(layer)
        return dataclasses.replace(self, layers=tuple(layers))

    # ------------------------------------------------------------------
    def _cache_span(self, index: int) -> Optional[int]:
        """What layer `index`'s cache must keep for the layers that read it: None if its own
        window says enough, 0 (everything) if a reader has none, else the widest window."""
        users = [self.layers[index].mixer] + [layer.mixer for layer in self.layers
                                              if getattr(layer.mixer, "kv_from", None) == index]
        if len(users) == 1:
            return None
        if any(user.window is None for user in users):
            return 0
        return max(user.window for user in users)

    @staticmethod
    def _position(rot: Optional[LemotarRotation], kind: str) -> PositionSpec:
        if rot is None:
            return PositionSpec(kind="none")
        return PositionSpec(kind=kind, theta=rot.base, dim=rot.dims, scaling=rot.scaling)

    def _mixer_spec(self, index: int, mixer):
        if isinstance(mixer, LemotarLatent):
            return LatentAttentionSpec(
                n_heads=mixer.heads, head_dim=mixer.dim, rot_dim=mixer.rot_dim,
                value_dim=mixer.vdim, kv_rank=mixer.kv_rank, q_rank=0, scale=mixer.scale,
                norm_eps=self.norm_eps, position=self._position(mixer.rot, "rope_half"), sink=True,
                output_gate="element", window=mixer.window, shared_kv=mixer.kv_from is not None,
                cache_span=None if mixer.kv_from is not None else self._cache_span(index))
        left, right = mixer.left, mixer.right
        softmax = AttentionSpec(
            n_heads=left.heads, n_kv_heads=left.kv_heads, head_dim=left.dim, value_dim=left.vdim,
            qkv_bias=False, o_bias=False, qk_norm=True, qk_norm_scope="projection",
            qk_norm_eps=self.norm_eps, values_from_keys=True, scale=left.scale,
            softcap=left.softcap, window=left.window, unit_sink=True,
            position=self._position(left.rot, "rope_pairs"))
        delta = GatedDeltaSpec(
            n_heads=right.heads, n_kv_heads=right.kv_heads, key_dim=right.dim,
            value_dim=right.vdim, conv_taps=right.conv, out_norm_eps=self.norm_eps,
            unit_eps=UNIT_EPS, decay_rank=right.decay_rank or right.dim,
            gate_rank=right.gate_rank or right.vdim, gate_activation="sigmoid")
        return ParallelSpec(branches=(softmax, delta), names=("left", "right"),
                            norm_eps=self.norm_eps)

    def model_spec(self) -> ModelSpec:
        norm = NormSpec(kind="rmsnorm", eps=self.norm_eps, weight_offset=WEIGHT_OFFSET)
        layers, schedule = [], []
        for index, layer in enumerate(self.layers):
            feed_forward = None if layer.ff is None else GatedMLPSpec(
                intermediate_size=layer.ff, activation="silu", bias=False)
            layers.append(LayerSpec(block="postnorm", norm=norm,
                                    mixer=self._mixer_spec(index, layer.mixer),
                                    feed_forward=feed_forward, stream_scale=self.alpha))
            source = getattr(layer.mixer, "kv_from", None)
            schedule.append(ScheduleEntry(layer=index, cache=index) if source is None else
                            ScheduleEntry(layer=index, cache=source, writes_cache=False))
        spec = ModelSpec(architecture=ARCHITECTURE, vocab_size=self.vocab, hidden_size=self.width,
                         layers=tuple(layers), schedule=tuple(schedule), final_norm=norm,
                         tie_word_embeddings=False, max_position_embeddings=MAX_POSITIONS,
                         bos_token_id=None, eos_token_id=None,
                         embedding_scale=self.embedding_scale)
        spec.validate()
        return spec

    # ------------------------------------------------------------------
    _LATENT_NAMES = {"q_proj.weight": "q", "kv_down.weight": "dkv", "kv_down_norm.weight": "dkv.norm",
                     "k_up.weight": "uk", "v_up.weight": "uv", "sink": "sink",
                     "gate_proj.weight": "g", "o_proj.weight": "o"}
    _SOFTMAX_NAMES = {"q_proj.weight": "q", "k_proj.weight": "k", "q_norm.weight": "q.norm",
                      "k_norm.weight": "k.norm", "o_proj.weight": "o"}
    _DELTA_NAMES = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v",
                    "q_conv.weight": "q.conv", "k_conv.weight": "k.conv", "v_conv.weight": "v.conv",
                    "beta_proj.weight": "b", "decay_down.weight": "a1", "decay_up.weight": "a2",
                    "decay_log_rate": "A_log", "decay_bias": "dt_bias", "gate_down.weight": "g1",
                    "gate_up.weight": "g2", "out_norm.weight": "norm", "o_proj.weight": "o"}
    _DENSE_NAMES = {"gate_proj.weight": "gate", "up_proj.weight": "up", "down_proj.weight": "down"}

    def checkpoint_name(self, parameter: str) -> str:
        """Name of a model parameter in the checkpoint."""
        top = {"embed.weight": "embed", "final_norm.weight": "final.norm", "head.weight": "head",
               "head.bias": "head.b"}
        if parameter in top:
            return top[parameter]
        parts = parameter.split(".", 3)
        if parts[0] == "layers" and len(parts) == 4 and parts[1].isdigit() \
                and int(parts[1]) < len(self.layers):
            index, part, rest = int(parts[1]), parts[2], parts[3]
            if part in ("norm1", "norm2") and rest == "weight":
                return f"l{index}.{part}"
            if part == "mixer":
                if isinstance(self.layers[index].mixer, LemotarLatent):
                    if rest in self._LATENT_NAMES:
                        return f"l{index}.mix.{self._LATENT_NAMES[rest]}"
                else:
                    side, _, inner = rest.partition(".")
                    if side in ("left_out", "right_out") and inner == "weight":
                        return f"l{index}.mix.{side[:-4]}.out"
                    table = {"left": self._SOFTMAX_NAMES, "right": self._DELTA_NAMES}.get(side)
                    if table is not None and inner in table:
                        return f"l{index}.mix.{side}.{table[inner]}"
            if part == "ffn" and rest in self._DENSE_NAMES:
                return f"l{index}.mlp.{self._DENSE_NAMES[rest]}"
        raise KeyError(f"Lemotar has no checkpoint tensor for parameter '{parameter}'")
