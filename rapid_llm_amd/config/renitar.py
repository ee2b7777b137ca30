"""The Renitar decoder's typed configuration: the keys of its ``config.json``.

A Renitar model is a list of layers with one norm each, whose output the mixer and the feed-forward both
read; what they return is added to the stream times a constant.  A layer's mixer is gated linear
attention with a decay per key channel (``gla``), or two side by side (``parallel``): softmax attention in
chunks behind short convolutions, with capped scores and an output gate, and lightning attention with
fixed decays, each output normed before half of their sum is taken.  Its feed-forward is absent or a
mixture of ungated experts chosen by corrected scores, some of which return their input, with a gated
shared expert.  Every size and every constant that differs between models of the design is a key here,
or (the inner size of the decays' low-rank pair) in a tensor's shape.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .model_config import ConfigError, normalise_dtype_name, require

MIXER_TYPES = ("gla", "parallel")


def _object(where: str, data: Any) -> Mapping[str, Any]:
    if not isinstance(data, Mapping):
        raise ConfigError(f"{where} must be an object")
    return data


def _size(where: str, data: Any, key: str, least: int = 1) -> int:
    value = require(_object(where, data), key, int)
    if value < least:
        raise ConfigError(f"{where}: {key!r} must be at least {least}, got {value!r}")
    return value


def _number(where: str, data: Any, key: str, positive: bool = False) -> float:
    value = float(require(_object(where, data), key, float))
    if positive and not value > 0:
        raise ConfigError(f"{where}: {key!r} must be positive, got {value!r}")
    return value


@dataclass(frozen=True)
class GlaConfig:
    heads: int
    dim: int  # key channels of a head
    vdim: int  # value channels of a head
    tau: float  # decays are sigmoids to the power 1 / tau
    rank: int = 0  # inner size of the decays' two matrices; 0: whatever the checkpoint's tensors have

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "GlaConfig":
        rank = _size(where, data, "rank") if data.get("rank") else 0
        return cls(_size(where, data, "heads"), _size(where, data, "dim"), _size(where, data, "vdim"),
                   _number(where, data, "tau", positive=True), rank)

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}
        if self.rank:
            out["rank"] = self.rank
        return out


@dataclass(frozen=True)
class ChunkedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int  # size of a query or key head
    vdim: int  # size of a value head
    conv: int  # taps of the causal convolutions
    scale: float  # factor of the scores
    softcap: float  # and their cap
    chunk: int  # positions of a chunk
    rot_dims: int  # rotated channels of a head
    rot_base: float

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "ChunkedAttentionConfig":
        heads, kv_heads = _size(where, data, "heads"), _size(where, data, "kv_heads")
        if heads % kv_heads:
            raise ConfigError(f"{where}: {heads} heads are not divisible by {kv_heads} kv_heads")
        dim, vdim = _size(where, data, "dim"), _size(where, data, "vdim")
        if dim > 256 or vdim > 256:
            raise ConfigError(f"{where}: the attention kernels take head sizes up to 256, got {dim} and {vdim}")
        rot, mask = data.get("rot"), data.get("mask")
        dims = _size(where + ".rot", rot, "dims")
        if dims % 2 or dims > dim:
            raise ConfigError(f"{where}.rot: {dims} of a head's {dim} channels cannot rotate in pairs")
        return cls(heads, kv_heads, dim, vdim, _size(where, data, "conv"), _number(where, data, "scale"),
                   _number(where, data, "softcap", positive=True), _size(where + ".mask", mask, "size"), dims,
                   _number(where + ".rot", rot, "base", positive=True))

    def to_dict(self) -> dict[str, Any]:
        return {
            "heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv,
            "scale": self.scale, "softcap": self.softcap, "mask": {"size": self.chunk},
            "rot": {"dims": self.rot_dims, "base": self.rot_base},
        }


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]  # one a head

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "LightningConfig":
        heads = _size(where, data, "heads")
        decay = _object(where, data).get("decay")
        if not isinstance(decay, (list, tuple)) or len(decay) != heads:
            raise ConfigError(f"{where}: 'decay' must list one number for each of {heads} heads")
        if not all(isinstance(a, (int, float)) and not isinstance(a, bool) and 0 < a <= 1 for a in decay):
            raise ConfigError(f"{where}: decays are numbers in (0, 1], got {list(decay)}")
        return cls(heads, _size(where, data, "dim"), _size(where, data, "vdim"), tuple(float(a) for a in decay))

    def to_dict(self) -> dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}


@dataclass(frozen=True)
class ParallelConfig:
    left: ChunkedAttentionConfig
    right: LightningConfig

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "ParallelConfig":
        left, right = (_object(f"{where}.{side}", data.get(side)) for side in ("left", "right"))
        return cls(ChunkedAttentionConfig.from_dict(where + ".left", left), LightningConfig.from_dict(where + ".right", right))

    def to_dict(self) -> dict[str, Any]:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


_MIXER_CONFIGS = {"gla": GlaConfig, "parallel": ParallelConfig}


@dataclass(frozen=True)
class MixtureConfig:
    expert_ff: int  # hidden units of an expert
    experts: int  # experts with tensors
    identity: int  # and without: they return their input
    top: int  # experts a token uses
    scale: float  # factor of the chosen experts' scores
    shared_ff: int  # hidden units of the shared expert; 0: there is none

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "MixtureConfig":
        if data.get("kind", "moe") != "moe":
            raise ConfigError(f"{where}: feed-forward kind {data.get('kind')!r} is not known (only 'moe')")
        router, shared = data.get("router"), data.get("shared")
        r = where + ".router"
        experts = _size(r, router, "experts")
        identity = _size(r, router, "identity", least=0) if router.get("identity") is not None else 0
        top = _size(r, router, "top")
        if top > experts + identity:
            raise ConfigError(f"{r}: a token cannot use {top} of {experts + identity} experts")
        return cls(_size(where + ".expert", data.get("expert"), "ff"), experts, identity, top, _number(r, router, "scale"),
                   _size(where + ".shared", shared, "ff") if shared is not None else 0)

    def to_dict(self) -> dict[str, Any]:
        return {
            "kind": "moe", "expert": {"ff": self.expert_ff},
            "router": {"experts": self.experts, "identity": self.identity, "top": self.top, "scale": self.scale},
            "shared": {"ff": self.shared_ff} if self.shared_ff else None,
        }


@dataclass(frozen=True)
class RenitarLayerConfig:
    type: str  # one of MIXER_TYPES
    mixer: GlaConfig | ParallelConfig
    mlp: MixtureConfig | None  # None: the layer has no feed-forward

    def to_dict(self) -> dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None}


@dataclass(frozen=True)
class RenitarConfig:
    architecture: str
    width: int
    vocab: int
    norm_eps: float
    residual_mult: float  # factor of what a layer adds to the stream
    layers: tuple[RenitarLayerConfig, ...]
    torch_dtype: str
    eos_token_ids: tuple[int, ...] = ()

    # the names the rest of the engine asks any configuration for
    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], overrides: Mapping[str, Any] | None = None) -> "RenitarConfig":
        data = dict(data)
        if overrides:
            data.update(overrides)
        listed = data.get("layers")
        if not isinstance(listed, (list, tuple)) or not listed:
            raise ConfigError("config.json key 'layers' must list at least one layer")
        layers = []
        for i, entry in enumerate(listed):
            where = f"layers[{i}]"
            kind = require(_object(where, entry), "type", str)
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{where}: mixer type {kind!r} is not one of {', '.join(MIXER_TYPES)}")
            mixer = _object(where + ".mixer", entry.get("mixer"))
            mlp = entry.get("mlp")
            layers.append(RenitarLayerConfig(
                kind, _MIXER_CONFIGS[kind].from_dict(where + ".mixer", mixer),
                MixtureConfig.from_dict(where + ".mlp", _object(where + ".mlp", mlp)) if mlp is not None else None,
            ))
        eos = data.get("eos_token_id")
        eos_ids = () if eos is None else ((int(eos),) if isinstance(eos, int) else tuple(int(e) for e in eos))
        return cls(
            architecture=require(data, "architecture", str),
            width=_size("config.json", data, "width"),
            vocab=_size("config.json", data, "vocab"),
            norm_eps=_number("norm", data.get("norm"), "eps", positive=True),
            residual_mult=_number("config.json", data, "residual_mult"),
            layers=tuple(layers),
            torch_dtype=normalise_dtype_name(data.get("torch_dtype") or data.get("dtype") or "bfloat16"),
            eos_token_ids=eos_ids,
        )

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "architecture": self.architecture,
            "width": self.width,
            "vocab": self.vocab,
            "norm": {"eps": self.norm_eps},
            "residual_mult": self.residual_mult,
            "layers": [layer.to_dict() for layer in self.layers],
            "torch_dtype": self.torch_dtype,
        }
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out
