"""The Pefulorn decoder's typed configuration: the keys of its ``config.json``.

A Pefulorn model is a list of pre-norm layers whose norm weights are stored around zero.  A layer's
mixer is one of three: a gated delta rule with a decay per key channel behind short convolutions
(``channel_delta``), softmax attention without rotation beside a gated recurrence of one number a
channel, both reading the same input (``parallel``), or an RWKV-style recurrence with token-shift mixes
(``wkv``).  Its feed-forward is dense and gated with the tanh form of gelu and biases, or absent.  A span
of the layers may run several times in a row with the same weights; the embedding's output and a
learned vector return to the stream as a pass begins.  Every size and every constant that differs
between models of the design is a key here, or (inner sizes of low-rank pairs) in a tensor's shape.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .model_config import ConfigError, normalise_dtype_name, require

MIXER_TYPES = ("channel_delta", "parallel", "wkv")


def _object(where: str, data: Any) -> Mapping[str, Any]:
    if not isinstance(data, Mapping):
        raise ConfigError(f"{where} must be an object")
    return data


def _positive(where: str, data: Any, key: str) -> int:
    value = require(_object(where, data), key, int)
    if value < 1:
        raise ConfigError(f"{where}: {key!r} must be a positive integer, got {value!r}")
    return value


def _number(where: str, data: Any, key: str) -> float:
    return float(require(_object(where, data), key, float))


def _rank(where: str, data: Mapping[str, Any], key: str) -> int:
    """An optional inner size; 0: whatever the checkpoint's tensors have."""
    rank = data.get(key) or 0
    if not isinstance(rank, int) or isinstance(rank, bool) or rank < 0:
        raise ConfigError(f"{where}: {key} must be a size, got {rank!r}")
    return rank


def _grouped(where: str, data: Mapping[str, Any]) -> tuple[int, int]:
    heads = _positive(where, data, "heads")
    kv_heads = _positive(where, data, "kv_heads") if data.get("kv_heads") is not None else heads
    if heads % kv_heads:
        raise ConfigError(f"{where}: {heads} heads are not divisible by {kv_heads} kv_heads")
    return heads, kv_heads


@dataclass(frozen=True)
class ChannelDeltaConfig:
    heads: int
    kv_heads: int  # heads of queries and keys
    dim: int  # key channels of a head
    vdim: int  # value channels of a head
    conv: int  # taps of the causal convolutions
    decay_rank: int = 0
    gate_rank: int = 0

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "ChannelDeltaConfig":
        heads, kv_heads = _grouped(where, data)
        dim = _positive(where, data, "dim")
        vdim = _positive(where, data, "vdim") if data.get("vdim") is not None else dim
        return cls(heads, kv_heads, dim, vdim, _positive(where, data, "conv"), _rank(where, data, "decay_rank"),
                   _rank(where, data, "gate_rank"))

    def to_dict(self) -> dict[str, Any]:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}
        if self.decay_rank:
            out["decay_rank"] = self.decay_rank
        if self.gate_rank:
            out["gate_rank"] = self.gate_rank
        return out


@dataclass(frozen=True)
class DistanceAttentionConfig:
    heads: int
    kv_heads: int
    dim: int  # size of a query or key head
    vdim: int  # size of a value head
    scale: float  # factor of the scores
    # queries are multiplied by 1 + temp_coef * ln(floor((p + 1) / temp_every) + 1); 0: they are not
    temp_coef: float
    temp_every: float

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "DistanceAttentionConfig":
        heads, kv_heads = _grouped(where, data)
        dim = _positive(where, data, "dim")
        vdim = _positive(where, data, "vdim") if data.get("vdim") is not None else dim
        if dim > 256 or vdim > 256:
            raise ConfigError(f"{where}: the attention kernels take head sizes up to 256, got {dim} and {vdim}")
        coef, every = 0.0, 1.0
        temp = data.get("q_temp")
        if temp is not None:
            coef, every = _number(where + ".q_temp", temp, "coef"), _number(where + ".q_temp", temp, "every")
            if not every > 0:
                raise ConfigError(f"{where}.q_temp: every must be positive, got {every}")
        return cls(heads, kv_heads, dim, vdim, _number(where, data, "scale"), coef, every)

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
        }
        if self.temp_coef:
            out["q_temp"] = {"coef": self.temp_coef, "every": self.temp_every}
        return out


@dataclass(frozen=True)
class ParallelConfig:
    left: DistanceAttentionConfig
    right_width: int  # channels of the gated recurrence
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "ParallelConfig":
        left = DistanceAttentionConfig.from_dict(where + ".left", _object(where + ".left", data.get("left")))
        return cls(left, _positive(where + ".right", data.get("right"), "width"), _number(where, data, "left_scale"),
                   _number(where, data, "right_scale"))

    def to_dict(self) -> dict[str, Any]:
        return {"left": self.left.to_dict(), "right": {"width": self.right_width}, "left_scale": self.left_scale,
                "right_scale": self.right_scale}


@dataclass(frozen=True)
class WkvConfig:
    heads: int
    dim: int  # key and value channels of a head
    rank: int = 0  # inner size of the decay's two small matrices

    @classmethod
    def from_dict(cls, where: str, data: Mapping[str, Any]) -> "WkvConfig":
        return cls(_positive(where, data, "heads"), _positive(where, data, "dim"), _rank(where, data, "rank"))

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"heads": self.heads, "dim": self.dim}
        if self.rank:
            out["rank"] = self.rank
        return out


_MIXER_CONFIGS = {"channel_delta": ChannelDeltaConfig, "parallel": ParallelConfig, "wkv": WkvConfig}


@dataclass(frozen=True)
class PefulornLayerConfig:
    type: str  # one of MIXER_TYPES
    mixer: ChannelDeltaConfig | ParallelConfig | WkvConfig
    ff: int  # hidden units of the dense feed-forward; 0: the layer has none

    def to_dict(self) -> dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(),
                "mlp": {"kind": "dense", "ff": self.ff} if self.ff else None}


@dataclass(frozen=True)
class PefulornConfig:
    architecture: str
    width: int
    vocab: int
    norm_eps: float
    layers: tuple[PefulornLayerConfig, ...]
    # layers loop_start .. loop_stop - 1 run loop_times times in a row; 0 times: no loop
    loop_start: int
    loop_stop: int
    loop_times: int
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
    def from_dict(cls, data: Mapping[str, Any], overrides: Mapping[str, Any] | None = None) -> "PefulornConfig":
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
            mixer = entry.get("mixer")
            if not isinstance(mixer, Mapping):
                raise ConfigError(f"{where}: 'mixer' must give the mixer's sizes")
            mlp, ff = entry.get("mlp"), 0
            if mlp is not None:
                if _object(where + ".mlp", mlp).get("kind", "dense") != "dense":
                    raise ConfigError(f"{where}.mlp: feed-forward kind {mlp.get('kind')!r} is not known (only 'dense')")
                ff = _positive(where + ".mlp", mlp, "ff")
            layers.append(PefulornLayerConfig(kind, _MIXER_CONFIGS[kind].from_dict(where + ".mixer", mixer), ff))
        loop = data.get("loop")
        start = stop = times = 0
        if loop is not None:
            start, stop, times = (require(_object("loop", loop), k, int) for k in ("start", "stop", "times"))
            if times < 1 or not 0 <= start < stop <= len(layers):
                raise ConfigError(f"loop over layers {start}..{stop} x {times} does not fit {len(layers)} layers")
        eps = require(data.get("norm") or {}, "eps", float)
        if not eps > 0:
            raise ConfigError(f"norm.eps must be positive, got {eps!r}")
        eos = data.get("eos_token_id")
        eos_ids = () if eos is None else ((int(eos),) if isinstance(eos, int) else tuple(int(e) for e in eos))
        return cls(
            architecture=require(data, "architecture", str),
            width=_positive("config.json", data, "width"),
            vocab=_positive("config.json", data, "vocab"),
            norm_eps=eps,
            layers=tuple(layers),
            loop_start=start, loop_stop=stop, loop_times=times,
            torch_dtype=normalise_dtype_name(data.get("torch_dtype") or data.get("dtype") or "bfloat16"),
            eos_token_ids=eos_ids,
        )

    def run_order(self) -> tuple[int, ...]:
        """Layer indices in the order they run: the looped span repeated in place."""
        n = len(self.layers)
        if not self.loop_times:
            return tuple(range(n))
        span = tuple(range(self.loop_start, self.loop_stop))
        return tuple(range(self.loop_start)) + span * self.loop_times + tuple(range(self.loop_stop, n))

    def pass_places(self) -> tuple[int, ...]:
        """Places in the run order at which a pass of the loop begins, one per pass."""
        span = self.loop_stop - self.loop_start
        return tuple(self.loop_start + t * span for t in range(self.loop_times))

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "architecture": self.architecture,
            "width": self.width,
            "vocab": self.vocab,
            "norm": {"eps": self.norm_eps},
            "layers": [layer.to_dict() for layer in self.layers],
            "torch_dtype": self.torch_dtype,
        }
        if self.loop_times:
            out["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out
