"""Two mixers side by side on one input: ``left_scale * left(h) + right_scale * right(h)``.

Both are :class:`~rapid_llm_amd.parts.base.PackedMixer` s, so the pair costs what one mixer does in
products: their input projections are the rows of one packed matrix, their output projections lie
side by side in another, applied to the concatenation of what the two leave, each multiplied by its
scale in the kernel that finishes it.  With ``out_norm_names`` each output is divided by its root mean square
over the model width and multiplied by a weight of that name before it is scaled and added: the two
output projections are then products of their own, and what they return travels on as a
:class:`~rapid_llm_amd.parts.lazy.LayerSum`.  The cache holds what both ask for (the pages of one of them;
the states of both, told apart by a prefix).
"""

from __future__ import annotations

from dataclasses import replace

import torch

from .base import MIXERS, CacheNeed, Mixer, ParamSpec, Source
from .lazy import DeferredProduct, LayerSum
from .linear import Linear

SIDES = ("left", "right")


class SideBySide(Mixer):
    replayable = True

    def __init__(self, hidden_size: int, left, right, left_scale: float, right_scale: float, position=None,
                 name: str = "mixer", out_norm_names: tuple[str, str] | None = None, out_norm_eps: float = 0.0) -> None:
        self.hidden_size, self.name = hidden_size, name
        self.mixers = tuple(
            MIXERS.create(spec.kind, **spec.params, position=position, name=f"{name}.{side}")
            for side, spec in zip(SIDES, (left, right))
        )
        self.scales = (float(left_scale), float(right_scale))
        self.out_norm_names, self.out_norm_eps = out_norm_names, float(out_norm_eps)
        if out_norm_names is not None and not self.out_norm_eps > 0:
            raise ValueError(f"normed outputs need a positive epsilon, got {out_norm_eps}")
        for side, mixer in zip(SIDES, self.mixers):
            if not getattr(mixer, "packs", False):
                raise ValueError(f"the {side} mixer, {type(mixer).__name__}, does not run on columns of a shared product")
            if out_norm_names is None and getattr(mixer, "o_bias", False):
                raise ValueError(f"the {side} mixer's output projection has a bias, which a shared product has no place for")
            if mixer.hidden_size != hidden_size:
                raise ValueError(f"the {side} mixer reads rows of {mixer.hidden_size}, not of {hidden_size}")
        # every mixer's columns begin at a multiple of 8
        self.pads = tuple(-m.packed_rows % 8 for m in self.mixers)
        self.columns = (0, self.mixers[0].packed_rows + self.pads[0])
        self.inner_width = sum(m.inner_width for m in self.mixers)
        self.in_proj = Linear(hidden_size, sum(m.packed_rows for m in self.mixers) + sum(self.pads))
        self.o = Linear(self.inner_width, hidden_size)

    # ---- tensors ---------------------------------------------------------------
    def param_specs(self) -> list[ParamSpec]:
        packed: list[Source] = []
        for mixer, pad in zip(self.mixers, self.pads):
            packed += mixer.packed_sources()
            if pad:
                packed.append(Source("", pad))  # rows of zeros
        specs = [
            ParamSpec(self.name + ".in", (self.in_proj.out_features, self.hidden_size), "matrix", tuple(packed)),
        ]
        h = self.hidden_size
        if self.out_norm_names is None:
            specs.append(ParamSpec(self.name + ".o", (h, self.inner_width), "matrix",
                                   tuple(Source(m.output_source(), m.inner_width) for m in self.mixers), axis=1))
        else:
            for side, m, norm in zip(SIDES, self.mixers, self.out_norm_names):
                specs += [
                    ParamSpec(f"{self.name}.{side}.o", (h, m.inner_width), "matrix", (Source(m.output_source(), h),)),
                    ParamSpec(f"{self.name}.{side}.out_norm", (h,), "vector", (Source(norm, h),), init="norm"),
                ]
        for mixer in self.mixers:
            specs += mixer.inner_specs()
        return specs

    def bind(self, params, runtime) -> None:
        self.in_proj.bind(params[self.name + ".in"])
        if self.out_norm_names is None:
            self.o.bind(params[self.name + ".o"])
        else:
            self.outs, self.out_weights = [], []
            for side, m, scale in zip(SIDES, self.mixers, self.scales):
                o = Linear(m.inner_width, self.hidden_size)
                o.bind(params[f"{self.name}.{side}.o"], params[f"{m.name}.o_bias"] if getattr(m, "o_bias", False) else None)
                self.outs.append(o)
                self.out_weights.append(params[f"{self.name}.{side}.out_norm"] * scale)  # behind the norm: it commutes
        for mixer in self.mixers:
            mixer.bind_inner(params, runtime)

    # ---- cache -----------------------------------------------------------------
    def cache_need(self) -> CacheNeed:
        needs = [m.cache_need() for m in self.mixers]
        paged = [n for n in needs if n.kind == "paged"]
        if len(paged) > 1:
            raise ValueError("two mixers side by side both ask for pages")
        states = tuple(
            replace(spec, name=f"{side}.{spec.name}")
            for side, need in zip(SIDES, needs)
            for spec in need.state_specs()
        )
        if paged:
            return replace(paged[0], states=states, state_shape=None, state_dtype=None)  # (all else as that mixer asks)
        return CacheNeed("state" if states else "none", states=states)

    def _cache_of(self, side: str, cache):
        """What one of the two sees of the cache: the pages, and its own states under its own names."""
        prefix = side + "."
        return replace(cache, states={k[len(prefix):]: t for k, t in cache.states.items() if k.startswith(prefix)})

    def recorded_step_bytes(self, rows: int, context_bound: int, page_size: int) -> int:
        return sum(m.recorded_step_bytes(rows, context_bound, page_size) for m in self.mixers)

    # ---- step ------------------------------------------------------------------
    @property
    def accepts_scaled_rows(self) -> bool:
        return self.in_proj.takes_scaled_rows()

    def forward(self, x, ctx, cache):
        packed = self.in_proj(x)
        if self.out_norm_names is not None:
            terms = []
            for side, mixer, col0, o, weight in zip(SIDES, self.mixers, self.columns, self.outs, self.out_weights):
                y = torch.empty((x.shape[0], mixer.inner_width), dtype=packed.dtype, device=packed.device)
                mixer.run(packed, col0, y, 0, 1.0, ctx, self._cache_of(side, cache))
                terms.append(DeferredProduct(o, y).term(weight))
            return LayerSum(terms, eps=self.out_norm_eps)
        both = torch.empty((x.shape[0], self.inner_width), dtype=packed.dtype, device=packed.device)
        out_col = 0
        for side, mixer, col0, scale in zip(SIDES, self.mixers, self.columns, self.scales):
            mixer.run(packed, col0, both, out_col, scale, ctx, self._cache_of(side, cache))
            out_col += mixer.inner_width
        return self.o.deferred(both, ctx)


MIXERS.register("side_by_side", SideBySide)
