"""A gated recurrence whose gates read only the current token (minGRU), as a mixer with one number of
state per channel.

``z = sigmoid(W_z h + b_z)`` and ``u = W_x h + b_x``, both of ``width`` channels; the candidate is ``u + 1/2``
where ``u >= 0`` and ``sigmoid(u)`` elsewhere.  Element by element ``S_t = (1 - z) S_(t-1) + z candidate``,
and the output is ``W_o (S_t * silu(W_g h))``.

The three projections run in the compute type as one packed product ``[z | x | g]``; biases, gates,
candidate, state and output gate are float32 (``csrc/recurrent.hip``).  The state lives in the
request's slot (``cache.states``).
"""

from __future__ import annotations

import torch

from ..kernels import ops
from .base import MIXERS, CacheNeed, PackedMixer, ParamSpec, Source, StateSpec
from .linear import Linear


class MinGRU(PackedMixer):
    replayable = True
    packs = True

    def __init__(
        self,
        hidden_size: int,
        width: int,
        checkpoint_prefix: str,
        position=None,  # the recurrence knows order by itself
        name: str = "mixer",
        z_name: str = "z",
        x_name: str = "x",
        gate_name: str = "g",
        o_name: str = "o",
        bias_suffix: str = ".b",
    ) -> None:
        if width < 1:
            raise ValueError(f"a recurrence of {width} channels")
        self.hidden_size, self.width = hidden_size, width
        self.prefix, self.name = checkpoint_prefix, name
        self.names = (z_name, x_name, gate_name)
        self.o_name, self.bias_suffix = o_name, bias_suffix
        self.packed_rows, self.inner_width = 3 * width, width
        self.in_proj = Linear(hidden_size, self.packed_rows)
        self.o = Linear(width, hidden_size)

    # ---- tensors ---------------------------------------------------------------
    def packed_sources(self) -> tuple[Source, ...]:
        return tuple(Source(self.prefix + n, self.width) for n in self.names)

    def output_source(self) -> str:
        return self.prefix + self.o_name

    def inner_specs(self) -> list[ParamSpec]:
        return [
            ParamSpec(f"{self.name}.{which}_bias", (self.width,), "vector",
                      (Source(self.prefix + source + self.bias_suffix, self.width),))
            for which, source in zip(("z", "x"), self.names)
        ]

    def param_specs(self) -> list[ParamSpec]:
        return [
            ParamSpec(self.name + ".in", (self.packed_rows, self.hidden_size), "matrix", self.packed_sources()),
            ParamSpec(self.name + ".o", (self.hidden_size, self.width), "matrix",
                      (Source(self.output_source(), self.hidden_size),)),
            *self.inner_specs(),
        ]

    def bind(self, params, runtime) -> None:
        self.in_proj.bind(params[self.name + ".in"])
        self.o.bind(params[self.name + ".o"])
        self.bind_inner(params, runtime)

    def bind_inner(self, params, runtime) -> None:
        self.z_bias, self.x_bias = params[self.name + ".z_bias"], params[self.name + ".x_bias"]

    # ---- cache -----------------------------------------------------------------
    def cache_need(self) -> CacheNeed:
        return CacheNeed("state", states=(StateSpec("S", (self.width,), "float32"),))

    # ---- step ------------------------------------------------------------------
    @property
    def accepts_scaled_rows(self) -> bool:
        return self.in_proj.takes_scaled_rows()

    def run(self, packed, col0, out, out_col, out_scale, ctx, cache):
        w = self.width
        ops.min_gru(packed, (col0, col0 + w, col0 + 2 * w), self.z_bias, self.x_bias, out, ctx, cache.states["S"],
                    out_col, out_scale)

    def forward(self, x, ctx, cache):
        packed = self.in_proj(x)
        out = torch.empty((x.shape[0], self.width), dtype=packed.dtype, device=packed.device)
        self.run(packed, 0, out, 0, 1.0, ctx, cache)
        return self.o.deferred(out, ctx)


MIXERS.register("min_gru", MinGRU)
