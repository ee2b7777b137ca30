"""Linear attention with decays, as a mixer with a fixed-size memory per request.

Per head, with the memory ``S [key channel, value channel]``::

    S_t = diag(a_t) S_(t-1) + k_t v_t^T          o_t = S_t^T q_t

``decay="channel"``: the decay is a number a key channel that depends on the token,
``a = sigmoid(z)^(1 / tau)`` with ``z = W_a2 (W_a1 h) + b`` (gated linear attention).  ``decay="fixed"``: one
given number a head (lightning attention).  ``silu``: q, k and v pass it; ``query_scale`` multiplies q.  The
outputs are divided by their root mean square per head (``norm="head"``, one weight for all heads) or over
all heads together (``norm="row"``), multiplied by ``silu`` or ``sigmoid`` of ``W_g h`` (``gate``), and the
output projection follows.

Everything that reads ``h`` is one packed product ``[q | k | v | g]``, with ``W_a1``'s columns behind it whose
float32 accumulation is kept; ``W_a2`` is held in float32 and applied inside the kernels that form the
decays.  Decays, memory, sums and norms are float32 (``csrc/linear_attention.hip``).  The memory lives in
the request's slot (``cache.states``).  With fixed decays the mixer runs on columns of a product that
another mixer shares (``packs``).
"""

from __future__ import annotations

import math
from typing import Sequence

import torch

from ..kernels import ops
from .base import MIXERS, CacheNeed, PackedMixer, ParamSpec, Source, StateSpec
from .linear import Linear


class LinearAttention(PackedMixer):
    replayable = True

    def __init__(
        self,
        hidden_size: int,
        num_heads: int,
        key_dim: int,
        value_dim: int,
        norm_eps: float,
        checkpoint_prefix: str,
        decay: str,
        norm: str,
        gate: str,
        silu: bool = False,
        query_scale: float = 1.0,
        tau: float = 1.0,
        decay_rank: int = 0,  # decay="channel"; 0: the size the checkpoint's tensors have
        decays: Sequence[float] = (),  # decay="fixed": one a head
        position=None,  # the recurrence knows order by itself
        name: str = "mixer",
        q_name: str = "q",
        k_name: str = "k",
        v_name: str = "v",
        gate_name: str = "g",
        o_name: str = "o",
        norm_name: str = "norm",
        decay_in_name: str = "a1",
        decay_out_name: str = "a2",
        decay_bias_name: str = "a2.b",
    ) -> None:
        if not 1 <= key_dim <= ops.LINEAR_MAX_KEY_DIM or not 1 <= value_dim <= ops.LINEAR_MAX_VALUE_DIM or num_heads < 1:
            raise ValueError(
                f"the kernels take heads of up to {ops.LINEAR_MAX_KEY_DIM} key and {ops.LINEAR_MAX_VALUE_DIM} value "
                f"channels, got {num_heads} heads of {key_dim} and {value_dim}"
            )
        if decay not in ("channel", "fixed"):
            raise ValueError(f"decays are one a 'channel' or 'fixed' ones a head, not {decay!r}")
        if norm not in ("head", "row") or gate not in ops.HEAD_GATES:
            raise ValueError(f"outputs are normed by 'head' or 'row' behind one of the gates {sorted(ops.HEAD_GATES)}, not {norm!r}, {gate!r}")
        if decay == "channel" and not tau > 0:
            raise ValueError(f"decays are taken to the power 1 / {tau}")
        if decay == "fixed" and (len(decays) != num_heads or not all(0 < a <= 1 for a in decays)):
            raise ValueError(f"fixed decays are one number in (0, 1] a head, got {list(decays)} for {num_heads} heads")
        self.hidden_size, self.heads, self.d, self.dv = hidden_size, num_heads, key_dim, value_dim
        self.eps, self.gate, self.silu, self.query_scale = float(norm_eps), gate, bool(silu), float(query_scale)
        self.channel_decay, self.tau, self.decays = decay == "channel", float(tau), tuple(float(a) for a in decays)
        self.rank = int(decay_rank) or -1
        self.prefix, self.name = checkpoint_prefix, name
        self.names = dict(q=q_name, k=k_name, v=v_name, g=gate_name, o=o_name, norm=norm_name, a1=decay_in_name,
                          a2=decay_out_name, a2b=decay_bias_name)
        self.packs = not self.channel_decay
        keys, inner = num_heads * key_dim, num_heads * value_dim
        self.inner_width = inner
        self.norm_parts = num_heads if norm == "head" else 1
        self.norm_size = value_dim if norm == "head" else inner
        self.columns = (0, keys, 2 * keys, 2 * keys + inner)  # of q, k, v and the gate
        self.packed_rows = 2 * keys + 2 * inner
        self.in_proj = Linear(hidden_size, self.packed_rows)  # (sized anew where decays ride along)
        self.o = Linear(inner, hidden_size)

    # ---- tensors ---------------------------------------------------------------
    def packed_sources(self) -> tuple[Source, ...]:
        keys, inner = self.heads * self.d, self.inner_width
        return tuple(Source(self.prefix + self.names[s], rows)
                     for s, rows in (("q", keys), ("k", keys), ("v", inner), ("g", inner)))

    def output_source(self) -> str:
        return self.prefix + self.names["o"]

    def inner_specs(self) -> list[ParamSpec]:
        p, n = self.prefix, self.names
        specs = [ParamSpec(self.name + ".norm", (self.norm_size,), "vector", (Source(p + n["norm"], self.norm_size),), init="norm")]
        if self.channel_decay:
            keys = self.heads * self.d
            specs += [
                ParamSpec(self.name + ".decay_in", (self.rank, self.hidden_size), "matrix", (Source(p + n["a1"], max(self.rank, 0)),)),
                ParamSpec(self.name + ".decay_out", (keys, self.rank), "matrix_f32", (Source(p + n["a2"], keys),)),
                ParamSpec(self.name + ".decay_bias", (keys,), "vector", (Source(p + n["a2b"], keys),)),
            ]
        return specs

    def param_specs(self) -> list[ParamSpec]:
        return [
            ParamSpec(self.name + ".in", (self.packed_rows, self.hidden_size), "matrix", self.packed_sources()),
            ParamSpec(self.name + ".o", (self.hidden_size, self.inner_width), "matrix",
                      (Source(self.output_source(), self.hidden_size),)),
            *self.inner_specs(),
        ]

    def bind(self, params, runtime) -> None:
        packed = params[self.name + ".in"]
        if self.channel_decay:
            # the decays' first matrix is the last rows of the packed product, from a multiple of 8 on
            a1 = params[self.name + ".decay_in"]
            pad = -self.packed_rows % 8
            self.split = self.packed_rows + pad
            kept = torch.float32 if torch.float32 in (packed.dtype, a1.dtype) else packed.dtype
            rows = [packed, packed.new_zeros(pad, self.hidden_size), a1]
            packed = torch.cat([t.to(kept) for t in rows])
            # whoever holds the loaded tensors holds these rows from now on, not a second copy
            params[self.name + ".in"] = packed[: self.packed_rows]
            params[self.name + ".decay_in"] = packed[self.split :]
            self.in_proj = Linear(self.hidden_size, packed.shape[0])
        self.in_proj.bind(packed)
        self.o.bind(params[self.name + ".o"])
        self.bind_inner(params, runtime)

    def bind_inner(self, params, runtime) -> None:
        self.norm_weight = params[self.name + ".norm"]
        if self.channel_decay:
            a1, a2 = params[self.name + ".decay_in"], params[self.name + ".decay_out"]
            if a1.shape[0] != a2.shape[1]:
                raise ValueError(f"the decay's two matrices do not meet: {tuple(a1.shape)} and {tuple(a2.shape)}")
            self.decay_out_t = a2.t().contiguous()
            self.decay_bias = params[self.name + ".decay_bias"]
        else:
            self.fixed = ops.FixedDecay(torch.tensor([math.log(a) for a in self.decays], dtype=torch.float32, device=runtime.device))

    # ---- cache -----------------------------------------------------------------
    def cache_need(self) -> CacheNeed:
        return CacheNeed("state", states=(StateSpec("S", (self.heads, self.d, self.dv), "float32"),))

    # ---- step ------------------------------------------------------------------
    @property
    def accepts_scaled_rows(self) -> bool:
        return self.in_proj.takes_scaled_rows()

    def _mix(self, packed, col0, decay, out, out_col, ctx, cache):
        ops.linear_attention(packed, tuple(col0 + c for c in self.columns), decay, self.norm_weight, out, ctx,
                             cache.states["S"], self.heads, self.d, self.dv, self.query_scale, self.silu, self.norm_parts,
                             self.gate, self.eps, out_col)

    def run(self, packed, col0, out, out_col, out_scale, ctx, cache):
        if out_scale != 1.0:
            raise ValueError("the outputs of linear attention are not scaled: scale what reads them")
        self._mix(packed, col0, self.fixed, out, out_col, ctx, cache)

    def forward(self, x, ctx, cache):
        if self.channel_decay:
            packed, low = self.in_proj.split(x, self.split)
            decay = ops.ChannelDecay(low, self.decay_out_t, self.decay_bias, self.tau)
        else:
            packed, decay = self.in_proj(x), self.fixed
        out = torch.empty((x.shape[0], self.inner_width), dtype=packed.dtype, device=packed.device)
        self._mix(packed, 0, decay, out, 0, ctx, cache)
        return self.o.deferred(out, ctx)


MIXERS.register("linear_attention", LinearAttention)
