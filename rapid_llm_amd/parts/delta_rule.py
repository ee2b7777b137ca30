"""Gated delta rule with a decay per key channel, as a mixer with a fixed-size state per request.

``q``, ``k`` (``kv_heads x key_dim``) and ``v`` (``heads x value_dim``) are projections that pass a short causal
convolution per channel (``taps`` taps, the last one meeting the current token, zeros before a
request's start, no bias) and silu; ``q`` and ``k`` are then unit vectors per head, ``q`` times
``key_dim^(-1/2)``; head h reads q and k of head ``h // (heads / kv_heads)``.  With ``beta = sigmoid(W_b h)`` and
the decays ``g = exp(-exp(A_log_h) softplus(W_a2 (W_a1 h) + dt_bias))`` (heads x key_dim), per head with the
state ``S [key channel, value channel]``::

    S <- diag(g) S        u = beta (v - S^T k)        S <- S + k u^T        o = S^T q

Each head's ``o`` is divided by its root mean square, multiplied by a weight that the heads share and by
``sigmoid(W_g2 (W_g1 h))``, and the output projection follows.

Everything that reads ``h`` is one packed product, ``[q | k | v | g1]`` with a result in the compute type and
``[b | a1]`` with a float32 one; ``W_a2`` is held in float32.  The convolution's sums, unit norms, softplus, exponentials, the state and the head norm are float32
(``csrc/recurrent.hip``).  The state and the convolutions' last ``taps - 1`` inputs live in the request's
slot (``cache.states``).
"""

from __future__ import annotations

import torch

from ..kernels import ops
from .base import MIXERS, CacheNeed, Mixer, ParamSpec, Source, StateSpec
from .linear import Linear


class DeltaRule(Mixer):
    replayable = True

    def __init__(
        self,
        hidden_size: int,
        num_heads: int,
        num_kv_heads: int,
        key_dim: int,
        value_dim: int,
        conv_taps: int,
        norm_eps: float,
        checkpoint_prefix: str,
        decay_rank: int = 0,  # 0: the size the checkpoint's tensors have
        gate_rank: int = 0,
        position=None,  # the recurrence knows order by itself
        name: str = "mixer",
        q_name: str = "q",
        k_name: str = "k",
        v_name: str = "v",
        conv_suffix: str = ".conv",
        beta_name: str = "b",
        decay_log_name: str = "A_log",
        decay_in_name: str = "a1",
        decay_out_name: str = "a2",
        decay_bias_name: str = "dt_bias",
        gate_in_name: str = "g1",
        gate_out_name: str = "g2",
        norm_name: str = "norm",
        o_name: str = "o",
    ) -> None:
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} heads are not divisible by {num_kv_heads} kv heads")
        if not 1 <= key_dim <= ops.DELTA_MAX_HEAD_DIM or not 1 <= value_dim <= ops.DELTA_MAX_HEAD_DIM:
            raise ValueError(
                f"the recurrence's kernel takes heads of up to {ops.DELTA_MAX_HEAD_DIM} channels, got {key_dim} and {value_dim}"
            )
        if not 1 <= conv_taps <= ops.CONV_MAX_TAPS:
            raise ValueError(f"the convolution's kernel takes up to {ops.CONV_MAX_TAPS} taps, got {conv_taps}")
        self.hidden_size, self.heads, self.kv_heads = hidden_size, num_heads, num_kv_heads
        self.d, self.dv, self.taps, self.eps = key_dim, value_dim, conv_taps, float(norm_eps)
        self.decay_rank, self.gate_rank = int(decay_rank) or -1, int(gate_rank) or -1
        self.prefix, self.name = checkpoint_prefix, name
        self.names = dict(q=q_name, k=k_name, v=v_name, b=beta_name, a_log=decay_log_name, a1=decay_in_name,
                          a2=decay_out_name, dt_bias=decay_bias_name, g1=gate_in_name, g2=gate_out_name,
                          norm=norm_name, o=o_name)
        self.conv_suffix = conv_suffix
        self.inner = num_heads * value_dim
        self.channels = 2 * num_kv_heads * key_dim + self.inner  # what the convolutions mix
        self.in_proj = None  # sized when the tensors are bound
        self.o = Linear(self.inner, hidden_size)

    # ---- tensors ---------------------------------------------------------------
    def _sources(self, suffix: str = "") -> tuple[Source, ...]:
        p, n, kv = self.prefix, self.names, self.kv_heads * self.d
        return tuple(Source(p + n[s] + suffix, rows) for s, rows in (("q", kv), ("k", kv), ("v", self.inner)))

    def param_specs(self) -> list[ParamSpec]:
        p, n, h = self.prefix, self.names, self.hidden_size
        keys = self.heads * self.d

        def one(name: str, shape: tuple[int, ...], role: str, source: str, **more) -> ParamSpec:
            return ParamSpec(f"{self.name}.{name}", shape, role, (Source(p + n[source], max(shape[0], 0)),), **more)

        return [
            ParamSpec(self.name + ".qkv", (self.channels, h), "matrix", self._sources()),
            ParamSpec(self.name + ".conv", (self.channels, self.taps), "vector", self._sources(self.conv_suffix)),
            one("beta", (self.heads, h), "matrix", "b"),
            one("decay_in", (self.decay_rank, h), "matrix", "a1"),
            one("decay_out", (keys, self.decay_rank), "matrix_f32", "a2"),
            one("decay_bias", (keys,), "vector", "dt_bias"),
            one("decay_log", (self.heads,), "vector", "a_log"),
            one("gate_in", (self.gate_rank, h), "matrix", "g1"),
            one("gate_out", (self.inner, self.gate_rank), "matrix", "g2"),
            one("norm", (self.dv,), "vector", "norm", init="norm"),
            one("o", (h, self.inner), "matrix", "o"),
        ]

    def bind(self, params, runtime) -> None:
        def get(which: str) -> torch.Tensor:
            return params[f"{self.name}.{which}"]

        a1, a2, g1, g2 = get("decay_in"), get("decay_out"), get("gate_in"), get("gate_out")
        for first, second, what in ((a1, a2, "decay"), (g1, g2, "gate")):
            if first.shape[0] != second.shape[1]:
                raise ValueError(f"the {what}'s two matrices do not meet: {tuple(first.shape)} and {tuple(second.shape)}")
        # The rows of the packed product.  The compute-type part is padded so that both parts are whole
        # groups of eight rows and the gate's columns begin at one.
        qkv, beta = get("qkv"), get("beta")
        pads = (-self.channels % 8, -g1.shape[0] % 8)
        self.gate_col = self.channels + pads[0]
        self.split = self.gate_col + g1.shape[0] + pads[1]
        kept = torch.float32 if any(t.dtype == torch.float32 for t in (qkv, beta, a1, g1)) else qkv.dtype
        rows = [qkv, qkv.new_zeros(pads[0], self.hidden_size), g1, qkv.new_zeros(pads[1], self.hidden_size), beta, a1]
        packed = torch.cat([t.to(kept) for t in rows])
        self.in_proj = Linear(self.hidden_size, packed.shape[0])
        self.in_proj.bind(packed)
        # whoever holds the loaded tensors holds these rows from now on, not a second copy
        at = 0
        for which, t in zip(("qkv", None, "gate_in", None, "beta", "decay_in"), rows):
            if which is not None:
                params[f"{self.name}.{which}"] = packed[at : at + t.shape[0]]
            at += t.shape[0]
        self.decay_out = a2
        self.gate_out = Linear(g1.shape[0], self.inner)
        self.gate_out.bind(g2)
        self.conv, self.decay_bias, self.decay_log = get("conv"), get("decay_bias"), get("decay_log")
        self.norm_weight = get("norm")
        self.o.bind(get("o"))

    # ---- cache -----------------------------------------------------------------
    def cache_need(self) -> CacheNeed:
        return CacheNeed(
            "state",
            states=(
                StateSpec("conv", (max(self.taps - 1, 1), self.channels), "float32"),
                StateSpec("S", (self.heads, self.dv, self.d), "float32"),  # [value channel, key channel]
            ),
        )

    # ---- step ------------------------------------------------------------------
    @property
    def accepts_scaled_rows(self) -> bool:
        return self.in_proj.takes_scaled_rows()

    def forward(self, x, ctx, cache):
        tokens, device = x.shape[0], x.device
        packed, low = self.in_proj.split(x, self.split)
        decay = torch.empty((tokens, self.heads * self.d), dtype=torch.float32, device=device)
        ops.gemm_f32(low[:, self.heads :], self.decay_out, decay)
        gate = self.gate_out(packed[:, self.gate_col : self.gate_col + self.gate_out.in_features])
        mixed = torch.empty((tokens, self.channels), dtype=torch.float32, device=device)
        ops.delta_prepare(packed, 0, self.conv, cache.states["conv"], decay, self.decay_bias, self.decay_log, mixed, ctx,
                          self.heads, self.kv_heads, self.d, self.dv)
        raw = torch.empty((tokens, self.inner), dtype=torch.float32, device=device)
        ops.delta_scan(mixed, decay, low, raw, ctx, cache.states["S"], self.heads, self.kv_heads, self.d, self.dv)
        out = torch.empty((tokens, self.inner), dtype=packed.dtype, device=device)
        ops.head_finish(raw, gate, self.norm_weight, out, self.heads, self.eps, "sigmoid")
        return self.o.deferred(out, ctx)


MIXERS.register("delta_rule", DeltaRule)
