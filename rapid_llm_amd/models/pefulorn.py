"""Pefulorn decoder: configuration -> model description, and its registry entry.

Layer ``i``'s tensors are ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*`` (``l<i>.mix.left.*`` and
``l<i>.mix.right.*`` for two mixers side by side) and ``l<i>.mlp.*``; the two ends are ``embed``,
``final.norm`` and ``head``; ``loop.step`` holds one vector per pass of the looped span.  A bias is its
projection's name with ``.b`` added.
"""

from __future__ import annotations

from ..config.pefulorn import ChannelDeltaConfig, ParallelConfig, PefulornConfig, WkvConfig
from ..config.registry import register_architecture
from .spec import IgnoreRule, LayerSpec, ModelSpec, PartSpec, StreamOffsets, StreamReturns, linear_output, token_embedding


def build_pefulorn_spec(cfg: PefulornConfig) -> ModelSpec:
    def norm(name: str) -> PartSpec:
        return PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.norm_eps, "checkpoint_name": name,
                                    "weight_offset": 1.0})

    layers, unread = [], []
    for i, layer in enumerate(cfg.layers):
        prefix = f"l{i}."
        mix = prefix + "mix."
        m = layer.mixer
        if isinstance(m, ChannelDeltaConfig):
            mixer = PartSpec(
                "delta_rule",
                {
                    "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "key_dim": m.dim,
                    "value_dim": m.vdim, "conv_taps": m.conv, "norm_eps": cfg.norm_eps, "decay_rank": m.decay_rank,
                    "gate_rank": m.gate_rank, "checkpoint_prefix": mix,
                },
            )
        elif isinstance(m, ParallelConfig):
            a = m.left
            left = PartSpec(
                "gqa_attention",
                {
                    "hidden_size": cfg.width, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim,
                    "value_dim": a.vdim, "softmax_scale": a.scale, "qk_norm_eps": cfg.norm_eps, "value_norm": True,
                    "query_temperature": (a.temp_coef, a.temp_every) if a.temp_coef else None,
                    "log_distance_names": ("r1", "r2"), "qkv_bias": True,
                    "bias_names": {"q": "q.b", "k": "k.b", "v": "v.b"}, "checkpoint_prefix": mix + "left.",
                    "q_name": "q", "k_name": "k", "v_name": "v", "o_name": "o", "q_norm_name": "q.norm",
                    "k_norm_name": "k.norm",
                },
            )
            right = PartSpec(
                "min_gru",
                {"hidden_size": cfg.width, "width": m.right_width, "checkpoint_prefix": mix + "right."},
            )
            mixer = PartSpec(
                "side_by_side",
                {"hidden_size": cfg.width, "left": left, "right": right, "left_scale": m.left_scale,
                 "right_scale": m.right_scale},
            )
        elif isinstance(m, WkvConfig):
            mixer = PartSpec(
                "wkv",
                {
                    "hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim, "decay_rank": m.rank,
                    "norm_eps": cfg.norm_eps, "checkpoint_prefix": mix,
                },
            )
        else:  # pragma: no cover  (the configuration class admits no other)
            raise ValueError(f"layer {i}: no mixer for {type(m).__name__}")
        ff = ff_norm = None
        if layer.ff:
            ff = PartSpec(
                "gated",
                {
                    "hidden_size": cfg.width, "intermediate_size": layer.ff, "activation": "gelu_tanh", "bias": True,
                    "checkpoint_prefix": prefix + "mlp.", "gate_name": "gate", "up_name": "up", "down_name": "down",
                },
            )
            ff_norm = norm(prefix + "norm2")
        else:
            unread.append(IgnoreRule(rf"l{i}\.norm2"))  # a norm that nothing stands behind
        layers.append(
            LayerSpec(mixer=mixer, feed_forward=ff, mixer_norm=norm(prefix + "norm1"), feed_forward_norm=ff_norm,
                      checkpoint_prefix=prefix)
        )
    places = cfg.pass_places()
    return ModelSpec(
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        layers=tuple(layers),
        final_norm=norm("final.norm"),
        embedding=token_embedding(cfg.vocab, cfg.width, "embed"),
        output=linear_output(cfg.vocab, cfg.width, "head", tied=False),
        run_order=cfg.run_order(),
        ignore_tensors=tuple(unread),
        stream_offsets=StreamOffsets("loop.step", places) if places else None,
        # every pass but the first begins with the embedding's output added to the stream
        stream_returns=StreamReturns(places[1:]) if places[1:] else None,
    )


register_architecture("Pefulorn", PefulornConfig, build_pefulorn_spec, aliases=("pefulorn",), replace=True)
