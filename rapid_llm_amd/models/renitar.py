"""Renitar decoder: configuration -> model description, and its registry entry.

Layer ``i``'s tensors are ``l<i>.norm1``, ``l<i>.mix.*`` (``l<i>.mix.left.*`` and ``l<i>.mix.right.*`` for two
mixers side by side) and ``l<i>.mlp.*`` (experts ``e<n>.up`` / ``e<n>.down``, ``shared.*``, ``router``, ``correction``);
the two ends are ``embed``, ``final.norm`` and ``head``.  A bias is its projection's name with ``.b`` added, a
convolution's taps with ``.conv``.
"""

from __future__ import annotations

from ..config.registry import register_architecture
from ..config.renitar import GlaConfig, ParallelConfig, RenitarConfig
from .spec import LayerSpec, ModelSpec, PartSpec, linear_output, token_embedding

# what the design fixes
OUTPUT_SHARE = 0.5  # of each of two mixers side by side, behind its norm


def build_renitar_spec(cfg: RenitarConfig) -> ModelSpec:
    def norm(name: str) -> PartSpec:
        return PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.norm_eps, "checkpoint_name": name,
                                    "weight_offset": 1.0})

    layers = []
    for i, layer in enumerate(cfg.layers):
        prefix = f"l{i}."
        mix = prefix + "mix."
        m = layer.mixer
        position = PartSpec("none")
        if isinstance(m, GlaConfig):
            mixer = PartSpec(
                "linear_attention",
                {
                    "hidden_size": cfg.width, "num_heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim,
                    "query_scale": m.dim**-0.5, "decay": "channel", "tau": m.tau, "decay_rank": m.rank, "norm": "head",
                    "gate": "silu", "norm_eps": cfg.norm_eps, "checkpoint_prefix": mix,
                },
            )
        elif isinstance(m, ParallelConfig):
            a, r = m.left, m.right
            left = PartSpec(
                "gqa_attention",
                {
                    "hidden_size": cfg.width, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim,
                    "value_dim": a.vdim, "softmax_scale": a.scale, "score_cap": a.softcap, "window": a.chunk,
                    "chunked": True, "conv_taps": a.conv, "qk_norm_eps": cfg.norm_eps, "qk_norm_scope": "projection",
                    "gate_name": "g", "qkv_bias": True, "o_bias": True,
                    "bias_names": {"q": "q.b", "k": "k.b", "v": "v.b", "o": "o.b"}, "checkpoint_prefix": mix + "left.",
                    "q_name": "q", "k_name": "k", "v_name": "v", "o_name": "o", "q_norm_name": "q.norm",
                    "k_norm_name": "k.norm",
                },
            )
            right = PartSpec(
                "linear_attention",
                {
                    "hidden_size": cfg.width, "num_heads": r.heads, "key_dim": r.dim, "value_dim": r.vdim, "silu": True,
                    "decay": "fixed", "decays": r.decay, "norm": "row", "gate": "sigmoid", "norm_eps": cfg.norm_eps,
                    "checkpoint_prefix": mix + "right.",
                },
            )
            mixer = PartSpec(
                "side_by_side",
                {
                    "hidden_size": cfg.width, "left": left, "right": right, "left_scale": OUTPUT_SHARE,
                    "right_scale": OUTPUT_SHARE, "out_norm_names": (mix + "left.out", mix + "right.out"),
                    "out_norm_eps": cfg.norm_eps,
                },
            )
            position = PartSpec("rope", {"head_dim": a.dim, "theta": a.rot_base, "rotary_dim": a.rot_dims})
        else:  # pragma: no cover  (the configuration class admits no other)
            raise ValueError(f"layer {i}: no mixer for {type(m).__name__}")
        ff = None
        if layer.mlp is not None:
            f = layer.mlp
            ff = PartSpec(
                "routed_experts",
                {
                    "hidden_size": cfg.width, "num_experts": f.experts, "top": f.top, "expert_size": f.expert_ff,
                    "activation": "gelu", "route_scale": f.scale, "scores": "softmax_raw", "identity": f.identity,
                    "correction_name": "correction", "shared_size": f.shared_ff,
                    "shared_gate_name": "shared.sg" if f.shared_ff else None, "checkpoint_prefix": prefix + "mlp.",
                },
            )
        layers.append(
            LayerSpec(mixer=mixer, feed_forward=ff, mixer_norm=norm(prefix + "norm1"), feed_forward_norm=None,
                      block=PartSpec("shared_norm", {"factor": cfg.residual_mult}), position=position, shared_norm=True,
                      checkpoint_prefix=prefix)
        )
    return ModelSpec(
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        layers=tuple(layers),
        final_norm=norm("final.norm"),
        embedding=token_embedding(cfg.vocab, cfg.width, "embed"),
        output=linear_output(cfg.vocab, cfg.width, "head", tied=False),
    )


register_architecture("Renitar", RenitarConfig, build_renitar_spec, aliases=("renitar",), replace=True)
