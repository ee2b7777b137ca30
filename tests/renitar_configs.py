"""Small Renitar configurations that differ in every size and option, and random weights for
them, made here tensor by tensor (names and shapes written out once more, independent of the
package's own list of parameters)."""

from __future__ import annotations

import json
import random
from pathlib import Path

import torch


def _gla(heads, dim, vdim, tau, rank):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "rank": rank}


def _pair(heads, kv_heads, dim, vdim, conv, scale, softcap, chunk, rot_dims, base, right_heads, right_dim, right_vdim, decay):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale, "softcap": softcap,
            "mask": {"size": chunk}, "rot": {"dims": rot_dims, "base": base}}
    return {"left": left, "right": {"heads": right_heads, "dim": right_dim, "vdim": right_vdim, "decay": decay}}


def _layer(kind, mixer, mlp=None):
    """``mlp``: units of an expert, experts, identity experts, chosen, scale, units of the shared expert."""
    if mlp is not None:
        ff, experts, identity, top, scale, shared = mlp
        mlp = {"kind": "moe", "expert": {"ff": ff},
               "router": {"experts": experts, "identity": identity, "top": top, "scale": scale}, "shared": {"ff": shared}}
    return {"type": kind, "mixer": mixer, "mlp": mlp}


# A: both mixers in turn, values wider and narrower than keys, three taps, chunks of 20 positions on pages
# of 8, a layer without a feed-forward, more identity experts than a token uses
RENI_A = {
    "architecture": "Renitar", "width": 96, "vocab": 211, "norm": {"eps": 3e-6}, "residual_mult": 0.8,
    "layers": [
        _layer("parallel", _pair(4, 2, 16, 32, 3, 0.3, 6.0, 20, 8, 1000.0, 3, 16, 24, [0.5, 0.9, 0.99]), (24, 6, 3, 2, 1.5, 40)),
        _layer("gla", _gla(3, 24, 16, 8.0, 5), (16, 5, 2, 3, 0.7, 24)),
        _layer("gla", _gla(2, 16, 48, 1.0, 12)),
        _layer("parallel", _pair(2, 1, 32, 16, 2, 0.2, 9.0, 7, 32, 50000.0, 4, 8, 12, [0.3, 0.7, 0.95, 1.0]), (20, 4, 1, 1, 1.0, 16)),
    ],
}
PAGE_A = 8

# B: the smallest of everything: one head, one channel, chunks of a single position, a convolution of a
# single tap, one expert that everybody uses and no identity expert, rank 1; pages of 4
RENI_B = {
    "architecture": "Renitar", "width": 64, "vocab": 130, "norm": {"eps": 1e-6}, "residual_mult": 1.0,
    "layers": [
        _layer("gla", _gla(1, 1, 1, 2.0, 1), (8, 1, 0, 1, 1.0, 8)),
        _layer("parallel", _pair(1, 1, 16, 16, 1, 0.25, 30.0, 1, 2, 10.0, 1, 1, 1, [0.8]), (16, 2, 1, 3, 1.0, 8)),
        _layer("gla", _gla(1, 16, 16, 16.0, 1), None),
    ],
}
PAGE_B = 4

# C: sizes that no vector access divides and that lie between the matrix cores' steps: heads of 12 and 10,
# linear attention of 20 and 13 channels, five taps, chunks of 33, experts of 9 units, width 100; pages of 8
RENI_C = {
    "architecture": "Renitar", "width": 100, "vocab": 97, "norm": {"eps": 1e-5}, "residual_mult": -0.6,
    "layers": [
        _layer("gla", _gla(5, 20, 13, 3.5, 7), (9, 7, 2, 4, 2.5, 11)),
        _layer("parallel", _pair(6, 3, 12, 10, 5, 0.35, 4.0, 33, 6, 300.0, 3, 9, 14, [0.2, 0.6, 0.97]), (13, 3, 4, 2, 1.2, 30)),
        _layer("parallel", _pair(3, 1, 22, 9, 4, 0.4, 15.0, 50, 22, 77.0, 2, 30, 7, [0.99, 0.01]), None),
    ],
}
PAGE_C = 8

# D: heads of the sizes real models have, with values narrower and wider: linear attention of 64 / 128 and 128 / 64
# channels, attention heads of 64 / 32 with eight query heads a kv head, seven taps, chunks of 48; pages of 16
RENI_D = {
    "architecture": "Renitar", "width": 128, "vocab": 300, "norm": {"eps": 2e-5}, "residual_mult": 0.7,
    "layers": [
        _layer("parallel", _pair(8, 1, 64, 32, 7, 0.11, 12.0, 48, 64, 20000.0, 2, 128, 64, [0.9, 0.999]), (64, 8, 2, 2, 1.8, 96)),
        _layer("gla", _gla(2, 64, 128, 16.0, 16), (32, 12, 6, 5, 2.2, 48)),
        _layer("gla", _gla(1, 160, 80, 5.0, 24), (48, 3, 1, 2, 0.9, 64)),
    ],
}
PAGE_D = 16

# E: linear attention alone, so that no request has pages; pages of 8 that nobody asks for
RENI_E = {
    "architecture": "Renitar", "width": 80, "vocab": 141, "norm": {"eps": 1e-5}, "residual_mult": 0.9,
    "layers": [
        _layer("gla", _gla(4, 48, 20, 4.0, 6), (24, 4, 2, 2, 1.1, 16)),
        _layer("gla", _gla(2, 32, 32, 12.0, 3), (16, 6, 1, 4, 0.8, 24)),
    ],
}
PAGE_E = 8

RENI = {"A": (RENI_A, PAGE_A, 801), "B": (RENI_B, PAGE_B, 802), "C": (RENI_C, PAGE_C, 803), "D": (RENI_D, PAGE_D, 804),
        "E": (RENI_E, PAGE_E, 805)}


def tensor_shapes(cfg) -> dict[str, tuple[int, ...]]:
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "head": (cfg["vocab"], w)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (w,)
        if layer["type"] == "gla":
            keys, values = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for s, rows in (("q", keys), ("k", keys), ("v", values), ("g", values)):
                out[p + "mix." + s] = (rows, w)
            out[p + "mix.o"] = (w, values)
            out[p + "mix.norm"] = (m["vdim"],)
            out[p + "mix.a1"] = (m["rank"], w)
            out[p + "mix.a2"] = (keys, m["rank"])
            out[p + "mix.a2.b"] = (keys,)
        else:
            a, r = m["left"], m["right"]
            for s, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                out[p + "mix.left." + s] = (rows, w)
                out[p + "mix.left." + s + ".b"] = (rows,)
                out[p + "mix.left." + s + ".conv"] = (rows, a["conv"])
                if s != "v":
                    out[p + "mix.left." + s + ".norm"] = (rows,)
            values = a["heads"] * a["vdim"]
            out[p + "mix.left.g"] = (values, w)
            out[p + "mix.left.o"] = (w, values)
            out[p + "mix.left.o.b"] = (w,)
            keys, values = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            for s, rows in (("q", keys), ("k", keys), ("v", values), ("g", values)):
                out[p + "mix.right." + s] = (rows, w)
            out[p + "mix.right.o"] = (w, values)
            out[p + "mix.right.norm"] = (values,)
            for side in ("left", "right"):
                out[p + f"mix.{side}.out"] = (w,)
        f = layer["mlp"]
        if f is None:
            continue
        for e in range(f["router"]["experts"]):
            out[p + f"mlp.e{e}.up"] = (f["expert"]["ff"], w)
            out[p + f"mlp.e{e}.down"] = (w, f["expert"]["ff"])
        choices = f["router"]["experts"] + f["router"]["identity"]
        out[p + "mlp.router"] = (choices, w)
        out[p + "mlp.correction"] = (choices,)
        out[p + "mlp.shared.up"] = (f["shared"]["ff"], w)
        out[p + "mlp.shared.down"] = (w, f["shared"]["ff"])
        out[p + "mlp.shared.sg"] = (1, w)
    return out


def make_weights(cfg, seed: int, sharp: float = 1.0) -> dict[str, torch.Tensor]:
    """Weights as a bfloat16 checkpoint stores them.  Projections are drawn at the scale that keeps
    activations of order one.  The norm weights of the queries are multiplied by ``sharp``, so that few keys carry
    a query's weight.  Decays are spread from fast to slow (a token far back still counts in some
    channels).  The router's rows are large, so that scores lie apart, and the corrections as large as the
    smaller scores, so that they decide some choices.  Norm weights stored around zero are drawn around
    zero, plain ones around one; biases are of the size of what they are added to."""
    gen = torch.Generator().manual_seed(seed)

    def normal(shape, std=1.0, mean=0.0):
        return mean + std * torch.randn(shape, generator=gen)

    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        fan = shape[-1] if len(shape) == 2 else 1
        if name == "embed":
            t = normal(shape, 0.9)
        elif last == "norm1" or name == "final.norm":
            t = normal(shape, 0.2)
        elif name.endswith("q.norm"):
            t = normal(shape, 0.1, sharp)
        elif last in ("norm", "out"):
            t = normal(shape, 0.1, 1.0)
        elif last == "conv":
            t = normal(shape, 0.6)
        elif last in ("a1", "a2"):
            t = normal(shape, 1.0 / fan**0.5)
        elif name.endswith("a2.b"):
            t = normal(shape, 2.5, 1.0)
        elif last == "b":
            t = normal(shape, 0.4)
        elif last == "router":
            t = normal(shape, 3.0 / fan**0.5)
        elif last == "correction":
            t = normal(shape, 0.15)
        else:
            t = normal(shape, 1.5 / fan**0.5)
        out[name] = t
    return {name: t.to(torch.bfloat16) for name, t in out.items()}


def make_model_dir(tmp_path: Path, which: str, sharp: float = 1.0, cfg=None, seed: int | None = None,
                   weights: dict[str, torch.Tensor] | None = None) -> Path:
    from safetensors.torch import save_file

    base, _page, base_seed = RENI[which]
    cfg = cfg or base
    out = Path(tmp_path) / f"reni_{which}_{sharp}_{seed}"
    out.mkdir(parents=True, exist_ok=True)
    (out / "config.json").write_text(json.dumps(cfg))
    weights = weights or make_weights(cfg, base_seed if seed is None else seed, sharp)
    save_file({k: v.contiguous() for k, v in weights.items()}, str(out / "model.safetensors"))
    return out


def load_plain(model_dir: Path):
    from safetensors.torch import load_file

    return json.loads((Path(model_dir) / "config.json").read_text()), load_file(str(Path(model_dir) / "model.safetensors"))


def random_tokens(n: int, vocab: int, seed: int) -> list[int]:
    rng = random.Random(seed)
    return [rng.randrange(vocab) for _ in range(n)]


# a bfloat16 engine's rows may be off by this many times what rounding does to the plain implementation
BF16_TIMES_ROUNDING = 3.0
# and this share of them may be off by more: a token whose experts' scores lie closer than rounding moves them
# takes another expert, in an engine as in the plain implementation with rounded activations
BF16_ROWS_BEYOND = 0.1


def row_errors(got: torch.Tensor, want: torch.Tensor) -> torch.Tensor:
    """Per row the root mean square of ``got - want`` over the spread of ``want``."""
    return (got.double() - want.double()).square().mean(dim=1).sqrt() / float(want.double().std())
