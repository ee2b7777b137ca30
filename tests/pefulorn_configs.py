"""Small Pefulorn configurations that differ in every size and option, and random weights for
them, made here tensor by tensor (names and shapes written out once more, independent of the
package's own list of parameters)."""

from __future__ import annotations

import json
import random
from pathlib import Path

import torch


def _delta(heads, kv_heads, dim, vdim, conv, decay_rank, gate_rank):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "decay_rank": decay_rank,
            "gate_rank": gate_rank}


def _parallel(heads, kv_heads, dim, vdim, scale, width, left_scale, right_scale, q_temp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if q_temp:
        left["q_temp"] = {"coef": q_temp[0], "every": q_temp[1]}
    return {"left": left, "right": {"width": width}, "left_scale": left_scale, "right_scale": right_scale}


def _wkv(heads, dim, rank):
    return {"heads": heads, "dim": dim, "rank": rank}


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


# A: grouped heads with values wider than the keys and a temperature that steps every 7 positions; a
# delta rule with grouped keys, values wider than keys, three taps and no feed-forward; a time mixing;
# the last two run twice; then attention whose values are narrower and whose queries have no
# temperature, beside a wider recurrence; pages of 8
PEFU_A = {
    "architecture": "Pefulorn", "width": 96, "vocab": 211, "norm": {"eps": 3e-6},
    "layers": [
        _layer("parallel", _parallel(4, 2, 16, 32, 0.3, 40, 0.7, 1.2, (0.4, 7)), 80),
        _layer("channel_delta", _delta(4, 2, 16, 24, 3, 8, 6), 0),
        _layer("wkv", _wkv(3, 16, 8), 64),
        _layer("parallel", _parallel(2, 1, 32, 16, 0.2, 72, 1.0, 0.5), 48),
    ],
    "loop": {"start": 1, "stop": 3, "times": 2},
}
PAGE_A = 8

# B: the smallest of everything: one head, a convolution of a single tap, low-rank pairs of rank 1, a
# recurrence of one channel, a temperature that steps at every position; all layers run three times,
# from the first on; pages of 4
PEFU_B = {
    "architecture": "Pefulorn", "width": 64, "vocab": 130, "norm": {"eps": 1e-6},
    "layers": [
        _layer("channel_delta", _delta(1, 1, 16, 16, 1, 1, 1), 16),
        _layer("parallel", _parallel(1, 1, 16, 16, 0.25, 1, -0.5, 1.0, (0.2, 1)), 0),
        _layer("wkv", _wkv(1, 32, 1), 24),
    ],
    "loop": {"start": 0, "stop": 3, "times": 3},
}
PAGE_B = 4

# C: sizes that no vector access divides and that lie between the matrix cores' steps: heads of 12
# and of an odd size, a delta rule of 20 key and 13 value channels with two taps, a recurrence of 37
# channels, feed-forwards of 50 and 27, width 100, vocabulary 97, no loop; pages of 8
PEFU_C = {
    "architecture": "Pefulorn", "width": 100, "vocab": 97, "norm": {"eps": 1e-5},
    "layers": [
        _layer("channel_delta", _delta(6, 3, 20, 13, 2, 5, 3), 50),
        _layer("parallel", _parallel(6, 3, 12, 10, 0.3, 37, 0.8, 0.9, (0.3, 5)), 27),
        _layer("wkv", _wkv(5, 20, 3), 36),
        _layer("parallel", _parallel(3, 1, 9, 22, 0.4, 50, 1.1, 0.6, (-0.1, 16)), 0),
    ],
}
PAGE_C = 8

# D: heads of the sizes real models have: a delta rule of 64 key and 128 value channels with four
# taps, another of 32 with seven, keys of 64 with values of 32, a time mixing with heads of 64, a loop
# of a single pass over one layer; pages of 16
PEFU_D = {
    "architecture": "Pefulorn", "width": 128, "vocab": 300, "norm": {"eps": 2e-5},
    "layers": [
        _layer("wkv", _wkv(2, 64, 16), 160),
        _layer("channel_delta", _delta(2, 1, 64, 128, 4, 16, 24), 96),
        _layer("parallel", _parallel(4, 1, 64, 32, 0.11, 160, 0.6, 0.8, (0.25, 20)), 128),
        _layer("channel_delta", _delta(3, 3, 32, 32, 7, 12, 8), 64),
    ],
    "loop": {"start": 2, "stop": 3, "times": 1},
}
PAGE_D = 16

# E: recurrent layers alone, so that no request has pages: a delta rule of 48 key channels, time
# mixing with heads of 24, passes over the last layer only; pages of 8 that nobody asks for
PEFU_E = {
    "architecture": "Pefulorn", "width": 80, "vocab": 141, "norm": {"eps": 1e-5},
    "layers": [
        _layer("channel_delta", _delta(4, 4, 48, 20, 5, 7, 9), 40),
        _layer("wkv", _wkv(2, 24, 5), 56),
    ],
    "loop": {"start": 1, "stop": 2, "times": 4},
}
PAGE_E = 8

PEFU = {"A": (PEFU_A, PAGE_A, 701), "B": (PEFU_B, PAGE_B, 702), "C": (PEFU_C, PAGE_C, 703), "D": (PEFU_D, PAGE_D, 704),
        "E": (PEFU_E, PAGE_E, 705)}


def tensor_shapes(cfg) -> dict[str, tuple[int, ...]]:
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "head": (cfg["vocab"], w)}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], w)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (w,)
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]["width"]
            for s, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                out[p + "mix.left." + s] = (rows, w)
                out[p + "mix.left." + s + ".b"] = (rows,)
            for s in ("q.norm", "k.norm"):
                out[p + "mix.left." + s] = (a["dim"],)
            for s in ("r1", "r2"):
                out[p + "mix.left." + s] = (a["heads"],)
            out[p + "mix.left.o"] = (w, a["heads"] * a["vdim"])
            for s in ("z", "x", "g"):
                out[p + "mix.right." + s] = (r, w)
            for s in ("z.b", "x.b"):
                out[p + "mix.right." + s] = (r,)
            out[p + "mix.right.o"] = (w, r)
        elif layer["type"] == "wkv":
            inner = m["heads"] * m["dim"]
            for s in "rkvgw":
                out[p + "mix.mu." + s] = (w,)
            for s in "rkvg":
                out[p + "mix." + s] = (inner, w)
            out[p + "mix.w1"] = (m["rank"], w)
            out[p + "mix.w2"] = (inner, m["rank"])
            out[p + "mix.w0"] = (inner,)
            out[p + "mix.u"] = (m["heads"], m["dim"])
            out[p + "mix.norm"] = (inner,)
            out[p + "mix.o"] = (w, inner)
        else:
            keys, kv, values = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for s, rows in (("q", kv), ("k", kv), ("v", values)):
                out[p + "mix." + s] = (rows, w)
                out[p + "mix." + s + ".conv"] = (rows, m["conv"])
            out[p + "mix.b"] = (m["heads"], w)
            out[p + "mix.A_log"] = (m["heads"],)
            out[p + "mix.a1"] = (m["decay_rank"], w)
            out[p + "mix.a2"] = (keys, m["decay_rank"])
            out[p + "mix.dt_bias"] = (keys,)
            out[p + "mix.g1"] = (m["gate_rank"], w)
            out[p + "mix.g2"] = (values, m["gate_rank"])
            out[p + "mix.norm"] = (m["vdim"],)
            out[p + "mix.o"] = (w, values)
        if layer["mlp"] is None:
            continue
        out[p + "norm2"] = (w,)
        for s in ("gate", "up"):
            out[p + "mlp." + s] = (layer["mlp"]["ff"], w)
            out[p + "mlp." + s + ".b"] = (layer["mlp"]["ff"],)
        out[p + "mlp.down"] = (w, layer["mlp"]["ff"])
        out[p + "mlp.down.b"] = (w,)
    return out


def make_weights(cfg, seed: int, sharp: float = 1.0) -> dict[str, torch.Tensor]:
    """Weights as a bfloat16 checkpoint stores them.  Projections are drawn at the scale that keeps
    activations of order one.  The norms' weights of the query heads are multiplied by ``sharp``, so that
    few keys carry a query's weight.  Decays and the recurrence's gates are spread from fast to very
    slow (a token far back still counts in some channels).  Norm weights stored around zero are drawn
    around zero, plain ones around one; biases are of the size of what they are added to."""
    gen = torch.Generator().manual_seed(seed)

    def normal(shape, std=1.0, mean=0.0):
        return mean + std * torch.randn(shape, generator=gen)

    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        fan = shape[-1] if len(shape) == 2 else 1
        if name == "embed":
            t = normal(shape, 0.7)
        elif name == "loop.step":
            t = normal(shape, 0.4)
        elif last in ("norm1", "norm2") or name == "final.norm":
            t = normal(shape, 0.2)
        elif name.endswith("q.norm"):
            t = normal(shape, 0.1, sharp)
        elif last == "norm":
            t = normal(shape, 0.1, 1.0)
        elif ".mu." in name:
            t = torch.rand(shape, generator=gen)
        elif last == "r1":
            t = 0.3 + torch.rand(shape, generator=gen)
        elif last == "r2":
            t = 0.05 + 0.5 * torch.rand(shape, generator=gen)
        elif last == "w0":
            t = normal(shape, 1.5, -2.5)
        elif last in ("w1", "w2", "a1", "a2", "g1", "g2"):
            t = normal(shape, 1.0 / fan**0.5)
        elif last == "u":
            t = normal(shape, 0.5)
        elif last == "conv":
            t = normal(shape, 0.7)
        elif last == "dt_bias":
            t = normal(shape, 1.5, -3.0)
        elif last == "A_log":
            t = normal(shape, 1.0, -0.5)
        elif name.endswith("right.z.b"):
            t = normal(shape, 1.5, -2.5)
        elif last == "b" and len(shape) == 1:
            t = normal(shape, 0.4)
        else:
            t = normal(shape, 1.5 / fan**0.5)
        out[name] = t
    return {name: t.to(torch.bfloat16) for name, t in out.items()}


def make_model_dir(tmp_path: Path, which: str, sharp: float = 1.0, cfg=None, seed: int | None = None,
                   weights: dict[str, torch.Tensor] | None = None) -> Path:
    from safetensors.torch import save_file

    base, _page, base_seed = PEFU[which]
    cfg = cfg or base
    out = Path(tmp_path) / f"pefu_{which}_{sharp}_{seed}"
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


# a bfloat16 engine's rows may be off by this many times what rounding does to the worst row of the
# plain implementation with rounded activations
BF16_TIMES_ROUNDING = 2.5


def row_errors(got: torch.Tensor, want: torch.Tensor) -> torch.Tensor:
    """Per row the root mean square of ``got - want`` over the spread of ``want``."""
    return (got.double() - want.double()).square().mean(dim=1).sqrt() / float(want.double().std())
