"""A plain, slow implementation of the Renitar decoder in float64 torch on the CPU: the oracle of
the tests.  One function per mechanism, whole sequences only, no cache, no batching; it shares
no code with the package.

``cfg`` is the ``config.json`` dictionary, ``w`` maps checkpoint tensor names to tensors.  ``cast``
(optional) is applied wherever an engine that computes in a narrower type would round: the
normed rows, the projections' results, the activations; never to what the design keeps in 32-bit.
"""

from __future__ import annotations

import math

import torch

F = torch.float64


def same(x):
    return x


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """``x`` divided by the root of (the mean of its squares over the last axis, plus eps)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def around_one_norm(x, weight, eps):
    return rms(x, eps) * (1.0 + weight)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_exact(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def projection(w, name, h, cast=same):
    """The product with a matrix and, where the checkpoint has one, its bias."""
    y = h @ w[name].T
    if name + ".b" in w:
        y = y + w[name + ".b"]
    return cast(y)


# --------------------------------------------------------------------------- #
# linear attention
# --------------------------------------------------------------------------- #


def decayed_memory(q, k, v, alpha):
    """``q, k [T, H, d]``, ``v [T, H, dv]``, ``alpha`` a factor for every row of the memory (``[T, H, d]`` or
    broadcast to it) -> ``[T, H, dv]``: the memory is decayed, takes the token in, and is read."""
    T, H, d = k.shape
    alpha = alpha.expand(T, H, d)
    S = torch.zeros(H, d, v.shape[2], dtype=F)
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for t in range(T):
        S = alpha[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out


def channel_decay(z: torch.Tensor, tau: float) -> torch.Tensor:
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def gla(m: dict, w: dict, p: str, h: torch.Tensor, eps: float, cast=same) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = projection(w, p + "q", h, cast).view(T, H, d) * d**-0.5
    k = projection(w, p + "k", h, cast).view(T, H, d)
    v = projection(w, p + "v", h, cast).view(T, H, dv)
    z = projection(w, p + "a2", projection(w, p + "a1", h))
    o = decayed_memory(q, k, v, channel_decay(z.view(T, H, d), m["tau"]))
    y = (rms(o, eps) * w[p + "norm"]).reshape(T, H * dv) * silu(projection(w, p + "g", h, cast))
    return projection(w, p + "o", cast(y), cast)


def lightning(m: dict, w: dict, p: str, h: torch.Tensor, eps: float, cast=same) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = silu(projection(w, p + "q", h, cast)).view(T, H, d)
    k = silu(projection(w, p + "k", h, cast)).view(T, H, d)
    v = silu(projection(w, p + "v", h, cast)).view(T, H, dv)
    o = decayed_memory(q, k, v, torch.tensor(m["decay"], dtype=F).view(1, H, 1))
    y = rms(o.reshape(T, H * dv), eps) * w[p + "norm"] * torch.sigmoid(projection(w, p + "g", h, cast))
    return projection(w, p + "o", cast(y), cast)


# --------------------------------------------------------------------------- #
# attention in chunks behind short convolutions
# --------------------------------------------------------------------------- #


def short_convolution(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """``x [T, channels]``, ``taps [channels, n]``; the last tap meets the current token."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=x.dtype), x], 0)
    y = torch.zeros_like(x)
    for tap in range(n):
        y = y + padded[tap : tap + T] * taps[:, tap]
    return y


def rotate(x: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """``x [T, heads, d]``: channels ``i`` and ``i + dims / 2`` turn by ``position * base^(-2i / dims)``."""
    T, half = x.shape[0], dims // 2
    freq = base ** (-2.0 * torch.arange(half, dtype=F) / dims)
    angle = (torch.arange(T, dtype=F).view(T, 1) * freq).view(T, 1, half)
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([u * angle.cos() - v * angle.sin(), v * angle.cos() + u * angle.sin(), rest], -1)


def chunk_mask(T: int, size: int) -> torch.Tensor:
    """``[i, j]``: whether position i sees position j."""
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    return (j <= i) & (i // size == j // size)


def soft_cap(s: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(s / cap)


def chunked_attention(m: dict, w: dict, p: str, h: torch.Tensor, eps: float, cast=same) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_convolution(projection(w, p + s, h, cast), w[p + s + ".conv"]) for s in "qkv")
    q = (rms(q, eps) * w[p + "q.norm"]).view(T, H, d)
    k = (rms(k, eps) * w[p + "k.norm"]).view(T, G, d)
    q = cast(rotate(q, m["rot"]["dims"], m["rot"]["base"]))
    k = cast(rotate(k, m["rot"]["dims"], m["rot"]["base"]))
    v = cast(v).view(T, G, dv)
    seen = chunk_mask(T, m["mask"]["size"])
    out = torch.zeros(T, H, dv, dtype=F)
    for head in range(H):
        kv = head // (H // G)
        s = soft_cap((q[:, head] @ k[:, kv].T) * m["scale"], m["softcap"])
        out[:, head] = torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ v[:, kv]
    y = out.reshape(T, H * dv) * torch.sigmoid(projection(w, p + "g", h, cast))
    return projection(w, p + "o", cast(y), cast)


def parallel(m: dict, w: dict, p: str, h: torch.Tensor, eps: float, cast=same) -> torch.Tensor:
    left = chunked_attention(m["left"], w, p + "left.", h, eps, cast)
    right = lightning(m["right"], w, p + "right.", h, eps, cast)
    return 0.5 * (rms(left, eps) * w[p + "left.out"] + rms(right, eps) * w[p + "right.out"])


MIXERS = {"gla": gla, "parallel": parallel}


# --------------------------------------------------------------------------- #
# feed-forward and the model
# --------------------------------------------------------------------------- #


def expert(w: dict, p: str, h: torch.Tensor, cast=same, weight=None) -> torch.Tensor:
    hidden = gelu_exact(projection(w, p + "up", h, cast))
    if weight is not None:  # (the second product is linear: an engine may weigh the hidden units)
        hidden = hidden * weight
    return projection(w, p + "down", cast(hidden))


def expert_weights(r: dict, w: dict, p: str, h: torch.Tensor) -> torch.Tensor:
    """``[T, experts + identity]``: the chosen experts' weights, 0 for the others."""
    s = torch.softmax(h @ w[p + "router"].T, -1)
    chosen = torch.topk(s + w[p + "correction"], r["top"], -1).indices
    mask = torch.zeros_like(s).scatter_(-1, chosen, 1.0)
    return s * mask * r["scale"]


def mixture(m: dict, w: dict, p: str, h: torch.Tensor, cast=same) -> torch.Tensor:
    r = m["router"]
    weights = expert_weights(r, w, p, h)
    y = torch.zeros_like(h)
    for e in range(r["experts"]):
        y = y + expert(w, p + f"e{e}.", h, cast, weights[:, e : e + 1])
    for e in range(r["experts"], r["experts"] + r["identity"]):
        y = y + weights[:, e : e + 1] * h
    return y + expert(w, p + "shared.", h, cast, torch.sigmoid(h @ w[p + "shared.sg"].T))


def forward(cfg: dict, w: dict, tokens: list[int], streams: list | None = None, cast=same) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence from its start.  ``streams``: a list that receives
    the residual stream after every layer."""
    w = {name: t.to(F) for name, t in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = cast(around_one_norm(x, w[p + "norm1"], eps))
        y = MIXERS[layer["type"]](layer["mixer"], w, p + "mix.", h, eps, cast)
        if layer.get("mlp") is not None:
            y = y + mixture(layer["mlp"], w, p + "mlp.", h, cast)
        x = x + cfg["residual_mult"] * y
        if streams is not None:
            streams.append(x.clone())
    return cast(around_one_norm(x, w["final.norm"], eps)) @ w["head"].T


def greedy(cfg: dict, w: dict, prompt: list[int], steps: int) -> list[int]:
    ids, out = list(prompt), []
    for _ in range(steps):
        tok = int(forward(cfg, w, ids)[-1].argmax())
        out.append(tok)
        ids.append(tok)
    return out
