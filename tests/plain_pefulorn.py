"""A plain, slow implementation of the Pefulorn decoder in float64 torch on the CPU: the oracle of
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


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z**3)))


def projection(w, name, h, cast=same):
    """The product with a matrix and, where the checkpoint has one, its bias."""
    y = h @ w[name].T
    if name + ".b" in w:
        y = y + w[name + ".b"]
    return cast(y)


# --------------------------------------------------------------------------- #
# the gated delta rule with a decay per key channel
# --------------------------------------------------------------------------- #


def short_convolution(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """``x [T, channels]``, ``taps [channels, n]``; the last tap meets the current token."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=x.dtype), x], 0)
    y = torch.zeros_like(x)
    for tap in range(n):
        y = y + padded[tap : tap + T] * taps[:, tap]
    return silu(y)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """``q, k, g [T, H, d]``, ``v [T, H, dv]``, ``beta [T, H]`` -> ``[T, H, dv]``."""
    T, H, d = k.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F)
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for t in range(T):
        S = g[t].unsqueeze(-1) * S
        held = (S * k[t].unsqueeze(-1)).sum(1)
        u = beta[t].unsqueeze(-1) * (v[t] - held)
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(-2)
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out


def channel_delta(m: dict, w: dict, p: str, h: torch.Tensor, eps: float, cast=same) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_convolution(projection(w, p + "q", h, cast), w[p + "q.conv"]).view(T, G, d)
    k = short_convolution(projection(w, p + "k", h, cast), w[p + "k.conv"]).view(T, G, d)
    v = short_convolution(projection(w, p + "v", h, cast), w[p + "v.conv"]).view(T, H, dv)
    q, k = unit(q) * d**-0.5, unit(k)
    of = torch.tensor([i // (H // G) for i in range(H)])
    beta = torch.sigmoid(projection(w, p + "b", h))
    low = projection(w, p + "a1", h)
    rate = torch.exp(w[p + "A_log"]).view(1, H, 1)
    g = torch.exp(-rate * softplus(projection(w, p + "a2", low) + w[p + "dt_bias"]).view(T, H, d))
    o = delta_rule(q[:, of], k[:, of], v, g, beta)
    gate = torch.sigmoid(projection(w, p + "g2", projection(w, p + "g1", h, cast), cast)).view(T, H, dv)
    y = rms(o, eps) * w[p + "norm"] * gate
    return projection(w, p + "o", cast(y.reshape(T, H * dv)))


# --------------------------------------------------------------------------- #
# attention beside a gated recurrence
# --------------------------------------------------------------------------- #


def temperature(positions: torch.Tensor, coef: float, every) -> torch.Tensor:
    return 1.0 + coef * torch.log(torch.floor((positions + 1).to(F) / every) + 1.0)


def distance_attention(m: dict, w: dict, p: str, h: torch.Tensor, eps: float, cast=same) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = projection(w, p + "q", h, cast).view(T, H, d)
    k = projection(w, p + "k", h, cast).view(T, G, d)
    v = projection(w, p + "v", h, cast).view(T, G, dv)
    q = rms(q, eps) * w[p + "q.norm"]
    k = cast(rms(k, eps) * w[p + "k.norm"])
    v = cast(rms(v, eps))
    if m.get("q_temp"):
        q = q * temperature(torch.arange(T), m["q_temp"]["coef"], m["q_temp"]["every"]).view(T, 1, 1)
    q = cast(q)
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    distance = (i - j).clamp(min=0).to(F)
    out = torch.zeros(T, H, dv, dtype=F)
    for head in range(H):
        kv = head // (H // G)
        s = (q[:, head] @ k[:, kv].T) * m["scale"]
        s = s - w[p + "r1"][head] * torch.log(1.0 + w[p + "r2"][head] * distance)
        s = s.masked_fill(j > i, -math.inf)
        out[:, head] = torch.softmax(s, -1) @ v[:, kv]
    return projection(w, p + "o", cast(out.reshape(T, H * dv)))


def min_gru(m: dict, w: dict, p: str, h: torch.Tensor, cast=same) -> torch.Tensor:
    z = torch.sigmoid(projection(w, p + "z", h, cast))
    u = projection(w, p + "x", h, cast)
    candidate = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    S = torch.zeros(m["width"], dtype=F)
    rows = []
    for t in range(h.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * candidate[t]
        rows.append(S)
    y = torch.stack(rows) * silu(projection(w, p + "g", h, cast))
    return projection(w, p + "o", cast(y))


def parallel(m: dict, w: dict, p: str, h: torch.Tensor, eps: float, cast=same) -> torch.Tensor:
    left = distance_attention(m["left"], w, p + "left.", h, eps, cast)
    right = min_gru(m["right"], w, p + "right.", h, cast)
    return m["left_scale"] * left + m["right_scale"] * right


# --------------------------------------------------------------------------- #
# time mixing with the token before
# --------------------------------------------------------------------------- #


def wkv(m: dict, w: dict, p: str, h: torch.Tensor, eps: float, cast=same) -> torch.Tensor:
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    before = torch.cat([torch.zeros(1, h.shape[1], dtype=F), h[:-1]], 0)
    mix = {s: h + (before - h) * w[p + "mu." + s] for s in "rkvgw"}
    r, k, v, g = (projection(w, p + s, cast(mix[s]), cast) for s in "rkvg")
    r, k, v = (x.view(T, H, d) for x in (r, k, v))
    pre = torch.tanh(mix["w"] @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]
    decay = torch.exp(-torch.exp(pre)).view(T, H, d)
    S = torch.zeros(H, d, d, dtype=F)  # [head, key channel, value channel]
    out = torch.zeros(T, H, d, dtype=F)
    for t in range(T):
        kv = k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        out[t] = ((S + w[p + "u"].unsqueeze(-1) * kv) * r[t].unsqueeze(-1)).sum(1)
        S = decay[t].unsqueeze(-1) * S + kv
    y = rms(out, eps).reshape(T, H * d) * w[p + "norm"] * silu(g)
    return projection(w, p + "o", cast(y))


MIXERS = {"channel_delta": channel_delta, "parallel": parallel, "wkv": wkv}


# --------------------------------------------------------------------------- #
# feed-forward and the model
# --------------------------------------------------------------------------- #


def dense(w: dict, p: str, h: torch.Tensor, cast=same) -> torch.Tensor:
    hidden = gelu_tanh(projection(w, p + "gate", h, cast)) * projection(w, p + "up", h, cast)
    return projection(w, p + "down", cast(hidden))


def passes(cfg: dict) -> list[tuple[int, int | None]]:
    """(layer, pass that begins right before it or ``None``) in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    order = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        order += [(i, t if i == a else None) for i in range(a, b)]
    return order + [(i, None) for i in range(b, n)]


def forward(cfg: dict, w: dict, tokens: list[int], streams: list | None = None, cast=same) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence from its start.  ``streams``: a list that receives
    the residual stream after every layer run."""
    w = {name: t.to(F) for name, t in w.items()}
    eps = cfg["norm"]["eps"]
    x0 = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    x = x0
    for i, begins in passes(cfg):
        if begins is not None:
            if begins > 0:
                x = x + x0
            x = x + w["loop.step"][begins]
        layer, p = cfg["layers"][i], f"l{i}."
        h = cast(around_one_norm(x, w[p + "norm1"], eps))
        x = x + MIXERS[layer["type"]](layer["mixer"], w, p + "mix.", h, eps, cast)
        if layer.get("mlp") is not None:
            x = x + dense(w, p + "mlp.", cast(around_one_norm(x, w[p + "norm2"], eps)), cast)
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
