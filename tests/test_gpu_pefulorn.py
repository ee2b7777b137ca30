"""The Pefulorn decoder in the engine against the plain implementation of ``plain_pefulorn.py``:
every mechanism alone, every way of cutting requests into steps, state slots and pages that are
used again, keys far away and at page borders, long decoding, and greedy generation through the
entry point."""

import math
import random
from types import SimpleNamespace

import pytest
import torch

import parity
import plain_pefulorn as pp
import replay_util as ru
from pefulorn_configs import (
    BF16_TIMES_ROUNDING,
    PEFU,
    load_plain,
    make_model_dir,
    random_tokens,
    row_errors,
)

pytestmark = pytest.mark.gpu

DEV = "cuda"
F32_ROW = 2e-4  # float32 rows against float64: root mean square over a row, relative to the logits' spread
D64 = torch.float64
TYPES = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


def _ops():
    from rapid_llm_amd.kernels import ops

    return ops


def bf16_round(t):
    return t.bfloat16().to(t.dtype)


def _tol(dtype, f32=2e-5, bf16=2e-2):
    return dict(rtol=f32, atol=f32) if dtype == torch.float32 else dict(rtol=bf16, atol=bf16)


def _step(lens, slots):
    """What the recurrent kernels read of a step: the requests' offsets and their state rows."""
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    return SimpleNamespace(
        cu_seqlens=torch.tensor(cu, dtype=torch.int32, device=DEV),
        seq_slots=torch.tensor(slots, dtype=torch.int32, device=DEV),
        num_seqs=len(lens), h_seq_lens=list(lens), h_seq_slots=list(slots),
    )


def _cuts(total, sizes):
    """``total`` tokens cut into portions of the given sizes in turn."""
    out, at, i = [], 0, 0
    while at < total:
        n = min(sizes[i % len(sizes)], total - at)
        out.append((at, at + n))
        at += n
        i += 1
    return out


def _interleaved(lengths, sizes, slots, states, run):
    """Feed requests in portions of the given sizes through shared steps; a request that starts finds
    the rows of its slot zeroed (what taking a slot does).  ``run(ctx, [(request, first, end), ..])``
    returns the step's rows; the result is the rows per request."""
    cuts = {r: _cuts(lengths[r], sizes[r]) for r in lengths}
    waiting = list(lengths)
    live: list = []
    got = {r: [] for r in lengths}
    while waiting or live:
        for r in list(waiting):
            if slots[r] not in [slots[x] for x in live]:  # its slot is free
                waiting.remove(r)
                live.append(r)
        now = [(r, *cuts[r].pop(0)) for r in live]
        for r, a, _b in now:
            if a == 0:
                for s in states:
                    s[slots[r]].zero_()
        rows = run(_step([b - a for _r, a, b in now], [slots[r] for r, _a, _b in now]), now)
        at = 0
        for r, a, b in now:
            got[r].append(rows[at : at + b - a].double().cpu())
            at += b - a
        live = [r for r in live if cuts[r]]
    return {r: torch.cat(parts) for r, parts in got.items()}


# --------------------------------------------------------------------------- #
# the gated delta rule
# --------------------------------------------------------------------------- #
DELTA_SHAPES = [  # heads, kv heads, key channels, value channels, taps
    (4, 2, 16, 24, 3), (6, 3, 20, 13, 2), (2, 1, 64, 128, 4), (1, 1, 16, 16, 1), (3, 3, 100, 8, 4), (2, 2, 200, 33, 13),
    (1, 1, 1, 1, 4), (2, 1, 128, 64, 7),
]


@TYPES
@pytest.mark.parametrize("heads,kv,d,dv,taps", DELTA_SHAPES)
def test_delta_rule_continues_from_the_slot(dtype, heads, kv, d, dv, taps):
    """Convolution, unit vectors, decays and the scan: four requests in portions down to one token
    (shorter than the convolution's reach, so that kept inputs are shifted and not replaced), on
    shuffled slots of which one is taken again by a later request."""
    ops = _ops()
    gen = torch.Generator().manual_seed(heads * 1000 + d * 10 + taps)
    channels = 2 * kv * d + heads * dv
    col0, width = 8, channels + 8 + 5  # columns on both sides are not this kernel's
    conv = torch.randn(channels, taps, generator=gen) * 0.7
    dt_bias = torch.randn(heads * d, generator=gen) * 1.5 - 2.0
    a_log = torch.randn(heads, generator=gen) - 0.5
    lengths = {"a": 41, "b": 5, "c": 64, "d": 9}
    data, want_mixed, want = {}, {}, {}
    of = torch.arange(heads) // (heads // kv)
    for rid, T in lengths.items():
        packed = torch.randn(T, width, generator=gen).to(dtype).float()
        pre, beta = torch.randn(T, heads * d, generator=gen), torch.randn(T, heads + 3, generator=gen)
        data[rid] = (packed, pre, beta)
        y = pp.short_convolution(packed[:, col0 : col0 + channels].double(), conv.double())
        q = pp.unit(y[:, : kv * d].view(T, kv, d)) * d**-0.5
        k = pp.unit(y[:, kv * d : 2 * kv * d].view(T, kv, d))
        v = y[:, 2 * kv * d :].view(T, heads, dv)
        g = torch.exp(-torch.exp(a_log.double()).view(1, heads, 1)
                      * pp.softplus(pre.double() + dt_bias.double()).view(T, heads, d))
        want_mixed[rid] = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1)
        want[rid] = pp.delta_rule(q[:, of], k[:, of], v, g, torch.sigmoid(beta[:, :heads].double())).reshape(T, heads * dv)
    conv_state = torch.full((5, max(taps - 1, 1), channels), float("nan"), device=DEV)
    S = torch.full((5, heads, dv, d), float("nan"), device=DEV)

    def run(ctx, now):
        packed, pre, beta = (torch.cat([data[r][i][a:b] for r, a, b in now]).to(DEV) for i in range(3))
        tokens = packed.shape[0]
        mixed = torch.full((tokens, channels), float("nan"), device=DEV)
        ops.delta_prepare(packed.to(dtype), col0, conv.to(DEV), conv_state, pre, dt_bias.to(DEV), a_log.to(DEV), mixed,
                          ctx, heads, kv, d, dv)
        raw = torch.full((tokens, heads * dv), float("nan"), device=DEV)
        ops.delta_scan(mixed, pre, beta, raw, ctx, S, heads, kv, d, dv)
        return torch.cat([mixed, raw], 1)

    got = _interleaved(lengths, {"a": (7, 1, 2, 1, 1, 11), "b": (2, 1, 2), "c": (1, 1, 30, 2), "d": (9,)},
                       {"a": 3, "b": 0, "c": 1, "d": 0}, [conv_state, S], run)
    for rid in lengths:
        torch.testing.assert_close(got[rid][:, :channels], want_mixed[rid], rtol=2e-5, atol=2e-5)
        torch.testing.assert_close(got[rid][:, channels:], want[rid], rtol=2e-4, atol=5e-5)


def test_delta_rule_is_the_same_bit_for_bit_however_it_is_cut():
    ops = _ops()
    heads, kv, d, dv, taps = 3, 1, 48, 40, 4
    channels, T = 2 * kv * d + heads * dv, 75
    packed = torch.randn(T, channels, device=DEV).bfloat16()
    conv, dt_bias, a_log = torch.randn(channels, taps, device=DEV), torch.randn(heads * d, device=DEV) - 2, torch.randn(heads, device=DEV)
    pre, beta = torch.randn(T, heads * d, device=DEV), torch.randn(T, heads, device=DEV)

    def run(cuts):
        conv_state, S = torch.zeros(1, taps - 1, channels, device=DEV), torch.zeros(1, heads, dv, d, device=DEV)
        rows = []
        for a, b in cuts:
            mixed, decay = torch.empty(b - a, channels, device=DEV), pre[a:b].clone()
            raw = torch.empty(b - a, heads * dv, device=DEV)
            ctx = _step([b - a], [0])
            ops.delta_prepare(packed[a:b].contiguous(), 0, conv, conv_state, decay, dt_bias, a_log, mixed, ctx, heads, kv, d, dv)
            ops.delta_scan(mixed, decay, beta[a:b].contiguous(), raw, ctx, S, heads, kv, d, dv)
            rows.append(raw)
        return torch.cat(rows), S

    whole = run([(0, T)])
    for sizes in ((1,), (2, 3), (16,), (17, 5, 1)):
        cut = run(_cuts(T, sizes))
        assert torch.equal(cut[0], whole[0]) and torch.equal(cut[1], whole[1]), sizes


@TYPES
@pytest.mark.parametrize("gate", ["silu", "sigmoid"])
@pytest.mark.parametrize("heads,d,shared", [(4, 24, True), (3, 64, False), (1, 130, True), (5, 13, False)])
def test_head_norm_weight_and_gate(dtype, gate, heads, d, shared):
    ops = _ops()
    raw = torch.randn(11, heads * d) * 3.0
    g = torch.randn(11, heads * d).to(dtype)
    w = 1.0 + 0.2 * torch.randn(d if shared else heads * d)
    out = torch.empty((11, heads * d), dtype=dtype, device=DEV)
    ops.head_finish(raw.to(DEV), g.to(DEV), w.to(DEV), out, heads, 1e-5, gate)
    factor = torch.sigmoid(g.double()) * (g.double() if gate == "silu" else 1.0)
    want = pp.rms(raw.double().view(11, heads, d), 1e-5) * (w.double() if shared else w.double().view(heads, d))
    torch.testing.assert_close(out.double().cpu(), want.reshape(11, -1) * factor, **_tol(dtype, 1e-5, 1e-2))


# --------------------------------------------------------------------------- #
# the gated recurrence of one number a channel
# --------------------------------------------------------------------------- #


@TYPES
@pytest.mark.parametrize("width", [40, 37, 1, 300])
def test_min_gru_continues_from_the_slot(dtype, width):
    ops = _ops()
    gen = torch.Generator().manual_seed(width)
    zc, xc, gc = 5 + 2 * width, 5, 5 + width  # anywhere in a wider row
    row = 5 + 3 * width + 2
    zb, xb = torch.randn(width, generator=gen) - 1.5, torch.randn(width, generator=gen) * 0.4
    lengths = {"a": 150, "b": 5, "c": 64, "d": 9, "e": 65}
    data, want = {}, {}
    for rid, T in lengths.items():
        packed = torch.randn(T, row, generator=gen).to(dtype).float()
        data[rid] = packed
        p64 = packed.double()
        eye = torch.eye(width, dtype=D64)
        # the plain mechanism on identity projections of the three parts
        h = torch.cat([p64[:, c : c + width] for c in (zc, xc, gc)], 1)
        w = {s: torch.zeros(width, 3 * width, dtype=D64) for s in "zxg"}
        for i, s in enumerate("zxg"):
            w[s][:, i * width : (i + 1) * width] = eye
        w.update({"z.b": zb.double(), "x.b": xb.double(), "o": eye})
        want[rid] = pp.min_gru({"width": width}, w, "", h) * 0.7
    S = torch.full((4, width), float("nan"), device=DEV)

    def run(ctx, now):
        packed = torch.cat([data[r][a:b] for r, a, b in now]).to(DEV, dtype)
        out = torch.full((packed.shape[0], width + 7), float("nan"), dtype=dtype, device=DEV)
        ops.min_gru(packed, (zc, xc, gc), zb.to(DEV), xb.to(DEV), out, ctx, S, out_col=3, out_scale=0.7)
        assert torch.isnan(out[:, :3]).all() and torch.isnan(out[:, 3 + width :]).all()
        return out[:, 3 : 3 + width]

    got = _interleaved(lengths, {"a": (70, 1, 2, 64), "b": (2, 1, 2), "c": (1, 1, 30, 2), "d": (9,), "e": (65,)},
                       {"a": 3, "b": 0, "c": 1, "d": 0, "e": 2}, [S], run)
    for rid in lengths:
        torch.testing.assert_close(got[rid], want[rid], **_tol(dtype, 2e-5, 2e-2))


# --------------------------------------------------------------------------- #
# feed-forward, norms, the stream
# --------------------------------------------------------------------------- #


@TYPES
@pytest.mark.parametrize("inter", [48, 27, 3000])
def test_gelu_gate_with_biases(dtype, inter):
    ops = _ops()
    gate_up = (torch.randn(13, 2 * inter) * 2.0).to(dtype)
    bias = torch.randn(2 * inter)
    out = torch.empty((13, inter), dtype=dtype, device=DEV)
    ops.swiglu(gate_up.to(DEV), out, activation="gelu_tanh", bias=bias.to(DEV))
    z = gate_up.double() + bias.double()
    want = pp.gelu_tanh(z[:, :inter]) * z[:, inter:]
    torch.testing.assert_close(out.double().cpu(), want, **_tol(dtype, 1e-5, 2e-2))
    ops.swiglu(gate_up.to(DEV), out, bias=bias.to(DEV))  # the other activation takes a bias too
    torch.testing.assert_close(out.double().cpu(), pp.silu(z[:, :inter]) * z[:, inter:], **_tol(dtype, 1e-5, 2e-2))


@pytest.mark.parametrize("rows,width,inter", [(1, 128, 96), (8, 136, 50), (16, 256, 4208), (8, 1024, 4608), (30, 256, 2304), (300, 128, 2048),
                                              (40, 1024, 6144)])
def test_gelu_gate_with_biases_inside_the_products(rows, width, inter):
    """Every fused kernel: few rows, few rows over many tiles, one-launch tiles, wide matrices."""
    ops = _ops()
    gen = torch.Generator().manual_seed(rows + inter)
    x = torch.randn(rows, width, generator=gen).bfloat16()
    w = (torch.randn(2 * inter, width, generator=gen) / width**0.5).bfloat16()
    bias = torch.randn(2 * inter, generator=gen)
    got = ops.gemm_bf16_swiglu(x.to(DEV), w.to(DEV), activation="gelu_tanh", bias=bias.to(DEV))
    assert got is not None
    z = bf16_round(x.float() @ w.float().T).double() + bias.double()  # the products are rounded before the activation
    torch.testing.assert_close(got.double().cpu(), pp.gelu_tanh(z[:, :inter]) * z[:, inter:], rtol=2e-2, atol=2e-2)


@pytest.mark.parametrize("rows,narrow,wide", [(1, 80, 20), (16, 144, 36), (17, 80, 20), (100, 160, 3), (300, 80, 41), (8, 6272, 144)])
def test_product_whose_last_columns_stay_float32(rows, narrow, wide):
    ops = _ops()
    x, w = torch.randn(rows, 256).bfloat16(), torch.randn(narrow + wide, 256).bfloat16()
    a, b = ops.gemm_bf16_split(x.to(DEV), w.to(DEV), narrow)
    want = x.double() @ w.double().T
    assert a.dtype == torch.bfloat16 and b.dtype == torch.float32 and a.is_contiguous() and b.is_contiguous()
    torch.testing.assert_close(a.double().cpu(), want[:, :narrow], rtol=1e-2, atol=1e-2)
    torch.testing.assert_close(b.double().cpu(), want[:, narrow:], rtol=1e-5, atol=1e-4)
    # columns of a wider row as the left operand
    part = torch.randn(rows, 64 + 40).bfloat16().to(DEV)[:, 40:]
    v = torch.randn(48, 64).bfloat16().to(DEV)
    got = ops.gemm_bf16(part, v, torch.bfloat16)
    torch.testing.assert_close(got.double().cpu(), part.double().cpu() @ v.double().cpu().T, rtol=1e-2, atol=1e-1)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rows", [3, 16, 40, 150, 400])
@pytest.mark.parametrize("width", [512, 100])
def test_a_biased_product_joins_the_stream_in_the_next_norm(dtype, rows, width):
    """Whatever kernel adds a feed-forward's last product to the stream (few rows, runs of K, the plain
    norm) adds its bias; the norm's weights are stored around zero."""
    from rapid_llm_amd.parts.linear import Linear
    from rapid_llm_amd.parts.norm import RMSNorm

    t = getattr(torch, dtype)
    gen = torch.Generator().manual_seed(rows)
    k = 1024
    x = torch.randn(rows, k, generator=gen).to(t)
    w = (torch.randn(width, k, generator=gen) / k**0.5).to(t)
    bias, weight = torch.randn(width, generator=gen), 0.2 * torch.randn(width, generator=gen)
    residual = torch.randn(rows, width, generator=gen)
    linear, norm = Linear(k, width), RMSNorm(width, 1e-5, "n", weight_offset=1.0)
    linear.bind(w.to(DEV), bias.to(DEV))
    norm.bind({"norm.weight": weight.to(DEV)}, SimpleNamespace(dtype=t, device=DEV))
    stream = residual.double() + x.double() @ w.double().T + bias.double()
    want = pp.around_one_norm(stream, weight.double(), 1e-5)
    tol = _tol(t, 2e-5, 2e-2)
    for rows_of in (None, torch.tensor([rows - 1, 0], dtype=torch.int32, device=DEV)):
        res = residual.clone().to(DEV)
        y = norm.forward(res, linear.deferred(x.to(DEV)), None, rows_of)
        pick = slice(None) if rows_of is None else rows_of.long().cpu()
        torch.testing.assert_close(y.double().cpu(), want[pick], **tol)
        torch.testing.assert_close(res.double().cpu()[pick], stream[pick], **tol)
    if dtype == "bfloat16" and rows <= 16:
        res = residual.clone().to(DEV)
        scaled = norm.forward(res, linear.deferred(x.to(DEV)), None, None, scaled_ok=True)
        assert not isinstance(scaled, torch.Tensor)
        torch.testing.assert_close(res.double().cpu(), stream, **tol)
        torch.testing.assert_close(scaled.rows.double().cpu(), stream * (1.0 + weight.double()), **tol)


@pytest.mark.parametrize("width", [96, 100, 7])
def test_what_a_pass_begins_with(width):
    ops = _ops()
    residual, first, row = torch.randn(9, width), torch.randn(9, width), torch.randn(width)
    for f, r in ((first, row), (first, None), (None, row)):
        got = residual.clone().to(DEV)
        ops.stream_add(got, None if f is None else f.to(DEV), None if r is None else r.to(DEV))
        want = residual + (0 if f is None else f) + (0 if r is None else r)
        torch.testing.assert_close(got.cpu(), want, rtol=1e-6, atol=1e-6)


# --------------------------------------------------------------------------- #
# attention: heads as they are cached, and the distance term
# --------------------------------------------------------------------------- #


@TYPES
@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 16, 32), (6, 3, 12, 10), (3, 1, 9, 22), (4, 1, 64, 48), (2, 2, 160, 200)])
@pytest.mark.parametrize("tokens", [1, 5, 40])
def test_heads_are_normed_biased_and_tempered_on_their_way(dtype, H, G, d, dv, tokens):
    """Biases, the query and key norms, the temperature of the queries and the norm of the values, from
    columns in the middle of a packed row, into queries and cache pages."""
    ops = _ops()
    gen = torch.Generator().manual_seed(H * 100 + d + tokens)
    own = H * d + G * (d + dv)
    col0, page, eps, coef, every = 16, 8, 1e-5, 0.4, 7.0
    width = col0 + own + (-(col0 + own)) % 8 + 8
    packed = torch.randn(tokens, width, generator=gen).to(dtype)
    bias = torch.randn(own + 3, generator=gen)
    qn, kn = 1.0 + 0.3 * torch.randn(d, generator=gen), 1.0 + 0.3 * torch.randn(d, generator=gen)
    start = 5
    positions = torch.arange(start, start + tokens, dtype=torch.int32)
    pages = -(-(start + tokens) // page)
    order = torch.randperm(pages, generator=gen) + 1
    table = torch.zeros((2, pages), dtype=torch.int32)
    table[1] = order.int()
    kc = torch.zeros((pages + 1, G, page, d), dtype=dtype, device=DEV)
    vc = torch.zeros((pages + 1, G, dv, page), dtype=dtype, device=DEV)
    q = torch.empty((tokens, H * d), dtype=dtype, device=DEV)
    ops.qknorm_rope_kvwrite(
        packed.to(DEV), q, kc, vc, qn.to(DEV), kn.to(DEV), None, None, positions.to(DEV),
        torch.ones(tokens, dtype=torch.int32, device=DEV), table.to(DEV), page, H, G, d, eps, int(positions[-1]),
        bias=bias.to(DEV), value_dim=dv, col0=col0, query_temperature=(coef, every), norm_values=True)
    x = packed[:, col0 : col0 + own].double() + bias[:own].double()
    want_q = pp.rms(x[:, : H * d].view(tokens, H, d), eps) * qn.double()
    want_q = want_q * pp.temperature(positions, coef, every).view(tokens, 1, 1)
    want_k = pp.rms(x[:, H * d : (H + G) * d].view(tokens, G, d), eps) * kn.double()
    want_v = pp.rms(x[:, (H + G) * d :].view(tokens, G, dv), eps)
    tol = _tol(dtype, 1e-5, 1e-2)
    torch.testing.assert_close(q.double().cpu().view(tokens, H, d), want_q, **tol)
    for t, p in enumerate(positions.tolist()):
        pid = int(order[p // page])
        torch.testing.assert_close(kc[pid, :, p % page].double().cpu(), want_k[t], **tol)
        torch.testing.assert_close(vc[pid, :, :, p % page].double().cpu(), want_v[t], **tol)


def _attention_oracle(q, k, v, scale, r1, r2, first_row):
    """The last ``q.shape[0]`` positions of one request: ``q [n, H, d]``, ``k [t, G, d]``, ``v [t, G, dv]``."""
    t, n, H, G = k.shape[0], q.shape[0], q.shape[1], k.shape[1]
    i, j = torch.arange(first_row, first_row + n).view(n, 1), torch.arange(t).view(1, t)
    out = torch.zeros(n, H, v.shape[2], dtype=D64)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h].double() @ k[:, g].double().T) * scale
        s = s - r1[h].double() * torch.log(1.0 + r2[h].double() * (i - j).clamp(min=0))
        out[:, h] = torch.softmax(s.masked_fill(j > i, -math.inf), 1) @ v[:, g].double()
    return out.reshape(n, -1)


def _paged(seqs, H, G, d, dv, page, dtype, seed, scale, r1, r2, spike=None):
    """``seqs`` = (tokens already cached, tokens of this step) per request, on shuffled pages and
    slots; unwritten slots of a page are NaN."""
    rng = random.Random(seed)
    gen = torch.Generator().manual_seed(seed)
    total = sum(-(-(a + n) // page) for a, n in seqs) + 1
    free = list(range(1, total))
    rng.shuffle(free)
    table = torch.zeros((len(seqs) + 2, max(-(-(a + n) // page) for a, n in seqs) + 1), dtype=torch.int32)
    kc, vc = torch.full((total, G, page, d), float("nan")), torch.full((total, G, dv, page), float("nan"))
    slots = list(range(len(seqs) + 2))
    rng.shuffle(slots)
    rows, positions, token_slot, want = [], [], [], []
    for i, (a, n) in enumerate(seqs):
        t = a + n
        k, v, q = torch.randn(t, G, d, generator=gen), torch.randn(t, G, dv, generator=gen), torch.randn(n, H, d, generator=gen)
        k, q = (x / x.square().mean(-1, keepdim=True).sqrt() for x in (k, q))  # as the head norm leaves them
        if spike is not None and spike[0] == i:
            # one key matches the request's last query in every head, far beyond every other score
            q[-1] = q[-1, 0]
            k[spike[1]] = q[-1, 0] * 6.0
            v[spike[1]] = 7.0
        if dtype == torch.bfloat16:
            q, k, v = (x.bfloat16().float() for x in (q, k, v))
        for p in range(-(-t // page)):
            pid = free.pop()
            table[slots[i], p] = pid
            lo, hi = p * page, min(t, (p + 1) * page)
            kc[pid, :, : hi - lo] = k[lo:hi].transpose(0, 1)
            vc[pid, :, :, : hi - lo] = v[lo:hi].permute(1, 2, 0)
        want.append(_attention_oracle(q, k, v, scale, r1, r2, a))
        rows.append(q.reshape(n, H * d))
        positions += list(range(a, t))
        token_slot += [slots[i]] * n
    ctx = SimpleNamespace(
        positions=torch.tensor(positions, dtype=torch.int32, device=DEV),
        token_slot=torch.tensor(token_slot, dtype=torch.int32, device=DEV),
        token_ids=torch.zeros(len(positions), dtype=torch.int32, device=DEV),
        h_seq_starts=[a for a, _ in seqs], h_seq_lens=[n for _, n in seqs], max_position=max(positions), extra={},
    )
    return torch.cat(rows).to(DEV, dtype), kc.to(DEV, dtype), vc.to(DEV, dtype), table.to(DEV), ctx, torch.cat(want)


def _run_attention(case, dtype, spike=None, seed=5, out_scale=1.0):
    ops = _ops()
    H, G, d, dv, page, seqs = case
    gen = torch.Generator().manual_seed(seed)
    r1, r2 = 0.3 + torch.rand(H, generator=gen), 0.05 + 0.6 * torch.rand(H, generator=gen)
    scale = 3.0 / d  # heads of unit root mean square: |q . k| <= d
    q, kc, vc, table, ctx, want = _paged(seqs, H, G, d, dv, page, dtype, seed, scale, r1, r2, spike)
    before = 8 if dv % 2 == 0 else 3
    out = torch.full((q.shape[0], before + H * dv + (-(before + H * dv)) % 4 + 4), float("nan"), dtype=dtype, device=DEV)
    ops.paged_attention(q, kc, vc, out, ctx, table, page, H, G, d, 0, scale, value_dim=dv,
                        log_distance=(r1.to(DEV), r2.to(DEV)), out_col=before, out_scale=out_scale)
    assert torch.isnan(out[:, :before]).all() and torch.isnan(out[:, before + H * dv :]).all()
    return out[:, before : before + H * dv].double().cpu(), want * out_scale


ATTENTION_CASES = [
    # H, G, d, dv, page, (cached, new) per request
    (4, 2, 16, 32, 8, [(0, 60), (45, 1), (200, 1), (30, 31), (0, 1), (18, 1), (19, 2)]),
    (6, 3, 12, 10, 8, [(0, 50), (32, 1), (33, 1), (100, 2)]),          # sizes off the grid of 16
    (3, 1, 9, 22, 4, [(0, 30), (8, 1), (9, 1), (50, 1)]),
    (8, 2, 64, 32, 16, [(300, 1), (5, 70), (0, 2), (69, 1), (70, 1)]),
    (1, 1, 16, 16, 4, [(0, 40), (120, 1), (39, 3)]),
    (4, 1, 128, 64, 16, [(2000, 1), (590, 30), (0, 700)]),             # long contexts
    (2, 2, 64, 128, 16, [(1500, 1), (1024, 1)]),                       # a step of single tokens: keys dealt to workgroups
    (5, 1, 13, 7, 16, [(10, 1), (0, 17)]),                             # odd value heads
]


@pytest.mark.parametrize("case", ATTENTION_CASES, ids=lambda c: f"h{c[0]}kv{c[1]}d{c[2]}v{c[3]}p{c[4]}")
@TYPES
def test_attention_with_a_logarithmic_distance_term(case, dtype):
    got, want = _run_attention(case, dtype, out_scale=0.6)
    torch.testing.assert_close(got, want, **_tol(dtype, 2e-5, 3e-2))


@TYPES
@pytest.mark.parametrize("d,dv,page", [(64, 32, 16), (16, 32, 8), (24, 10, 8)])
def test_one_key_holds_the_mass_wherever_it_lies(dtype, d, dv, page):
    """The last query's weight lies on one key: the request's first, the first and last of a page, the
    query's own; in a prompt's portion and decoded alone.  The value of that key is 7 in every
    channel, every other value is of order one."""
    H, G = 4, 2
    for cached, new in ((100, 1), (70, 31), (0, 101)):
        last = cached + new - 1
        for far in (0, 1, last, last - 1, last - last % page, last - last % page - 1, page - 1, page, 16, 15):
            case = (H, G, d, dv, page, [(3, 2), (cached, new), (50, 1)])
            got, want = _run_attention(case, dtype, spike=(1, far), seed=far + 3)
            torch.testing.assert_close(got, want, **_tol(dtype, 3e-5, 4e-2))
            assert float(got[2 + new - 1].min()) > 6.0, (cached, new, far)


# --------------------------------------------------------------------------- #
# the model through the engine's step function
# --------------------------------------------------------------------------- #
LENGTHS = {
    "A": [1, 2, 3, 6, 7, 8, 9, 17, 57, 130],  # the first tokens; around steps of the temperature and pages of 8
    "B": [1, 2, 4, 5, 9, 33, 80],
    "C": [1, 2, 8, 9, 10, 34, 90],
    "D": [2, 15, 16, 17, 20, 70, 150],
    "E": [1, 2, 16, 17, 40],
}


def _requests(which):
    cfg, _page, seed = PEFU[which]
    return {f"q{i}": random_tokens(n, cfg["vocab"], seed * 100 + i) for i, n in enumerate(LENGTHS[which])}


def _oracles(pcfg, pw, requests):
    """Per request the plain logits in float64, and what rounding alone does to the worst row of the
    plain implementation with rounded activations."""
    want = {rid: pp.forward(pcfg, pw, toks) for rid, toks in requests.items()}
    order = sorted(want)
    rounded = torch.cat([pp.forward(pcfg, pw, requests[r], cast=bf16_round) for r in order])
    return want, float(row_errors(rounded, torch.cat([want[r] for r in order])).max())


def _runner(model_dir, dtype, page, num_pages, max_seq_len, slots=4):
    from rapid_llm_amd import EngineConfig, ModelRunner

    runner = ModelRunner(
        model_dir,
        EngineConfig(dtype=dtype, max_seq_len=max_seq_len, page_size=page, num_pages=num_pages,
                     max_num_seqs=slots, use_graph=False),
    )
    for layer in runner.device_cache.layers:  # whatever is read before it is written shows
        for t in layer.pages.values() if layer.owns_pages else ():
            t.fill_(float("nan"))
    return runner


def _check(got, want, dtype, label, rounding=None):
    bound = F32_ROW if dtype == "float32" else BF16_TIMES_ROUNDING * rounding
    order = sorted(want)
    spread = float(torch.cat([want[r] for r in order]).double().std())
    worst = 0.0
    for rid in order:
        assert got[rid].shape == want[rid].shape and torch.isfinite(got[rid]).all(), (label, rid)
        rows = (got[rid].double() - want[rid].double()).square().mean(dim=1).sqrt() / spread
        worst = max(worst, float(rows.max()))
        bad = rows > bound
        assert not bad.any(), (
            f"{label}: request {rid}, first wrong position {int(torch.nonzero(bad)[0])}, "
            f"worst row {float(rows.max()):.3e} of the spread, bound {bound:.3e}"
        )
    if dtype == "bfloat16":
        parity.record(label, worst, worst)


@pytest.mark.parametrize("which", ["A", "B", "C", "D", "E"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_every_cut_matches_plain(tmp_path, which, dtype):
    cfg, page, seed = PEFU[which]
    model_dir = make_model_dir(tmp_path, which, sharp=3.0)
    pcfg, pw = load_plain(model_dir)
    requests = _requests(which)
    want, rounding = _oracles(pcfg, pw, requests)
    longest = max(LENGTHS[which])
    schedules = {
        "whole": ru.whole(requests),
        "decode": ru.prefill_then_decode(requests, 50),
        "token_by_token": ru.prefill_then_decode(requests, 10 ** 6),
        "portions": ru.changing_portions(requests),
        "portions_of_two": ru.changing_portions(requests, sizes=(2, 2, 3, 2, 64, 2)),
        "mixed": ru.mixed(requests, seed, max_tokens=None),
        "mixed_tight": ru.mixed(requests, seed + 1, max_tokens=2 * 64 * ((longest + 63) // 64)),
    }
    first = None
    for label, steps in schedules.items():
        pages = ru.pages_for(steps, requests, page) + 1
        runner = _runner(model_dir, dtype, page, pages + 1, longest + 8)
        got = ru.run_in_process(runner, steps)
        _check(got, want, dtype, f"{which}/{dtype}/{label}", rounding)
        if dtype == "float32":
            # one order of summation however the requests are cut: the same bits
            if first is None:
                first = got
            else:
                for rid in got:
                    assert torch.equal(got[rid], first[rid]), (label, rid)
        runner.cache.check_invariants()
        assert not runner.cache.live_requests()
        del runner


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_batch_of_unequal_requests_equals_each_alone(tmp_path, dtype):
    """One step holds a long prompt, a short one, a single first token and decoded tokens of two
    requests at different depths; every row equals the row of the request run alone."""
    which = "A"
    cfg, page, seed = PEFU[which]
    model_dir = make_model_dir(tmp_path, which, sharp=3.0)
    requests = {f"u{i}": random_tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate((90, 5, 1, 61, 30))}
    runner = _runner(model_dir, dtype, page, 60, 100, slots=5)
    alone = ru.run_in_process(runner, ru.whole(requests))
    full = lambda r, a, b: {"id": r, "tokens": requests[r][a:b], "want": list(range(b - a))}  # noqa: E731
    steps = [
        {"step": 0, "entries": [full("u3", 0, 60), full("u4", 0, 29)], "end": []},
        {"step": 1, "entries": [full("u0", 0, 90), full("u3", 60, 61), full("u1", 0, 5), full("u2", 0, 1), full("u4", 29, 30)],
         "end": ["u0", "u1", "u2", "u3", "u4"]},
    ]
    got = ru.run_in_process(runner, steps)
    for rid in requests:
        if dtype == "float32":
            assert torch.equal(got[rid], alone[rid]), rid
        else:
            assert float(row_errors(got[rid], alone[rid]).max()) < 0.08, rid
    runner.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_and_slots_used_again(tmp_path, dtype):
    """Five requests through two slots, each a short prompt and then 200 tokens one by one, two at a
    time in a step: pages come back and are taken again, and a later request finds the states of its
    slot zeroed."""
    which = "A"
    cfg, page, seed = PEFU[which]
    model_dir = make_model_dir(tmp_path, which, sharp=3.0)
    pcfg, pw = load_plain(model_dir)
    requests = {f"d{i}": random_tokens(200 + 7 * i, cfg["vocab"], 40 + i) for i in range(5)}
    want, rounding = _oracles(pcfg, pw, requests)
    steps = ru.mixed(requests, 3, max_live=2, tail=195)
    runner = _runner(model_dir, dtype, page, 2 * (-(-240 // page) + 1) + 2, 240, slots=2)
    got = ru.run_in_process(runner, steps)
    _check(got, want, dtype, f"long decoding/{dtype}", rounding)
    runner.cache.check_invariants()


def test_a_far_token_still_counts(tmp_path):
    """A different first token changes the logits 150 positions later, alike whether the tokens in
    between came in one prompt or one by one."""
    which = "A"
    cfg, page, seed = PEFU[which]
    model_dir = make_model_dir(tmp_path, which)
    pcfg, pw = load_plain(model_dir)
    toks = random_tokens(150, cfg["vocab"], 12)
    other = [(toks[0] + 1) % cfg["vocab"]] + toks[1:]
    want = {"same": pp.forward(pcfg, pw, toks), "other": pp.forward(pcfg, pw, other)}
    assert float(row_errors(want["other"][-1:], want["same"][-1:]).max()) > 50 * F32_ROW
    for steps_of in (ru.whole, lambda r: ru.prefill_then_decode(r, 140)):
        runner = _runner(model_dir, "float32", page, 60, 160)
        got = ru.run_in_process(runner, steps_of({"same": toks, "other": other}))
        _check(got, want, "float32", "far token")


def test_trace_program(tmp_path):
    """``bin/trace_run`` as a child process on a mixed trace over a tight pool."""
    which = "B"
    cfg, page, seed = PEFU[which]
    model_dir = make_model_dir(tmp_path, which, sharp=3.0)
    pcfg, pw = load_plain(model_dir)
    requests = _requests(which)
    want, _rounding = _oracles(pcfg, pw, requests)
    steps = ru.mixed(requests, seed + 5, max_tokens=256)
    got = ru.run_trace_program(model_dir, "float32", steps, tmp_path / "out", 256, cfg["vocab"])
    _check(got, want, "float32", "trace_run")


@pytest.mark.parametrize("use_graph", [False, True])
@pytest.mark.parametrize("which,dtype", [("A", "float32"), ("C", "float32"), ("D", "bfloat16"), ("E", "float32")])
def test_greedy_generation_through_the_entry_point(tmp_path, which, dtype, use_graph):
    """``LLM.generate``: scheduler, chunked prompts beside decoding requests, sampling kernels;
    decode steps eagerly and replayed from graphs.  The plain implementation re-runs the whole
    sequence for every token; a bfloat16 engine may pick another of several nearly equal maxima."""
    from rapid_llm_amd import LLM, SamplingParams

    cfg, page, seed = PEFU[which]
    model_dir = make_model_dir(tmp_path, which)
    pcfg, pw = load_plain(model_dir)
    prompts = [random_tokens(n, cfg["vocab"], seed + n) for n in (1, 7, 30, 45)]
    llm = LLM(str(model_dir), dtype=dtype, page_size=page, num_pages=60, max_num_seqs=3, max_seq_len=96,
              max_chunk_size=16, max_num_batched_tokens=32, use_cuda_graph=use_graph)
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_gen_len=24))
    gap = 1e-3 if dtype == "float32" else 0.15
    for prompt, out in zip(prompts, outs):
        ids = list(prompt)
        for tok in out.token_ids:
            logits = pp.forward(pcfg, pw, ids)[-1]
            scale = 1.0 if dtype == "float32" else float(logits.std())
            assert float(logits.max() - logits[tok]) <= gap * scale, (len(prompt), len(ids))
            ids.append(tok)
        assert len(out.token_ids) == 24
    llm.scheduler.cache.check_invariants()
    assert not llm.scheduler.cache.live_requests()
