"""The Renitar decoder in the engine against the plain implementation of ``plain_renitar.py``:
every mechanism alone, every way of cutting requests into steps, state slots and pages that are
used again, keys at the edges of chunks and pages, long decoding, and greedy generation through the
entry point."""

import math
import random
from types import SimpleNamespace

import pytest
import torch

import parity
import plain_renitar as pr
import replay_util as ru
from renitar_configs import (
    BF16_ROWS_BEYOND,
    BF16_TIMES_ROUNDING,
    RENI,
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


def _step(lens, slots, starts=None, **more):
    """What the kernels read of a step: the requests' offsets, slots and positions."""
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    starts = [0] * len(lens) if starts is None else starts
    positions = [a + i for a, n in zip(starts, lens) for i in range(n)]
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)  # noqa: E731
    return SimpleNamespace(
        cu_seqlens=i32(cu), seq_slots=i32(slots), num_seqs=len(lens), h_seq_lens=list(lens), h_seq_slots=list(slots),
        h_seq_starts=list(starts), positions=i32(positions), max_position=max(positions), extra={}, static={},
        token_slot=i32([s for s, n in zip(slots, lens) for _ in range(n)]), token_ids=i32([0] * cu[-1]), **more,
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
        ctx = _step([b - a for _r, a, b in now], [slots[r] for r, _a, _b in now], [a for _r, a, _b in now])
        rows = run(ctx, now)
        at = 0
        for r, a, b in now:
            got[r].append(rows[at : at + b - a].double().cpu())
            at += b - a
        live = [r for r in live if cuts[r]]
    return {r: torch.cat(parts) for r, parts in got.items()}


# four requests in portions down to one token, on shuffled slots of which one is taken again
LENGTHS_OP = {"a": 75, "b": 5, "c": 64, "d": 19}
SIZES_OP = {"a": (7, 1, 2, 1, 1, 16, 17), "b": (2, 1, 2), "c": (1, 1, 32, 2), "d": (19,)}
SLOTS_OP = {"a": 3, "b": 0, "c": 1, "d": 0}


# --------------------------------------------------------------------------- #
# linear attention
# --------------------------------------------------------------------------- #
LINEAR_SHAPES = [  # heads, key channels, value channels
    (3, 24, 16), (2, 16, 48), (1, 1, 1), (5, 20, 13), (2, 64, 128), (2, 128, 64), (1, 160, 80), (1, 250, 33), (2, 33, 300), (1, 17, 512),
]


@TYPES
@pytest.mark.parametrize("kind", ["channel", "fixed"])
@pytest.mark.parametrize("heads,d,dv", LINEAR_SHAPES)
def test_linear_attention_continues_from_the_slot(dtype, kind, heads, d, dv):
    """Decays, memory, norm and gate from columns in the middle of a packed row into columns of a wider one; the
    gates of a head as silu with the norm a head, of the row as sigmoid with the norm over the row."""
    ops = _ops()
    gen = torch.Generator().manual_seed(heads * 1000 + d * 10 + dv)
    keys, inner, rank, tau, eps = heads * d, heads * dv, 7, 3.0, 1e-5
    cols = (5, 5 + keys, 5 + 2 * keys + inner, 5 + 2 * keys)  # q, k, v and the gate: in another order than the product's
    width = 5 + 2 * keys + 2 * inner + 3
    a2, bias = torch.randn(keys, rank, generator=gen) / rank**0.5, torch.randn(keys, generator=gen) * 2.5 + 1.0
    decays = [0.02, 1.0, 0.9, 0.6, 0.99][:heads]
    norm_w = 1.0 + 0.2 * torch.randn(dv if kind == "channel" else inner, generator=gen)
    data, want = {}, {}
    for rid, T in LENGTHS_OP.items():
        packed = torch.randn(T, width, generator=gen).to(dtype).float()
        low = torch.randn(T, rank + 2, generator=gen)
        data[rid] = (packed, low)
        x = packed.double()
        q, k = (x[:, c : c + keys].view(T, heads, d) for c in cols[:2])
        v, g = x[:, cols[2] : cols[2] + inner].view(T, heads, dv), x[:, cols[3] : cols[3] + inner]
        if kind == "channel":
            z = low[:, :rank].double() @ a2.double().T + bias.double()
            o = pr.decayed_memory(q * d**-0.5, k, v, pr.channel_decay(z.view(T, heads, d), tau))
            want[rid] = (pr.rms(o, eps) * norm_w.double()).reshape(T, inner) * pr.silu(g)
        else:
            o = pr.decayed_memory(pr.silu(q), pr.silu(k), pr.silu(v), torch.tensor(decays, dtype=D64).view(1, heads, 1))
            want[rid] = pr.rms(o.reshape(T, inner), eps) * norm_w.double() * torch.sigmoid(g)
    S = torch.full((5, heads, d, dv), float("nan"), device=DEV)
    out_t, log_decay = a2.T.contiguous().to(DEV), torch.tensor([math.log(a) for a in decays], dtype=torch.float32, device=DEV)

    def run(ctx, now):
        packed, low = (torch.cat([data[r][i][a:b] for r, a, b in now]).to(DEV) for i in range(2))
        out = torch.full((packed.shape[0], inner + 9), float("nan"), dtype=dtype, device=DEV)
        if kind == "channel":
            decay, more = ops.ChannelDecay(low, out_t, bias.to(DEV), tau), (d**-0.5, False, heads, "silu")
        else:
            decay, more = ops.FixedDecay(log_decay), (1.0, True, 1, "sigmoid")
        ops.linear_attention(packed.to(dtype), cols, decay, norm_w.to(DEV), out, ctx, S, heads, d, dv, *more, eps, out_col=4)
        assert torch.isnan(out[:, :4]).all() and torch.isnan(out[:, 4 + inner :]).all()
        return out[:, 4 : 4 + inner]

    got = _interleaved(LENGTHS_OP, SIZES_OP, SLOTS_OP, [S], run)
    for rid in LENGTHS_OP:
        torch.testing.assert_close(got[rid], want[rid], **_tol(dtype, 1e-4, 3e-2))


@TYPES
def test_linear_attention_far_and_fast(dtype):
    """Decays from 1 (a first token that is never forgotten) to e^-60 a token, side by side in one head, over
    600 tokens: nothing overflows, nothing is lost, portions and single tokens agree."""
    ops = _ops()
    T, d, dv, tau = 600, 32, 32, 1.0
    gen = torch.Generator().manual_seed(3)
    packed = torch.randn(T, 2 * d + 2 * dv, generator=gen) * 0.3
    packed[0, d : 2 * d] = 4.0  # the first key and value stand out
    packed[0, 2 * d : 2 * d + dv] = 4.0
    packed = packed.to(dtype).float()
    bias = torch.linspace(-60.0, 40.0, d)  # sigmoid(40) is 1 to 4e-18
    low, out_t, nw = torch.zeros(T, 1), torch.zeros(1, d), torch.ones(dv)
    x = packed.double()
    q, k, v = x[:, :d].view(T, 1, d), x[:, d : 2 * d].view(T, 1, d), x[:, 2 * d : 2 * d + dv].view(T, 1, dv)
    o = pr.decayed_memory(q, k, v, pr.channel_decay(bias.double().view(1, 1, d), tau))
    want = pr.rms(o, 1e-6).reshape(T, dv) * torch.sigmoid(x[:, 2 * d + dv :])
    assert float((pr.rms(pr.decayed_memory(q[1:], k[1:], v[1:], pr.channel_decay(bias.double().view(1, 1, d), tau)), 1e-6)[-1]
                  - pr.rms(o, 1e-6)[-1]).abs().max()) > 0.3  # the first token still counts at the end
    for sizes in ((T,), (1,), (31, 2, 1), (16,)):
        S = torch.zeros(1, 1, d, dv, device=DEV)
        rows = []
        for a, b in _cuts(T, sizes):
            out = torch.empty((b - a, dv), dtype=dtype, device=DEV)
            decay = ops.ChannelDecay(low[a:b].to(DEV), out_t.to(DEV), bias.to(DEV), tau)
            ops.linear_attention(packed[a:b].to(DEV, dtype), (0, d, 2 * d, 2 * d + dv), decay, nw.to(DEV), out, _step([b - a], [0]), S,
                                 1, d, dv, 1.0, False, 1, "sigmoid", 1e-6)
            rows.append(out.double().cpu())
        torch.testing.assert_close(torch.cat(rows), want, **_tol(dtype, 2e-4, 3e-2))


@TYPES
@pytest.mark.parametrize("heads,dv", [(4, 128), (16, 128), (3, 20), (1, 4096), (5, 13), (1, 1000)])
def test_gated_norm_of_many_rows(dtype, heads, dv):
    """The finishing kernels over steps of portions: parts narrower and wider than a wave, the whole row."""
    ops = _ops()
    tokens, eps = 37, 1e-5
    raw = torch.randn(tokens, heads * dv) * 3
    gate = torch.randn(tokens, heads * dv + 8).to(dtype)
    lib = ops.linear_attention_lib()
    for parts, shared, sig in ((heads, True, 0), (1, True, 1), (heads, False, 1)):
        size = heads * dv // parts
        w = 1.0 + 0.3 * torch.randn(size if shared else heads * dv)
        out = torch.full((tokens, heads * dv + 8), float("nan"), dtype=dtype, device=DEV)
        r, g, wd = raw.to(DEV), gate.to(DEV), w.to(DEV)
        import ctypes

        code = lib.rl_gated_norm(ops._p(r), ops._p(g), g.shape[1], 8, ops._p(wd), int(shared), sig, ctypes.c_float(eps), ops._p(out),
                                 out.shape[1], tokens, parts, size, ops._tag(dtype), ops._stream())
        assert code == 0
        z = gate[:, 8:].double()
        want = pr.rms(raw.double().view(tokens, parts, size), eps) * (w.double() if shared else w.double().view(parts, size))
        want = want.reshape(tokens, -1) * torch.sigmoid(z) * (1.0 if sig else z)
        torch.testing.assert_close(out[:, : heads * dv].double().cpu(), want, **_tol(dtype, 1e-5, 2e-2))
        assert torch.isnan(out[:, heads * dv :]).all()


# --------------------------------------------------------------------------- #
# heads behind short convolutions
# --------------------------------------------------------------------------- #
HEAD_SHAPES = [  # H, G, d, dv, taps, rotated channels, pairing, page
    (4, 2, 16, 32, 3, 8, "half_split", 8), (6, 3, 12, 10, 5, 6, "half_split", 8), (1, 1, 16, 16, 1, 2, "half_split", 4),
    (8, 1, 64, 32, 7, 64, "half_split", 16), (16, 4, 128, 128, 4, 32, "half_split", 16), (3, 1, 22, 9, 4, 22, "half_split", 8),
    (2, 2, 64, 64, 4, 24, "interleaved", 16), (4, 2, 32, 16, 4, 12, "half_split", 16), (40, 8, 128, 64, 4, 128, "half_split", 16),
    (2, 1, 20, 12, 16, 0, "half_split", 4), (4, 4, 24, 24, 0, 8, "half_split", 8),
]


@TYPES
@pytest.mark.parametrize("shape", HEAD_SHAPES, ids=lambda s: f"h{s[0]}kv{s[1]}d{s[2]}v{s[3]}t{s[4]}r{s[5]}{s[6][0]}")
def test_convolved_heads_continue_from_the_slot(dtype, shape):
    """Bias, convolution, norm over all heads, rotation and cache write, from columns in the middle of a packed
    row, with portions shorter than the convolution's reach, on shuffled pages."""
    ops = _ops()
    H, G, d, dv, taps, rot, pairing, page = shape
    gen = torch.Generator().manual_seed(H * 100 + d + taps)
    qk, own, eps, base = (H + G) * d, (H + G) * d + G * dv, 1e-5, 100.0
    col0 = 8 if d % 4 == 0 and dv % 4 == 0 else 3
    width = col0 + own + (-(col0 + own)) % 8 + 8
    bias = torch.randn(own + 2, generator=gen) * 0.5
    w = torch.randn(own, taps, generator=gen) * 0.6 if taps else None
    qn, kn = 1.0 + 0.3 * torch.randn(H * d, generator=gen), 1.0 + 0.3 * torch.randn(G * d, generator=gen)
    longest = max(LENGTHS_OP.values())
    if rot:
        freq = base ** (-2.0 * torch.arange(rot // 2, dtype=D64) / rot)
        angle = torch.arange(longest, dtype=D64).view(-1, 1) * freq
        cos, sin = angle.cos().float().to(DEV), angle.sin().float().to(DEV)
    else:
        cos = sin = None

    def turned(x):
        if not rot:
            return x
        if pairing == "half_split":
            return pr.rotate(x, rot, base)
        y = x.clone()
        y[..., :rot] = torch.cat([x[..., 0:rot:2], x[..., 1:rot:2]], -1)
        y = pr.rotate(y, rot, base)
        z = y.clone()
        z[..., 0:rot:2], z[..., 1:rot:2] = y[..., : rot // 2], y[..., rot // 2 : rot]
        return z

    data, want = {}, {}
    for rid, T in LENGTHS_OP.items():
        packed = torch.randn(T, width, generator=gen).to(dtype).float()
        data[rid] = packed
        x = packed[:, col0 : col0 + own].double() + bias[:own].double()
        y = pr.short_convolution(x, w.double()) if taps else x
        q = turned((pr.rms(y[:, : H * d], eps) * qn.double()).view(T, H, d))
        k = turned((pr.rms(y[:, H * d : qk], eps) * kn.double()).view(T, G, d))
        want[rid] = torch.cat([q.reshape(T, -1), k.reshape(T, -1), y[:, qk:]], 1)
    per = -(-longest // page)
    order = torch.randperm(5 * per, generator=gen) + 1
    table = order.view(5, per).to(torch.int32)
    kc = torch.full((5 * per + 1, G, page, d), float("nan"), dtype=dtype, device=DEV)
    vc = torch.full((5 * per + 1, G, dv, page), float("nan"), dtype=dtype, device=DEV)
    state = torch.full((5, max(taps - 1, 1), own), float("nan"), device=DEV)
    taps_t = w.T.contiguous().to(DEV) if taps else None

    def run(ctx, now):
        packed = torch.cat([data[r][a:b] for r, a, b in now]).to(DEV, dtype)
        tokens = packed.shape[0]
        q = torch.full((tokens, H * d), float("nan"), dtype=dtype, device=DEV)
        ops.conv_heads(packed, col0, bias.to(DEV), taps_t, state if taps else None, qn.to(DEV), kn.to(DEV), eps, cos, sin, pairing,
                       q, kc, vc, ctx, table.to(DEV), page, H, G, d, dv)
        rows, at = [], 0
        for r, a, b in now:
            for p in range(a, b):
                pid = int(table[SLOTS_OP[r], p // page])
                rows.append(torch.cat([q[at], kc[pid, :, p % page].reshape(-1), vc[pid, :, :, p % page].reshape(-1)]))
                at += 1
        return torch.stack(rows)

    got = _interleaved(LENGTHS_OP, SIZES_OP, SLOTS_OP, [state], run)
    for rid in LENGTHS_OP:
        torch.testing.assert_close(got[rid], want[rid], **_tol(dtype, 3e-5, 2e-2))


# --------------------------------------------------------------------------- #
# attention in chunks
# --------------------------------------------------------------------------- #


def _chunk_oracle(q, k, v, scale, cap, chunk, gate, first_row):
    """The last ``q.shape[0]`` positions of one request: ``q [n, H, d]``, ``k [t, G, d]``, ``v [t, G, dv]``."""
    t, n, H, G = k.shape[0], q.shape[0], q.shape[1], k.shape[1]
    seen = pr.chunk_mask(t, chunk)[first_row : first_row + n]
    out = torch.zeros(n, H, v.shape[2], dtype=D64)
    for h in range(H):
        g = h // (H // G)
        s = pr.soft_cap((q[:, h].double() @ k[:, g].double().T) * scale, cap)
        out[:, h] = torch.softmax(s.masked_fill(~seen, -math.inf), 1) @ v[:, g].double()
    return out.reshape(n, -1) * torch.sigmoid(gate.double())


def _run_chunks(case, dtype, spike=None, seed=5):
    """``seqs`` = (tokens already cached, tokens of this step) per request, on shuffled pages and slots.  Pages of
    complete chunks are unmapped (their table entries are the null page), unwritten slots are NaN, and so are
    the null page's.  ``spike`` (request, position): the key that matches the request's last query."""
    ops = _ops()
    H, G, d, dv, page, chunk, seqs = case
    rng = random.Random(seed)
    gen = torch.Generator().manual_seed(seed)
    total = sum(-(-(a + n) // page) for a, n in seqs) + 1
    free = list(range(1, total))
    rng.shuffle(free)
    table = torch.zeros((len(seqs) + 2, max(-(-(a + n) // page) for a, n in seqs) + 1), dtype=torch.int32)
    kc, vc = torch.full((total, G, page, d), float("nan")), torch.full((total, G, dv, page), float("nan"))
    slots = list(range(len(seqs) + 2))
    rng.shuffle(slots)
    cap, scale = 20.0, 3.0 / d
    before = 8 if dv % 4 == 0 else 3
    width = before + H * dv + (-(before + H * dv)) % 4 + 4
    rows, gates, want = [], [], []
    for i, (a, n) in enumerate(seqs):
        t = a + n
        k, v, q = torch.randn(t, G, d, generator=gen), torch.randn(t, G, dv, generator=gen), torch.randn(n, H, d, generator=gen)
        k, q = (x / x.square().mean(-1, keepdim=True).sqrt() for x in (k, q))
        gate = torch.randn(n, width, generator=gen)
        if spike is not None and spike[0] == i:
            q[-1] = q[-1, 0]
            k[spike[1]] = q[-1, 0] * 6.0
            v[spike[1]] = 7.0
            gate[-1] = 3.0
        if dtype == torch.bfloat16:
            q, k, v, gate = (x.bfloat16().float() for x in (q, k, v, gate))
        for p in range(-(-t // page)):
            pid = free.pop()
            if (p + 1) * page <= a // chunk * chunk:
                continue  # given back: no query of this step reads it
            table[slots[i], p] = pid
            lo, hi = p * page, min(t, (p + 1) * page)
            kc[pid, :, : hi - lo] = k[lo:hi].transpose(0, 1)
            vc[pid, :, :, : hi - lo] = v[lo:hi].permute(1, 2, 0)
        want.append(_chunk_oracle(q, k, v, scale, cap, chunk, gate[:, before : before + H * dv], a))
        rows.append(q.reshape(n, H * d))
        gates.append(gate)
    ctx = _step([n for _, n in seqs], slots[: len(seqs)], [a for a, _ in seqs])
    out = torch.full((ctx.positions.numel(), width), float("nan"), dtype=dtype, device=DEV)
    ops.paged_attention(torch.cat(rows).to(DEV, dtype), kc.to(DEV, dtype), vc.to(DEV, dtype), out, ctx, table.to(DEV), page, H, G, d,
                        chunk, scale, value_dim=dv, score_cap=cap, out_col=before, chunked=True,
                        gate=(torch.cat(gates).to(DEV, dtype), before))
    assert torch.isnan(out[:, :before]).all() and torch.isnan(out[:, before + H * dv :]).all()
    return out[:, before : before + H * dv].double().cpu(), torch.cat(want)


CHUNK_CASES = [
    # H, G, d, dv, page, chunk, (cached, new) per request
    (4, 2, 16, 32, 8, 20, [(0, 60), (45, 1), (200, 1), (30, 31), (0, 1), (19, 1), (20, 1), (19, 2)]),
    (6, 3, 12, 10, 8, 33, [(0, 70), (32, 1), (33, 1), (100, 2)]),        # sizes off the grid of 16
    (8, 2, 64, 32, 16, 48, [(300, 1), (5, 90), (0, 2), (47, 1), (48, 1), (96, 49)]),
    (1, 1, 16, 16, 4, 1, [(0, 9), (120, 1), (39, 3)]),                    # every position a chunk of its own
    (4, 1, 128, 64, 16, 512, [(2000, 1), (500, 30), (0, 700)]),
    (2, 2, 64, 128, 16, 1000, [(1999, 1), (2000, 1), (1500, 1)]),         # single tokens: keys dealt to workgroups
    (2, 1, 32, 32, 16, 5, [(3, 60), (64, 1), (14, 1), (15, 1)]),          # chunks that cut pages and tiles
    (32, 1, 64, 64, 16, 100, [(199, 1), (150, 60)]),                      # more heads than a tile of rows holds
]


@pytest.mark.parametrize("case", CHUNK_CASES, ids=lambda c: f"h{c[0]}kv{c[1]}d{c[2]}v{c[3]}p{c[4]}c{c[5]}")
@TYPES
def test_attention_in_chunks_with_cap_and_gate(case, dtype):
    got, want = _run_chunks(case, dtype)
    torch.testing.assert_close(got, want, **_tol(dtype, 2e-5, 3e-2))


@TYPES
@pytest.mark.parametrize("d,dv,page,chunk", [(64, 32, 16, 24), (16, 32, 8, 20), (24, 10, 8, 30), (32, 32, 16, 48)])
def test_one_key_just_inside_and_just_outside_a_chunk(dtype, d, dv, page, chunk):
    """One key matches the last query far beyond every other.  Inside the query's chunk it holds the mass (its
    value is 7 in every channel); one position before the chunk's first it must not be seen at all."""
    H, G = 4, 2
    gate = 1.0 / (1.0 + math.exp(-3.0))
    for cached, new in ((4 * chunk - 1, 1), (4 * chunk, 1), (4 * chunk + 5, 1), (2 * chunk - 3, 2 * chunk), (0, 3 * chunk - 1), (0, 3 * chunk + 2)):
        last = cached + new - 1
        edge = last // chunk * chunk  # the chunk's first position
        for far, inside in ((edge, True), (last, True), (edge - 1, False), (edge - chunk, False), (0, False)):
            case = (H, G, d, dv, page, chunk, [(3, 2), (cached, new), (50, 1)])
            got, want = _run_chunks(case, dtype, spike=(1, far), seed=far + 3)
            torch.testing.assert_close(got, want, **_tol(dtype, 3e-5, 4e-2))
            row = got[2 + new - 1]
            if inside:
                assert float(row.min()) > 6.0 * gate, (cached, new, far)
            else:
                assert float(row.max()) < 5.0, (cached, new, far)


# --------------------------------------------------------------------------- #
# experts, the layer's sum
# --------------------------------------------------------------------------- #


# (a router matrix of bfloat16 meets rows of bfloat16)
@pytest.mark.parametrize("dtype,weights_as", [(torch.float32, "f32"), (torch.bfloat16, "f32"), (torch.bfloat16, "bf16")],
                         ids=["f32", "bf16-f32", "bf16"])
@pytest.mark.parametrize("tokens,k,experts,identity,top,gate", [
    (1, 96, 6, 3, 2, True), (40, 100, 7, 2, 4, True), (17, 64, 1, 0, 1, False), (8, 2048, 16, 4, 3, True), (33, 256, 60, 30, 8, True),
    (5, 50, 200, 100, 20, False), (16, 128, 1000, 24, 5, True), (3, 7, 3, 1, 4, True),
])
def test_experts_chosen_by_corrected_scores(dtype, weights_as, tokens, k, experts, identity, top, gate):
    ops = _ops()
    gen = torch.Generator().manual_seed(k + experts)
    choices = experts + identity
    x = torch.randn(tokens, k, generator=gen).to(dtype)
    w = (torch.randn(choices + int(gate), k, generator=gen) * 2.0 / k**0.5).bfloat16().float()
    correction = torch.randn(choices, generator=gen) * 0.3 / choices
    got = ops.choose_experts(x.to(DEV), w.to(DEV, torch.bfloat16 if weights_as == "bf16" else torch.float32), experts, identity, top, 1.7,
                             correction.to(DEV), gate).double().cpu()
    want = pr.expert_weights({"top": top, "scale": 1.7}, {"router": w[:choices].double(), "correction": correction.double()}, "", x.double())
    torch.testing.assert_close(got[:, :experts], want[:, :experts], rtol=1e-5, atol=1e-7)
    torch.testing.assert_close(got[:, experts + 1], want[:, experts:].sum(1), rtol=1e-5, atol=1e-7)
    shared = torch.sigmoid(x.double() @ w[-1].double()) if gate else torch.ones(tokens, dtype=D64)
    torch.testing.assert_close(got[:, experts], shared, rtol=1e-5, atol=1e-6)
    # a token's weights do not depend on the rest of the step
    alone = ops.choose_experts(x[-1:].to(DEV), w.to(DEV, torch.bfloat16 if weights_as == "bf16" else torch.float32), experts, identity, top,
                               1.7, correction.to(DEV), gate).double().cpu()
    assert torch.equal(alone[0], got[-1])


def test_the_lower_expert_wins_a_tie():
    ops = _ops()
    x, w = torch.ones(2, 32, device=DEV), torch.zeros(70, 32, device=DEV)
    got = ops.choose_experts(x, w, 66, 4, 3, 1.0)
    assert torch.allclose(got[:, :3], torch.full((2, 3), 1 / 70, device=DEV)) and not got[:, 3:66].any() and not got[:, 67].any()


@TYPES
@pytest.mark.parametrize("ff,experts,shared", [(24, 6, 40), (9, 7, 11), (64, 2, 128)])
def test_exact_gelu_weighed_by_expert_and_gate(dtype, ff, experts, shared):
    ops = _ops()
    x = (torch.randn(13, experts * ff + shared) * 2.0).to(dtype)
    route = torch.rand(13, experts + 2)
    route[:, 1] = 0.0
    out = torch.empty_like(x, device=DEV)
    ops.unary_act(x.to(DEV), out, "gelu", route.to(DEV), ff, experts)
    factor = torch.cat([route[:, :experts].repeat_interleave(ff, 1), route[:, experts : experts + 1].expand(13, shared)], 1)
    torch.testing.assert_close(out.double().cpu(), pr.gelu_exact(x.double()) * factor.double(), **_tol(dtype, 1e-5, 1e-2))
    ops.unary_act(x.to(DEV), out, "gelu")
    torch.testing.assert_close(out.double().cpu(), pr.gelu_exact(x.double()), **_tol(dtype, 1e-5, 1e-2))


@TYPES
@pytest.mark.parametrize("width", [96, 100, 7, 4096, 8192])
def test_what_a_layer_returns_joins_the_stream_in_the_next_norm(dtype, width):
    """Normed terms with and without bias, plain terms, the returned input, a factor; all rows and selected
    ones (whose stream is left alone), and the sum without a norm behind it."""
    from rapid_llm_amd.parts.lazy import LayerSum, Returned, Term, plain
    from rapid_llm_amd.parts.norm import RMSNorm

    rows, eps = 11, 1e-5
    y = [torch.randn(rows, width).to(dtype) for _ in range(3)]
    bias, w0, w1, nw = torch.randn(width), 1.0 + 0.2 * torch.randn(width), 0.5 + 0.1 * torch.randn(width), 0.2 * torch.randn(width)
    x, numbers, residual = torch.randn(rows, width).to(dtype), torch.rand(rows, 5), torch.randn(rows, width)
    norm = RMSNorm(width, eps, "n", weight_offset=1.0)
    norm.bind({"norm.weight": nw.to(DEV)}, SimpleNamespace(dtype=dtype, device=DEV))
    dev = lambda t: None if t is None else t.to(DEV)  # noqa: E731
    cases = [
        ([(y[0], bias, w0), (y[1], None, w1), (y[2], None, None)], True, 0.7),
        ([(y[0], None, None), (y[2], None, None)], True, 0.5),
        ([(y[0], bias, None)], False, -1.3),
        ([(y[0], None, None), (y[1], bias, w1)], False, 1.0),
    ]
    for terms, back, factor in cases:
        total = torch.zeros(rows, width, dtype=D64)
        for t, b, w in terms:
            v = t.double() + (0 if b is None else b.double())
            total += pr.rms(v, 3e-4) * w.double() if w is not None else v
        if back:
            total += numbers[:, 3:4].double() * x.double()
        stream = residual.double() + factor * total
        pending = lambda: LayerSum([Term(dev(t), dev(b), dev(w)) for t, b, w in terms],  # noqa: E731
                                   Returned(dev(x), dev(numbers), 3) if back else None, factor, 3e-4)
        tol = _tol(dtype, 2e-5, 2e-2)
        res = residual.to(DEV)
        got = norm.forward(res, pending(), None)
        torch.testing.assert_close(got.double().cpu(), pr.around_one_norm(stream, nw.double(), eps), **tol)
        torch.testing.assert_close(res.double().cpu(), stream, rtol=2e-5, atol=2e-5)
        res = residual.to(DEV)
        pick = torch.tensor([rows - 1, 0, 0], dtype=torch.int32)
        got = norm.forward(res, pending(), None, pick.to(DEV))
        torch.testing.assert_close(got.double().cpu(), pr.around_one_norm(stream[pick.long()], nw.double(), eps), **tol)
        assert torch.equal(res.cpu(), residual)
        torch.testing.assert_close(plain(pending()).double().cpu(), factor * total, rtol=2e-5, atol=2e-5)


# --------------------------------------------------------------------------- #
# the model through the engine's step function
# --------------------------------------------------------------------------- #
LENGTHS = {
    "A": [1, 2, 3, 7, 8, 19, 20, 21, 57, 130],  # the first tokens; around pages of 8 and chunks of 7 and 20
    "B": [1, 2, 4, 5, 9, 33, 80],
    "C": [1, 2, 8, 9, 33, 34, 90],
    "D": [2, 15, 16, 17, 48, 49, 70, 150],
    "E": [1, 2, 16, 17, 40],
}


def _requests(which):
    cfg, _page, seed = RENI[which]
    return {f"q{i}": random_tokens(n, cfg["vocab"], seed * 100 + i) for i, n in enumerate(LENGTHS[which])}


def _oracles(pcfg, pw, requests):
    """Per request the plain logits in float64, and what rounding alone does to the rows of the plain
    implementation with rounded activations: half of them, and nine in ten."""
    want = {rid: pr.forward(pcfg, pw, toks) for rid, toks in requests.items()}
    order = sorted(want)
    rounded = torch.cat([pr.forward(pcfg, pw, requests[r], cast=bf16_round) for r in order])
    rows = row_errors(rounded, torch.cat([want[r] for r in order]))
    return want, (float(rows.median()), float(rows.quantile(0.9)))


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
    """float32: every row within the bound.  bfloat16: the engine's typical rows against the rounded plain
    implementation's typical rows; a token whose experts' scores lie closer than rounding moves them takes
    another expert, there as in an engine though not at the same tokens, and the memories carry the
    difference on, so a tenth of the rows may lie further out."""
    order = sorted(want)
    a, b = torch.cat([got[r] for r in order]), torch.cat([want[r] for r in order])
    assert a.shape == b.shape and torch.isfinite(a).all(), label
    rows = row_errors(a, b)
    if dtype == "float32":
        bad = rows > F32_ROW
        where = [(r, p) for r in order for p in range(want[r].shape[0])]
        assert not bad.any(), f"{label}: first wrong {where[int(torch.nonzero(bad)[0])]}, worst row {float(rows.max()):.3e} of the spread"
        return
    median, ninth = rounding
    parity.record(label, float(rows.max()), float((a.double() - b.double()).abs().max() / b.double().std()))
    assert float(rows.median()) <= BF16_TIMES_ROUNDING * median, (label, float(rows.median()), median)
    assert float((rows > BF16_TIMES_ROUNDING * ninth).double().mean()) <= BF16_ROWS_BEYOND, (label, float(rows.max()), ninth)


@pytest.mark.parametrize("which", ["A", "B", "C", "D", "E"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_every_cut_matches_plain(tmp_path, which, dtype):
    cfg, page, seed = RENI[which]
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
            # chunks begin where a portion does: the cuts differ by rounding, far less than the bound
            first = first or got
            for rid in got:
                torch.testing.assert_close(got[rid], first[rid], rtol=1e-4, atol=1e-4, msg=f"{label} {rid}")
        runner.cache.check_invariants()
        assert not runner.cache.live_requests()
        del runner


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_batch_of_unequal_requests_equals_each_alone(tmp_path, dtype):
    """One step holds a long prompt, a short one, a single first token and decoded tokens of two
    requests at different depths; every row equals the row of the request run alone, cut alike."""
    which = "A"
    cfg, page, seed = RENI[which]
    model_dir = make_model_dir(tmp_path, which, sharp=3.0)
    requests = {f"u{i}": random_tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate((90, 5, 1, 61, 30))}
    cut = {"u0": [90], "u1": [5], "u2": [1], "u3": [60, 1], "u4": [29, 1]}
    runner = _runner(model_dir, dtype, page, 60, 100, slots=5)
    full = lambda r, a, b: {"id": r, "tokens": requests[r][a:b], "want": list(range(b - a))}  # noqa: E731
    steps, n = [], 0
    for r, sizes in cut.items():
        at = 0
        for size in sizes:
            steps.append({"step": n, "entries": [full(r, at, at + size)], "end": [r] if at + size == len(requests[r]) else []})
            at, n = at + size, n + 1
    alone = ru.run_in_process(runner, steps)
    steps = [
        {"step": 0, "entries": [full("u3", 0, 60), full("u4", 0, 29)], "end": []},
        {"step": 1, "entries": [full("u0", 0, 90), full("u3", 60, 61), full("u1", 0, 5), full("u2", 0, 1), full("u4", 29, 30)],
         "end": ["u0", "u1", "u2", "u3", "u4"]},
    ]
    got = ru.run_in_process(runner, steps)
    for rid in requests:
        if dtype == "float32":
            torch.testing.assert_close(got[rid], alone[rid], rtol=1e-4, atol=1e-4)
        else:  # (products of few and of many rows differ by rounding, which may choose another expert)
            assert float(row_errors(got[rid], alone[rid]).median()) < 0.08, rid
    runner.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_and_slots_used_again(tmp_path, dtype):
    """Five requests through two slots, each a short prompt and then 200 tokens one by one, two at a time
    in a step, on a pool of the pages that two chunks take: pages of complete chunks come back and are taken
    again, and a later request finds the states of its slot zeroed."""
    which = "A"
    cfg, page, seed = RENI[which]
    model_dir = make_model_dir(tmp_path, which, sharp=3.0)
    pcfg, pw = load_plain(model_dir)
    requests = {f"d{i}": random_tokens(200 + 7 * i, cfg["vocab"], 40 + i) for i in range(5)}
    want, rounding = _oracles(pcfg, pw, requests)
    steps = ru.mixed(requests, 3, max_live=2, tail=195)
    runner = _runner(model_dir, dtype, page, 2 * (-(-40 // page) + 1) + 2, 240, slots=2)
    got = ru.run_in_process(runner, steps)
    _check(got, want, dtype, f"long decoding/{dtype}", rounding)
    runner.cache.check_invariants()


def test_a_far_token_still_counts(tmp_path):
    """A different first token changes the logits 150 positions later, beyond every chunk, alike whether the
    tokens in between came in one prompt or one by one."""
    which = "A"
    cfg, page, seed = RENI[which]
    model_dir = make_model_dir(tmp_path, which)
    pcfg, pw = load_plain(model_dir)
    toks = random_tokens(150, cfg["vocab"], 12)
    other = [(toks[0] + 1) % cfg["vocab"]] + toks[1:]
    want = {"same": pr.forward(pcfg, pw, toks), "other": pr.forward(pcfg, pw, other)}
    assert float(row_errors(want["other"][-1:], want["same"][-1:]).max()) > 50 * F32_ROW
    for steps_of in (ru.whole, lambda r: ru.prefill_then_decode(r, 140)):
        runner = _runner(model_dir, "float32", page, 60, 160)
        got = ru.run_in_process(runner, steps_of({"same": toks, "other": other}))
        _check(got, want, "float32", "far token")


def test_trace_program(tmp_path):
    """``bin/trace_run`` as a child process on a mixed trace over a tight pool."""
    which = "B"
    cfg, page, seed = RENI[which]
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

    cfg, page, seed = RENI[which]
    model_dir = make_model_dir(tmp_path, which)
    pcfg, pw = load_plain(model_dir)
    prompts = [random_tokens(n, cfg["vocab"], seed + n) for n in (1, 7, 30, 45)]
    llm = LLM(str(model_dir), dtype=dtype, page_size=page, num_pages=60, max_num_seqs=3, max_seq_len=96,
              max_chunk_size=16, max_num_batched_tokens=32, use_cuda_graph=use_graph)
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_gen_len=24))
    gaps = []
    for prompt, out in zip(prompts, outs):
        ids = list(prompt)
        for tok in out.token_ids:
            logits = pr.forward(pcfg, pw, ids)[-1]
            gaps.append(float((logits.max() - logits[tok]) / logits.std()))
            ids.append(tok)
        assert len(out.token_ids) == 24
    if dtype == "float32":
        assert max(gaps) <= 1e-3, max(gaps)
    else:
        gaps.sort()
        assert gaps[len(gaps) // 2] == 0.0 and gaps[int(0.85 * len(gaps))] <= 0.5, gaps[-10:]
    llm.scheduler.cache.check_invariants()
    assert not llm.scheduler.cache.live_requests()
