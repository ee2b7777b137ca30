"""CPU tests of the Renitar decoder: its configuration, its description as parts, its weights by
name (packed products, a size that only a tensor gives), the pages of chunks, and the plain
implementation that the GPU tests compare the engine with."""

import copy
import json
import math

import pytest
import torch

import plain_renitar as pr
from renitar_configs import RENI, make_model_dir, make_weights, random_tokens, row_errors, tensor_shapes

F32_ROW = 2e-4  # the GPU tests' float32 bound on a row, relative to the logits' spread
D64 = torch.float64


def bf16_round(t):
    return t.bfloat16().to(t.dtype)


def _spec(cfg):
    from rapid_llm_amd.config.registry import config_from_dict

    entry, typed = config_from_dict(cfg)
    return entry, typed, entry.build_spec(typed)


@pytest.mark.parametrize("which", sorted(RENI))
def test_configuration_round_trip(which):
    cfg, _page, _seed = RENI[which]
    entry, typed, spec = _spec(cfg)
    assert entry.name == "Renitar"
    assert type(typed).from_dict(json.loads(json.dumps(typed.to_dict()))) == typed
    assert list(spec.order()) == list(range(len(cfg["layers"])))
    assert all(layer.shared_norm and layer.block.params["factor"] == cfg["residual_mult"] for layer in spec.layers)


def test_configuration_refuses_what_the_design_does_not_have():
    from rapid_llm_amd.config.model_config import ConfigError

    cfg, _page, _seed = RENI["A"]
    for change in (
        lambda c: c["layers"][0].update(type="attention"),
        lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3),
        lambda c: c["layers"][0]["mixer"]["left"].update(dim=300),
        lambda c: c["layers"][0]["mixer"]["left"].update(softcap=0.0),
        lambda c: c["layers"][0]["mixer"]["left"].update(conv=0),
        lambda c: c["layers"][0]["mixer"]["left"].pop("scale"),
        lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0),
        lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=7),
        lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=18),
        lambda c: c["layers"][0]["mixer"].pop("right"),
        lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.5]),
        lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.0, 0.5]),
        lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 1.5, 0.5]),
        lambda c: c["layers"][0]["mlp"].update(kind="dense"),
        lambda c: c["layers"][0]["mlp"]["router"].update(top=10),
        lambda c: c["layers"][0]["mlp"]["router"].update(experts=0),
        lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1),
        lambda c: c["layers"][0]["mlp"].pop("expert"),
        lambda c: c["layers"][1]["mixer"].update(tau=0),
        lambda c: c["layers"][1]["mixer"].update(rank=-1),
        lambda c: c["layers"].clear(),
        lambda c: c.pop("residual_mult"),
        lambda c: c["norm"].update(eps=0.0),
    ):
        broken = copy.deepcopy(cfg)
        change(broken)
        with pytest.raises(ConfigError):
            _spec(broken)


@pytest.mark.parametrize("which", sorted(RENI))
def test_parameters_cover_the_checkpoint_tensor_by_tensor(which, tmp_path):
    from rapid_llm_amd.models.causal_lm import CausalLM
    from rapid_llm_amd.weights.loader import load_model_dir

    cfg, _page, _seed = RENI[which]
    model = CausalLM(_spec(cfg)[2])
    named = {}
    for spec in model.param_specs():
        for src in spec.sources:
            if src.name:
                assert src.name not in named
                named[src.name] = spec.source_shape(src.rows)
    assert named == tensor_shapes(cfg)
    params = load_model_dir(make_model_dir(tmp_path, which), model.param_specs(), engine_dtype=torch.bfloat16,
                            device="cpu")
    for name, t in params.items():
        if name.endswith((".decay_out", ".decay_bias", ".conv", "_bias", "norm", ".router", ".correction", ".weight")) and "embed" not in name and "output" not in name:
            assert t.dtype == torch.float32, name
    assert model.replayable()


def test_two_mixers_share_their_input_product(tmp_path):
    """Rows of one matrix, each mixer's from a multiple of 8 on with zeros between; biases only where the
    heads are; the output projections are matrices of their own."""
    from rapid_llm_amd.models.causal_lm import CausalLM
    from rapid_llm_amd.weights.loader import load_model_dir

    cfg, _page, seed = RENI["C"]
    model = CausalLM(_spec(cfg)[2])
    pair = model.blocks[1].mixer
    params = load_model_dir(make_model_dir(tmp_path, "C"), model.param_specs(), engine_dtype=torch.float32, device="cpu")
    w = {k: v.float() for k, v in make_weights(cfg, seed).items()}
    packed, at = params["layers.1.mixer.in"], pair.columns[1]
    left = torch.cat([w["l1.mix.left." + s] for s in "qkvg"])
    right = torch.cat([w["l1.mix.right." + s] for s in "qkvg"])
    assert at % 8 == 0 and at >= left.shape[0]
    assert torch.equal(packed[: left.shape[0]], left) and not packed[left.shape[0] : at].any()
    assert torch.equal(packed[at : at + right.shape[0]], right) and not packed[at + right.shape[0] :].any()
    bias = params["layers.1.mixer.left.qkv_bias"]
    heads = torch.cat([w[f"l1.mix.left.{s}.b"] for s in "qkv"])
    assert torch.equal(bias[: heads.shape[0]], heads) and not bias[heads.shape[0] :].any()
    assert torch.equal(params["layers.1.mixer.left.o"], w["l1.mix.left.o"])
    assert torch.equal(params["layers.1.mixer.right.o"], w["l1.mix.right.o"])
    assert torch.equal(params["layers.1.ff.router"], torch.cat([w["l1.mlp.router"], w["l1.mlp.shared.sg"]]))


def test_options_that_do_not_go_together_are_refused():
    from rapid_llm_amd.models.spec import PartSpec
    from rapid_llm_amd.parts import BLOCKS, FEED_FORWARDS, MIXERS
    from rapid_llm_amd.parts.lazy import LayerSum, Term

    attention = {"hidden_size": 32, "num_heads": 2, "num_kv_heads": 1, "head_dim": 16, "checkpoint_prefix": "c."}
    for more in (
        {"chunked": True},
        {"chunked": True, "window": 8, "keep_first": 2},
        {"conv_taps": 17},
        {"conv_taps": 2, "values": "keys"},
        {"conv_taps": 2, "qk_norm_eps": 1e-6},  # norms a head behind a convolution
        {"gate_name": "g", "head_gate_name": "h"},
        {"qk_norm_scope": "row", "qk_norm_eps": 1e-6},
    ):
        with pytest.raises(ValueError):
            MIXERS.create("gqa_attention", **{**attention, **more})
    linear = {"hidden_size": 32, "num_heads": 2, "key_dim": 8, "value_dim": 8, "norm_eps": 1e-6, "checkpoint_prefix": "d.",
              "decay": "fixed", "decays": (0.5, 0.9), "norm": "row", "gate": "silu"}
    MIXERS.create("linear_attention", **linear)
    for more in ({"decays": (0.5,)}, {"decays": (0.5, 1.1)}, {"decay": "none"}, {"norm": "all"}, {"gate": "tanh"}, {"key_dim": 257},
                 {"decay": "channel", "tau": 0.0}):
        with pytest.raises(ValueError):
            MIXERS.create("linear_attention", **{**linear, **more})
    # a biased output projection and decays of the channels do not share products
    left = PartSpec("gqa_attention", {**attention, "chunked": True, "window": 8, "qkv_bias": True, "o_bias": True})
    right = PartSpec("linear_attention", linear)
    scales = {"left_scale": 1.0, "right_scale": 1.0}
    MIXERS.create("side_by_side", hidden_size=32, left=left, right=right, **scales, out_norm_names=("a", "b"), out_norm_eps=1e-6)
    with pytest.raises(ValueError):
        MIXERS.create("side_by_side", hidden_size=32, left=left, right=right, **scales)
    with pytest.raises(ValueError):
        MIXERS.create("side_by_side", hidden_size=32, left=left, right=right, **scales, out_norm_names=("a", "b"))
    with pytest.raises(ValueError):
        MIXERS.create("side_by_side", hidden_size=32, left=left, right=PartSpec("linear_attention", {**linear, "decay": "channel"}),
                      **scales, out_norm_names=("a", "b"), out_norm_eps=1e-6)
    experts = {"hidden_size": 32, "num_experts": 4, "top": 2, "expert_size": 8, "checkpoint_prefix": "e.", "activation": "gelu"}
    for more in ({"identity": 1}, {"correction_name": "c"}, {"scores": "softmax_raw", "gated": True, "activation": "silu"},
                 {"scores": "softmax_raw", "shared_gate_name": "s"}, {"scores": "softmax_raw", "identity": 1, "top": 6}):
        with pytest.raises(ValueError):
            FEED_FORWARDS.create("routed_experts", **{**experts, **more})
    with pytest.raises(ValueError):
        BLOCKS.create("shared_norm", mixer=None, feed_forward=None, mixer_norm=None, feed_forward_norm=object())
    y, w = torch.zeros(1, 4), torch.ones(4)
    with pytest.raises(ValueError):  # two epsilons in one sum
        LayerSum.of([LayerSum([Term(y, None, w)], eps=1e-6), LayerSum([Term(y, None, w)], eps=1e-5)], 1.0)
    with pytest.raises(ValueError):  # a factor inside a sum
        LayerSum.of([LayerSum([Term(y)], factor=0.5)], 1.0)


def test_a_size_that_only_a_tensor_gives(tmp_path):
    from rapid_llm_amd.models.causal_lm import CausalLM
    from rapid_llm_amd.weights.loader import WeightsError, load_model_dir
    from rapid_llm_amd.weights.random_init import write_random_model

    cfg, _page, _seed = RENI["A"]
    folder = make_model_dir(tmp_path, "A")
    bare = copy.deepcopy(cfg)
    for layer in bare["layers"]:
        layer["mixer"].pop("rank", None)
    params = load_model_dir(folder, CausalLM(_spec(bare)[2]).param_specs(), engine_dtype=torch.float32, device="cpu")
    assert params["layers.1.mixer.decay_in"].shape == (5, 96) and params["layers.1.mixer.decay_out"].shape == (72, 5)
    with pytest.raises(ValueError):
        write_random_model(bare, 1, tmp_path / "bare")
    other = copy.deepcopy(cfg)
    other["layers"][1]["mixer"]["rank"] = 6
    with pytest.raises(WeightsError):
        load_model_dir(folder, CausalLM(_spec(other)[2]).param_specs(), engine_dtype=torch.float32, device="cpu")
    written = write_random_model(cfg, 3, tmp_path / "drawn")
    assert set(tensor_shapes(cfg)) == set(__import__("safetensors.torch", fromlist=["load_file"]).load_file(
        str(written / "model.safetensors")))


def test_cache_needs_pages_of_a_chunk_and_states():
    from rapid_llm_amd.cache.storage import plan_groups
    from rapid_llm_amd.models.causal_lm import CausalLM

    needs = CausalLM(_spec(RENI["A"][0])[2]).cache_needs()
    assert [n.kind for n in needs] == ["paged", "state", "state", "paged"]
    assert {p.name: p.shape for p in needs[0].paged} == {"k": (2, 16), "v": (2, 32)}
    assert needs[0].window == 20 and needs[0].chunked and needs[3].window == 7 and needs[3].chunked
    assert {s.name: s.shape for s in needs[0].state_specs()} == {"left.conv": (2, 4 * 16 + 2 * 16 + 2 * 32), "right.S": (3, 16, 24)}
    assert {s.name: s.shape for s in needs[1].states} == {"S": (3, 24, 16)}
    assert all(s.dtype == "float32" for n in needs for s in n.state_specs())
    groups, of = plan_groups(needs)
    assert of == [0, None, None, 1] and [(g.window, g.chunked) for g in groups] == [(20, True), (7, True)]
    # a sliding window of the same length is another group
    from dataclasses import replace

    groups, of = plan_groups([needs[0], replace(needs[0], chunked=False), needs[0]])
    assert of == [0, 1, 0]


@pytest.mark.parametrize("chunk,page", [(20, 8), (16, 4), (7, 8), (1, 4), (33, 16)])
def test_pages_of_a_chunk_come_back_when_it_is_complete(chunk, page):
    """After every step a request maps the pages from its current chunk's first position on (or none
    between two chunks), whether tokens come one by one or in portions."""
    from rapid_llm_amd.cache.manager import CacheManager, GroupSpec

    for sizes in ((1,), (5, 2, 17), (40,)):
        cache = CacheManager([GroupSpec(0, chunk, (0,), chunked=True)], 200, page, 2, 160)
        cache.admit("a")
        at, i = 0, 0
        while at < 120:
            n = min(sizes[i % len(sizes)], 120 - at)
            i += 1
            assert cache.reserve("a", at + n, at)
            row = cache.tables[0][cache.slot_of("a")]
            assert all(row[p // page] for p in range(at // chunk * chunk, at + n))  # what the step's queries read
            at += n
            cache.trim("a", at)
            first, last = at // chunk * chunk // page, -(-at // page)
            assert [p for p in range(len(row)) if row[p]] == list(range(first, last))
            cache.check_invariants()
        cache.release("a")
        cache.check_invariants()
        assert cache.num_free_pages(0) == 199


# --------------------------------------------------------------------------- #
# the plain implementation
# --------------------------------------------------------------------------- #


def test_plain_mechanisms_one_by_one():
    """Each mechanism of the plain implementation on inputs whose answer is known."""
    e = torch.eye(2, dtype=D64)
    # a memory: the read-out sees the token's own write, decays act on the rows of the key channels
    k = torch.stack([e[0], e[1], e[0]]).view(3, 1, 2)
    q = torch.stack([e[0], e[0] + e[1], e[0] + 10 * e[1]]).view(3, 1, 2)
    v = torch.tensor([3.0, 5.0, 7.0], dtype=D64).view(3, 1, 1)
    a = torch.tensor([[1.0, 1.0], [0.5, 1.0], [0.5, 0.1]], dtype=D64).view(3, 1, 2)
    assert torch.allclose(pr.decayed_memory(q, k, v, a).flatten(), torch.tensor([3.0, 1.5 + 5.0, 0.75 + 7.0 + 5.0], dtype=D64))
    assert torch.allclose(pr.decayed_memory(q, k, v, torch.tensor(0.5, dtype=D64).view(1, 1, 1)).flatten(),
                          torch.tensor([3.0, 1.5 + 5.0, 0.75 + 7.0 + 25.0], dtype=D64))
    assert abs(float(pr.channel_decay(torch.zeros(1, dtype=D64), 4.0)) - 0.5**0.25) < 1e-12
    # convolution: the last tap meets the current token, zeros before the start, no activation
    y = pr.short_convolution(torch.tensor([[1.0], [10.0], [100.0]], dtype=D64), torch.tensor([[2.0, 0.0, 3.0]], dtype=D64))
    assert y.flatten().tolist() == [3.0, 30.0, 302.0]
    # rotation: halves pair, position 0 stays, lengths stay, the rest passes
    x = torch.randn(5, 2, 10, dtype=D64)
    r = pr.rotate(x, 6, 50.0)
    assert torch.equal(r[0], x[0]) and torch.equal(r[..., 6:], x[..., 6:])
    assert torch.allclose(r[..., 0] ** 2 + r[..., 3] ** 2, x[..., 0] ** 2 + x[..., 3] ** 2)
    assert torch.allclose(r[2, :, 0], x[2, :, 0] * math.cos(2.0) - x[2, :, 3] * math.sin(2.0))
    f1 = 50.0 ** (-2 / 6)
    assert torch.allclose(r[3, :, 4], x[3, :, 4] * math.cos(3 * f1) + x[3, :, 1] * math.sin(3 * f1))
    # the mask, element by element
    seen = pr.chunk_mask(9, 4)
    assert [int(row.sum()) for row in seen] == [1, 2, 3, 4, 1, 2, 3, 4, 1]
    assert bool(seen[7, 4]) and not bool(seen[7, 3]) and not bool(seen[4, 5])
    assert abs(float(pr.soft_cap(torch.tensor(100.0, dtype=D64), 5.0)) - 5.0) < 1e-9
    assert abs(float(pr.gelu_exact(torch.tensor(1.0, dtype=D64))) - 0.8413447460685429) < 1e-12
    # the correction decides the choice, the weights are the scores without it, not renormalised
    r = {"top": 2, "scale": 3.0}
    w = {"router": torch.log(torch.tensor([[0.4], [0.3], [0.2], [0.1]], dtype=D64)), "correction": torch.tensor([0.0, 0.0, 0.0, 0.25], dtype=D64)}
    weights = pr.expert_weights(r, w, "", torch.ones(1, 1, dtype=D64))
    assert torch.allclose(weights, torch.tensor([[1.2, 0.0, 0.0, 0.3]], dtype=D64))
    # an identity expert returns its input; the shared expert is weighed by a sigmoid
    m = {"router": {"experts": 1, "identity": 1, "top": 2, "scale": 1.0}}
    w = {"router": torch.zeros(2, 2, dtype=D64), "correction": torch.zeros(2, dtype=D64), "e0.up": torch.zeros(1, 2, dtype=D64),
         "e0.down": torch.zeros(2, 1, dtype=D64), "shared.up": torch.tensor([[1.0, 0.0]], dtype=D64),
         "shared.down": torch.tensor([[1.0], [0.0]], dtype=D64), "shared.sg": torch.zeros(1, 2, dtype=D64)}
    h = torch.tensor([[1.0, 4.0]], dtype=D64)
    assert torch.allclose(pr.mixture(m, w, "", h), torch.tensor([[0.5 + 0.5 * 0.8413447460685429, 2.0]], dtype=D64))


# faults a comparison is there for: a function of the plain implementation replaced by a wrong one
_RIGHT = {n: getattr(pr, n) for n in ("decayed_memory", "channel_decay", "short_convolution", "rotate", "chunk_mask", "soft_cap",
                                      "expert_weights", "expert", "rms")}


def _read_before_write(q, k, v, a):
    return _RIGHT["decayed_memory"](q, k, v, a) - (q * k).sum(-1, keepdim=True) * v


def _decay_after_write(q, k, v, a):
    return _RIGHT["decayed_memory"](q * a.expand_as(q), k, v, a)


def _corrected_weights(r, w, p, h):
    s = torch.softmax(h @ w[p + "router"].T, -1) + w[p + "correction"]
    return s * torch.zeros_like(s).scatter_(-1, torch.topk(s, r["top"], -1).indices, 1.0) * r["scale"]


def _renormalised(r, w, p, h):
    y = _RIGHT["expert_weights"](r, w, p, h)
    return r["scale"] * y / y.sum(-1, keepdim=True)


def _uncorrected(r, w, p, h):
    return _RIGHT["expert_weights"](r, {**w, p + "correction": torch.zeros_like(w[p + "correction"])}, p, h)


def _no_identity(r, w, p, h):
    y = _RIGHT["expert_weights"](r, w, p, h).clone()
    y[:, r["experts"] :] = 0
    return y


WRONG = {
    "the read-out misses the token's own write": ("decayed_memory", _read_before_write),
    "the decay after the write": ("decayed_memory", _decay_after_write),
    "one decay a head": ("channel_decay", lambda z, tau: _RIGHT["channel_decay"](z, tau).mean(-1, keepdim=True)),
    "decays without their power": ("channel_decay", lambda z, tau: torch.sigmoid(z)),
    "a convolution that forgets the oldest tap": (
        "short_convolution",
        lambda x, taps: _RIGHT["short_convolution"](x, torch.cat([torch.zeros_like(taps[:, :1]), taps[:, 1:]], 1))),
    "an activation behind the convolution": ("short_convolution", lambda x, taps: pr.silu(_RIGHT["short_convolution"](x, taps))),
    "positions one late": ("rotate", lambda x, dims, base: _RIGHT["rotate"](torch.cat([torch.zeros_like(x[:1]), x]), dims, base * 1.1)[1:]),
    "the whole head rotates": ("rotate", lambda x, dims, base: _RIGHT["rotate"](x, x.shape[-1], base)),
    "a window that slides": ("chunk_mask", lambda T, size: torch.ones(T, T).tril().triu(-size + 1).bool()),
    "chunks one longer": ("chunk_mask", lambda T, size: _RIGHT["chunk_mask"](T, size + 1)),
    "chunks one shorter": ("chunk_mask", lambda T, size: _RIGHT["chunk_mask"](T, size - 1)),
    "no cap": ("soft_cap", lambda s, cap: s),
    "the tanh form of gelu": ("gelu_exact", lambda z: 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z**3)))),
    "the correction in the weights": ("expert_weights", _corrected_weights),
    "no correction": ("expert_weights", _uncorrected),
    "weights over their sum": ("expert_weights", _renormalised),
    "identity experts left out": ("expert_weights", _no_identity),
    "norm weights as they are": ("around_one_norm", lambda x, w, eps: pr.rms(x, eps) * w),
}


@pytest.mark.parametrize("fault", sorted(WRONG))
def test_plain_tells_a_wrong_mechanism(fault, monkeypatch):
    """With the tests' weights each fault moves some row by at least twenty times what the float32
    comparison allows."""
    cfg, _page, seed = RENI["A"]
    w = make_weights(cfg, seed, sharp=3.0)
    toks = random_tokens(60, cfg["vocab"], 9)
    want = pr.forward(cfg, w, toks)
    monkeypatch.setattr(pr, *WRONG[fault])
    times = 2 if fault == "the tanh form of gelu" else 20  # (the two forms lie within 5e-4 of each other)
    assert float(row_errors(pr.forward(cfg, w, toks), want).max()) > times * F32_ROW


def test_plain_tells_wrong_constants_and_lost_tensors():
    cfg, _page, seed = RENI["A"]
    w = make_weights(cfg, seed, sharp=3.0)
    toks = random_tokens(60, cfg["vocab"], 9)
    want = pr.forward(cfg, w, toks)

    def shows(c, weights):
        return float(row_errors(pr.forward(c, weights, toks), want).max()) > 20 * F32_ROW

    for change in (
        lambda c: c.update(residual_mult=0.75),
        lambda c: c["layers"][0]["mixer"]["left"].update(scale=0.25),
        lambda c: c["layers"][0]["mixer"]["left"].update(softcap=7.0),
        lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(base=900.0),
        lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.9, 0.98]),
        lambda c: c["layers"][1]["mixer"].update(tau=9.0),
        lambda c: c["layers"][0]["mlp"]["router"].update(scale=1.4),
        lambda c: c["layers"][0]["mlp"]["router"].update(top=3),
    ):
        c = copy.deepcopy(cfg)
        change(c)
        assert shows(c, w)
    lost = [n for n in tensor_shapes(cfg) if n.endswith((".b", "correction", "shared.sg", ".g", "a1"))]
    for name in lost:
        w2 = dict(w)
        w2[name] = torch.zeros_like(w[name])
        assert shows(cfg, w2), name
    # a norm over all heads is not one over each, and the sides are normed before they are added
    for name in ("l0.mix.left.q.norm", "l0.mix.left.k.norm", "l0.mix.right.norm", "l0.mix.left.out", "l0.mix.right.out", "l1.mix.norm"):
        assert shows(cfg, {**w, name: torch.ones_like(w[name])}), name


def test_plain_shows_a_state_that_is_not_carried():
    """A different first token changes the logits far behind it, and so does a state that starts
    anew in the middle: the comparison over cut requests sees both."""
    cfg, _page, seed = RENI["A"]
    w = make_weights(cfg, seed)
    toks = random_tokens(150, cfg["vocab"], 12)
    want = pr.forward(cfg, w, toks)
    other = pr.forward(cfg, w, [(toks[0] + 1) % cfg["vocab"]] + toks[1:])
    assert float(row_errors(other[-1:], want[-1:]).max()) > 50 * F32_ROW
    anew = pr.forward(cfg, w, toks[80:])  # (80: a multiple of the first layer's chunks)
    assert float(row_errors(anew[-1:], want[-1:]).max()) > 50 * F32_ROW


@pytest.mark.parametrize("which", sorted(RENI))
def test_rounding_alone_stays_within_the_bounds_of_the_gpu_tests(which):
    """What rounding does to half of the rows is small beside the logits' spread in every configuration."""
    cfg, _page, seed = RENI[which]
    w = make_weights(cfg, seed, sharp=3.0)
    toks = random_tokens(80, cfg["vocab"], 5)
    rows = row_errors(pr.forward(cfg, w, toks, cast=bf16_round), pr.forward(cfg, w, toks))
    assert float(rows.median()) < 0.04, float(rows.median())
