"""CPU tests of the Pefulorn decoder: its configuration, its description as parts, its weights by
name (packed products, sizes that only a tensor gives), and the plain implementation that the GPU
tests compare the engine with."""

import copy
import json
import math

import pytest
import torch

import plain_pefulorn as pp
from pefulorn_configs import PEFU, make_model_dir, make_weights, random_tokens, row_errors, tensor_shapes

F32_ROW = 2e-4  # the GPU tests' float32 bound on a row, relative to the logits' spread
D64 = torch.float64


def bf16_round(t):
    return t.bfloat16().to(t.dtype)


def _spec(cfg):
    from rapid_llm_amd.config.registry import config_from_dict

    entry, typed = config_from_dict(cfg)
    return entry, typed, entry.build_spec(typed)


@pytest.mark.parametrize("which", sorted(PEFU))
def test_configuration_round_trip_and_run_order(which):
    cfg, _page, _seed = PEFU[which]
    entry, typed, spec = _spec(cfg)
    assert entry.name == "Pefulorn"
    assert type(typed).from_dict(json.loads(json.dumps(typed.to_dict()))) == typed
    order = [i for i, _begins in pp.passes(cfg)]
    begins = {place: t for place, (_i, t) in enumerate(pp.passes(cfg)) if t is not None}
    assert list(spec.order()) == order
    if begins:
        assert dict(zip(spec.stream_offsets.places, range(len(begins)))) == begins
    else:
        assert spec.stream_offsets is None
    returns = set(spec.stream_returns.places) if spec.stream_returns else set()
    assert returns == {place for place, t in begins.items() if t > 0}


def test_configuration_refuses_what_the_design_does_not_have():
    from rapid_llm_amd.config.model_config import ConfigError

    cfg, _page, _seed = PEFU["A"]
    for change in (
        lambda c: c["layers"][0].update(type="attention"),
        lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3),
        lambda c: c["layers"][0]["mixer"]["left"].update(dim=300),
        lambda c: c["layers"][0]["mixer"]["left"]["q_temp"].update(every=0),
        lambda c: c["layers"][0]["mixer"].pop("right"),
        lambda c: c["layers"][0]["mixer"].pop("left_scale"),
        lambda c: c["layers"][0]["mlp"].update(kind="moe"),
        lambda c: c["layers"][0]["mlp"].update(ff=0),
        lambda c: c["layers"][1]["mixer"].update(kv_heads=3),
        lambda c: c["layers"][1]["mixer"].update(conv=0),
        lambda c: c["layers"][2]["mixer"].update(rank=-1),
        lambda c: c["layers"].clear(),
        lambda c: c["loop"].update(stop=5),
        lambda c: c["loop"].update(times=0),
        lambda c: c["norm"].update(eps=0.0),
    ):
        broken = copy.deepcopy(cfg)
        change(broken)
        with pytest.raises(ConfigError):
            _spec(broken)


@pytest.mark.parametrize("which", sorted(PEFU))
def test_parameters_cover_the_checkpoint_tensor_by_tensor(which, tmp_path):
    from rapid_llm_amd.models.causal_lm import CausalLM
    from rapid_llm_amd.weights.loader import load_model_dir

    cfg, _page, _seed = PEFU[which]
    model = CausalLM(_spec(cfg)[2])
    named = {}
    for spec in model.param_specs():
        for src in spec.sources:
            if src.name:
                named[src.name] = spec.source_shape(src.rows)
    assert named == tensor_shapes(cfg)
    params = load_model_dir(make_model_dir(tmp_path, which), model.param_specs(), engine_dtype=torch.bfloat16,
                            device="cpu")
    for name, t in params.items():
        if name.endswith((".decay_out", ".decay_bias", ".decay_log", ".conv", ".r1", ".r2", "_bias", ".mu", ".bonus", "norm")):
            assert t.dtype == torch.float32, name


def test_two_mixers_share_their_products(tmp_path):
    """The input projections of a pair are the rows of one matrix, each mixer's from a multiple of 8
    on with zeros between, and the output projections lie side by side in another."""
    from rapid_llm_amd.models.causal_lm import CausalLM
    from rapid_llm_amd.weights.loader import load_model_dir

    cfg, _page, seed = PEFU["C"]
    model = CausalLM(_spec(cfg)[2])
    pair = model.blocks[1].mixer
    params = load_model_dir(make_model_dir(tmp_path, "C"), model.param_specs(), engine_dtype=torch.float32, device="cpu")
    w = {k: v.float() for k, v in make_weights(cfg, seed).items()}
    packed = params["layers.1.mixer.in"]
    at = pair.columns[1]
    assert at % 8 == 0 and at >= 6 * 12 + 3 * 12 + 3 * 10
    left = torch.cat([w["l1.mix.left." + s] for s in "qkv"])
    right = torch.cat([w["l1.mix.right." + s] for s in "zxg"])
    assert torch.equal(packed[: left.shape[0]], left) and not packed[left.shape[0] : at].any()
    assert torch.equal(packed[at : at + right.shape[0]], right) and not packed[at + right.shape[0] :].any()
    assert torch.equal(params["layers.1.mixer.o"], torch.cat([w["l1.mix.left.o"], w["l1.mix.right.o"]], 1))


def test_a_pair_needs_mixers_that_share_products():
    from rapid_llm_amd.models.spec import PartSpec
    from rapid_llm_amd.parts import MIXERS

    gru = PartSpec("min_gru", {"hidden_size": 32, "width": 8, "checkpoint_prefix": "a."})
    other = PartSpec("wkv", {"hidden_size": 32, "num_heads": 2, "head_dim": 16, "norm_eps": 1e-5, "checkpoint_prefix": "b."})
    pair = MIXERS.create("side_by_side", hidden_size=32, left=gru, right=gru, left_scale=1.0, right_scale=1.0)
    need = pair.cache_need()  # no pages at all, two states told apart
    assert need.kind == "state" and {s.name: s.shape for s in need.state_specs()} == {"left.S": (8,), "right.S": (8,)}
    with pytest.raises(ValueError):
        MIXERS.create("side_by_side", hidden_size=32, left=gru, right=other, left_scale=1.0, right_scale=1.0)
    plain = PartSpec("gqa_attention", {"hidden_size": 32, "num_heads": 2, "num_kv_heads": 1, "head_dim": 16, "checkpoint_prefix": "c."})
    with pytest.raises(ValueError):
        MIXERS.create("side_by_side", hidden_size=32, left=plain, right=gru, left_scale=1.0, right_scale=1.0)


def test_sizes_that_only_a_tensor_gives(tmp_path):
    from rapid_llm_amd.models.causal_lm import CausalLM
    from rapid_llm_amd.weights.loader import WeightsError, load_model_dir
    from rapid_llm_amd.weights.random_init import write_random_model

    cfg, _page, _seed = PEFU["A"]
    folder = make_model_dir(tmp_path, "A")
    bare = copy.deepcopy(cfg)
    for layer in bare["layers"]:
        for key in ("rank", "decay_rank", "gate_rank"):
            layer["mixer"].pop(key, None)
    params = load_model_dir(folder, CausalLM(_spec(bare)[2]).param_specs(), engine_dtype=torch.float32, device="cpu")
    assert params["layers.1.mixer.decay_in"].shape == (8, 96) and params["layers.1.mixer.decay_out"].shape == (64, 8)
    assert params["layers.1.mixer.gate_in"].shape == (6, 96) and params["layers.1.mixer.gate_out"].shape == (96, 6)
    assert params["layers.2.mixer.decay_in"].shape == (8, 96)
    with pytest.raises(ValueError):
        write_random_model(bare, 1, tmp_path / "bare")
    other = copy.deepcopy(cfg)
    other["layers"][1]["mixer"]["gate_rank"] = 5
    with pytest.raises(WeightsError):
        load_model_dir(folder, CausalLM(_spec(other)[2]).param_specs(), engine_dtype=torch.float32, device="cpu")
    written = write_random_model(cfg, 3, tmp_path / "drawn")
    assert set(tensor_shapes(cfg)) == set(__import__("safetensors.torch", fromlist=["load_file"]).load_file(
        str(written / "model.safetensors")))


def test_a_norm_without_a_feed_forward_behind_it_is_dropped_unread(tmp_path):
    from rapid_llm_amd.models.causal_lm import CausalLM
    from rapid_llm_amd.weights.loader import WeightsError, load_model_dir

    cfg, _page, seed = PEFU["A"]
    _entry, _typed, spec = _spec(cfg)
    weights = make_weights(cfg, seed)
    weights["l1.norm2"] = torch.zeros(96, dtype=torch.bfloat16)  # layer 1 has no feed-forward
    folder = make_model_dir(tmp_path, "A", weights=weights)
    load_model_dir(folder, CausalLM(spec).param_specs(), engine_dtype=torch.float32, device="cpu",
                   ignore_rules=spec.ignore_tensors)
    weights["l1.norm3"] = torch.zeros(96, dtype=torch.bfloat16)
    folder = make_model_dir(tmp_path, "A", weights=weights)
    with pytest.raises(WeightsError):
        load_model_dir(folder, CausalLM(spec).param_specs(), engine_dtype=torch.float32, device="cpu",
                       ignore_rules=spec.ignore_tensors)


def test_cache_needs_one_cache_or_state_for_every_run():
    from rapid_llm_amd.models.causal_lm import CausalLM

    needs = CausalLM(_spec(PEFU["A"][0])[2]).cache_needs()
    assert [n.kind for n in needs] == ["paged", "state", "state", "state", "state", "paged"]
    assert {p.name: p.shape for p in needs[0].paged} == {"k": (2, 16), "v": (2, 32)} and needs[0].window == 0
    assert {s.name: s.shape for s in needs[0].state_specs()} == {"right.S": (40,)}
    for run in (1, 3):
        assert {s.name: s.shape for s in needs[run].states} == {"conv": (2, 2 * 2 * 16 + 4 * 24), "S": (4, 24, 16)}
        assert {s.name: s.shape for s in needs[run + 1].states} == {"shift": (96,), "S": (3, 16, 16)}
    assert all(s.dtype == "float32" for n in needs for s in n.state_specs())
    assert all(n.share_with is None for n in needs)


# --------------------------------------------------------------------------- #
# the plain implementation
# --------------------------------------------------------------------------- #


def test_plain_mechanisms_one_by_one():
    """Each mechanism of the plain implementation on inputs whose answer is known."""
    # delta rule: the read-out sees the token's own write; a key written again replaces its value;
    # the decay acts on the key channels before anything else
    e = torch.eye(2, dtype=D64)
    k = torch.stack([e[0], e[0], e[1], e[0]]).view(4, 1, 2)
    v = torch.tensor([[3.0], [5.0], [7.0], [5.0]], dtype=D64).view(4, 1, 1)
    q = torch.stack([e[0], e[0], e[0] + e[1], e[0]]).view(4, 1, 2)
    g = torch.ones(4, 1, 2, dtype=D64)
    g[3, 0, 0] = 0.5
    one = torch.ones(4, 1, dtype=D64)
    assert pp.delta_rule(q, k, v, g, one).flatten().tolist() == [3.0, 5.0, 12.0, 5.0]
    half = pp.delta_rule(q, k, v, g, 0.5 * one).flatten()
    # 1.5; 1.5 + (5 - 1.5)/2 = 3.25; 3.25 + 3.5; decayed to 1.625, then half way to 5
    assert torch.allclose(half, torch.tensor([1.5, 3.25, 6.75, 1.625 + 0.5 * (5 - 1.625)], dtype=D64))
    # convolution: the last tap meets the current token, zeros before the start
    y = pp.short_convolution(torch.tensor([[1.0], [10.0], [100.0]], dtype=D64), torch.tensor([[2.0, 0.0, 3.0]], dtype=D64))
    assert torch.allclose(y, pp.silu(torch.tensor([[3.0], [30.0], [302.0]], dtype=D64)))
    # temperature: steps where p + 1 reaches a multiple
    t = pp.temperature(torch.arange(8), 0.5, 4)
    assert torch.allclose(t[:3], torch.ones(3, dtype=D64))
    assert torch.allclose(t[3:7], torch.full((4,), 1 + 0.5 * math.log(2), dtype=D64))
    assert abs(float(t[7]) - (1 + 0.5 * math.log(3))) < 1e-12
    # minGRU: with z = 1/2 and u = 0 the candidate is 1/2 on both branches
    w = {"z": torch.zeros(1, 1, dtype=D64), "z.b": torch.zeros(1, dtype=D64), "x": torch.ones(1, 1, dtype=D64),
         "x.b": torch.zeros(1, dtype=D64), "g": torch.zeros(1, 1, dtype=D64), "o": torch.ones(1, 1, dtype=D64)}
    h = torch.tensor([[0.0], [2.0], [-2.0]], dtype=D64)
    gate = pp.silu(torch.tensor(1.0, dtype=D64))
    w["g.b"] = torch.ones(1, dtype=D64)
    s0 = 0.25
    s1 = 0.5 * s0 + 0.5 * 2.5
    s2 = 0.5 * s1 + 0.5 / (1 + math.exp(2.0))
    assert torch.allclose(pp.min_gru({"width": 1}, w, "", h).flatten(), torch.tensor([s0, s1, s2], dtype=D64) * gate)
    # the distance term of a head whose keys all score alike: weights (1 + r2 n)^-r1
    m = {"heads": 1, "kv_heads": 1, "dim": 1, "vdim": 2, "scale": 1.0}
    w = {"q": torch.zeros(1, 2, dtype=D64), "k": torch.zeros(1, 2, dtype=D64), "v": torch.eye(2, dtype=D64),
         "q.norm": torch.ones(1, dtype=D64), "k.norm": torch.ones(1, dtype=D64), "o": torch.eye(2, dtype=D64),
         "r1": torch.tensor([2.0], dtype=D64), "r2": torch.tensor([0.5], dtype=D64)}
    h = torch.tensor([[1.0, 0.0], [0.0, 3.0], [1.0, 0.0]], dtype=D64)
    root2 = math.sqrt(2.0)  # a value head divided by its root mean square has norm sqrt(2)
    far, mid, own = 2.0**-2, 1.5**-2, 1.0
    out = pp.distance_attention(m, w, "", h, 1e-12)[2]
    assert torch.allclose(out, root2 * torch.tensor([far + own, mid], dtype=D64) / (far + mid + own))


# faults a comparison is there for: a function of the plain implementation replaced by a wrong one
def _read_before_write(q, k, v, g, beta):
    S = torch.zeros(k.shape[1], k.shape[2], v.shape[2], dtype=D64)
    out = torch.zeros(k.shape[0], k.shape[1], v.shape[2], dtype=D64)
    for t in range(k.shape[0]):
        S = g[t].unsqueeze(-1) * S
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
        u = beta[t].unsqueeze(-1) * (v[t] - (S * k[t].unsqueeze(-1)).sum(1))
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(-2)
    return out


def _decay_after_write(q, k, v, g, beta):
    S = torch.zeros(k.shape[1], k.shape[2], v.shape[2], dtype=D64)
    out = torch.zeros(k.shape[0], k.shape[1], v.shape[2], dtype=D64)
    for t in range(k.shape[0]):
        u = beta[t].unsqueeze(-1) * (v[t] - (S * k[t].unsqueeze(-1)).sum(1))
        S = g[t].unsqueeze(-1) * (S + k[t].unsqueeze(-1) * u.unsqueeze(-2))
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out


_RIGHT = {name: getattr(pp, name) for name in ("delta_rule", "temperature", "short_convolution", "passes", "gelu_tanh")}
WRONG = {
    "the read-out misses the token's own write": ("delta_rule", _read_before_write),
    "the decay after the write": ("delta_rule", _decay_after_write),
    "one decay a head": ("delta_rule", lambda q, k, v, g, b: _RIGHT["delta_rule"](q, k, v, g.mean(-1, keepdim=True).expand_as(g), b)),
    "an additive write": ("delta_rule", lambda q, k, v, g, b: _RIGHT["delta_rule"](q, 0.01 * k, 100 * v, g, b)),
    "the temperature one position late": ("temperature", lambda p, c, e: _RIGHT["temperature"](p - 1, c, e)),
    "no temperature": ("temperature", lambda p, c, e: torch.ones(p.shape[0], dtype=D64)),
    "a convolution that forgets the oldest tap": (
        "short_convolution",
        lambda x, taps: _RIGHT["short_convolution"](x, torch.cat([torch.zeros_like(taps[:, :1]), taps[:, 1:]], 1))),
    "the embedding does not return": ("passes", lambda cfg: [(i, None if t is None else -t) for i, t in _RIGHT["passes"](cfg)]),
    "vectors not unit": ("unit", lambda x: x),
    "silu for gelu": ("gelu_tanh", lambda z: z * torch.sigmoid(z)),
    "norm weights as they are": ("around_one_norm", lambda x, w, eps: pp.rms(x, eps) * w),
}


@pytest.mark.parametrize("fault", sorted(WRONG))
def test_plain_tells_a_wrong_mechanism(fault, monkeypatch):
    """With the tests' weights each fault moves some row by at least fifty times what the float32
    comparison allows."""
    cfg, _page, seed = PEFU["A"]
    w = make_weights(cfg, seed, sharp=3.0)
    toks = random_tokens(60, cfg["vocab"], 9)
    want = pp.forward(cfg, w, toks)
    monkeypatch.setattr(pp, *WRONG[fault])
    assert float(row_errors(pp.forward(cfg, w, toks), want).max()) > 50 * F32_ROW


def test_plain_tells_wrong_constants_and_lost_tensors():
    cfg, _page, seed = PEFU["A"]
    w = make_weights(cfg, seed, sharp=3.0)
    toks = random_tokens(60, cfg["vocab"], 9)
    want = pp.forward(cfg, w, toks)
    assert float(row_errors(pp.forward(cfg, w, toks, cast=bf16_round), want).max()) < 0.1

    def shows(c, weights):
        return float(row_errors(pp.forward(c, weights, toks), want).max()) > 50 * F32_ROW

    for change in (
        lambda c: c["layers"][0]["mixer"].update(left_scale=1.0),
        lambda c: c["layers"][0]["mixer"].update(right_scale=1.0),
        lambda c: c["layers"][0]["mixer"]["left"].update(scale=0.25),
        lambda c: c["layers"][0]["mixer"]["left"]["q_temp"].update(every=8),
        lambda c: c["layers"][3]["mixer"]["left"].update(q_temp={"coef": 0.1, "every": 7}),
        lambda c: c.update(loop=None),
    ):
        c = copy.deepcopy(cfg)
        change(c)
        assert shows(c, w)
    lost = [n for n in tensor_shapes(cfg) if n.endswith((".b", "r1", "r2", "u", "w0", "dt_bias", "A_log", "loop.step")) or ".mu." in n]
    for name in lost:
        w2 = dict(w)
        w2[name] = torch.zeros_like(w[name])
        assert shows(cfg, w2), name


def test_plain_shows_a_state_that_is_not_carried():
    """A different first token changes the logits far behind it, and so does a state that starts
    anew in the middle: the comparison over cut requests sees both."""
    cfg, _page, seed = PEFU["A"]
    w = make_weights(cfg, seed)
    toks = random_tokens(150, cfg["vocab"], 12)
    want = pp.forward(cfg, w, toks)
    other = pp.forward(cfg, w, [(toks[0] + 1) % cfg["vocab"]] + toks[1:])
    assert float(row_errors(other[-1:], want[-1:]).max()) > 50 * F32_ROW
    anew = pp.forward(cfg, w, toks[75:])
    assert float(row_errors(anew[-1:], want[-1:]).max()) > 50 * F32_ROW
