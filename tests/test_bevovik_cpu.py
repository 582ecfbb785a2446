"""What pins the plain form of Bevovik (tests/plain/bevovik.py) without any library's model code, and the
parts of the framework that need no GPU: each mechanism against numbers worked out by hand or a second
writing, the whole model's causality, the configuration reader, the tensor names, what the caches keep."""

import copy
import math

import pytest
import torch

from .plain import bevovik as P
from .tiny_bevovik import BEV_A, BEV_B, BEV_C, CONFIGS

torch.manual_seed(0)
F64 = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed + sum(shape)), dtype=F64)


def test_small_functions_by_hand():
    z = torch.tensor([-800.0, -2.0, 0.0, 3.0, 800.0], dtype=F64)
    got = P.log_sigmoid(z)
    assert torch.isfinite(got).all() and got[0] == -800.0 and abs(float(got[2]) + math.log(2)) < 1e-15
    assert torch.allclose(got[1:4], torch.log(1 / (1 + torch.exp(-z[1:4])))) and abs(float(P.softplus(z)[3]) - math.log(1 + math.e**3)) < 1e-12
    assert abs(float(P.gelu_tanh(torch.tensor(1.5, dtype=F64))) - 0.75 * (1 + math.tanh(math.sqrt(2 / math.pi) * (1.5 + 0.044715 * 3.375)))) < 1e-15
    assert torch.allclose(P.unit_rms(torch.tensor([[3.0, 4.0]], dtype=F64), 0.5), torch.tensor([[3.0, 4.0]], dtype=F64) / math.sqrt(13.0))


def test_gated_linear_attention_against_the_unrolled_sum():
    m = {"heads": 2, "dim": 3, "vdim": 4, "tau": 5.0}
    n, width, eps = 6, 5, 1e-3
    w = {"p.q": rnd(6, width), "p.k": rnd(6, width, seed=1), "p.v": rnd(8, width), "p.g": rnd(8, width, seed=2), "p.a1": rnd(2, width),
         "p.a2": rnd(6, 2), "p.a2.b": rnd(6), "p.norm": rnd(4) + 2, "p.o": torch.eye(8, dtype=F64)}
    h = rnd(n, width, seed=5)
    got = P.gated_linear_attention(h, w, "p", m, eps).view(n, 2, 4)
    for a in range(2):
        for t in range(n):
            o = torch.zeros(4, dtype=F64)
            for s in range(t + 1):
                dot = 0.0
                for d in range(3):
                    row = a * 3 + d
                    fade = 1.0
                    for r in range(s + 1, t + 1):  # the decays of the tokens after s, up to and with t's
                        z = float(w["p.a2"][row] @ (w["p.a1"] @ h[r]) + w["p.a2.b"][row])
                        fade *= (1 / (1 + math.exp(-z))) ** (1 / 5.0)
                    dot += float(w["p.q"][row] @ h[t]) / math.sqrt(3.0) * float(w["p.k"][row] @ h[s]) * fade
                o += dot * (w["p.v"][a * 4 : a * 4 + 4] @ h[s])
            g = w["p.g"][a * 4 : a * 4 + 4] @ h[t]
            want = o / math.sqrt(float((o * o).mean()) + eps) * w["p.norm"] * g / (1 + torch.exp(-g))
            assert torch.allclose(got[t, a], want), (t, a)


def test_turn_rates_by_hand():
    rates, factor = P.turn_rates({"base": 10000.0, "dims": 8})
    assert factor == 1.0 and torch.allclose(rates, torch.tensor([1.0, 0.1, 0.01, 0.001], dtype=F64))
    # 16 turns in 1,000 positions belong to pair 0.998 (down to 0), one turn to pair 2.20 (up to 3)
    rates, factor = P.turn_rates({"base": 10000.0, "dims": 8, "scaling": {"factor": 4.0, "original": 1000, "fast": 16.0, "slow": 1.0}})
    assert abs(factor - (0.1 * math.log(4.0) + 1.0)) < 1e-15
    want = [p / 4 * r + p * (1 - r) for p, r in zip((1.0, 0.1, 0.01, 0.001), (0, 1 / 3, 2 / 3, 1))]
    assert torch.allclose(rates, torch.tensor(want, dtype=F64))


@pytest.mark.parametrize("base, dims, scaling", [(10000.0, 8, (4.0, 1000, 16.0, 1.0)), (500.0, 20, (2.0, 64, 8.0, 2.0)),
                                                 (1e6, 64, (8.0, 4096, 32.0, 1.0)), (10000.0, 4, (2.0, 4, 64.0, 32.0)),
                                                 (300.0, 6, (1.0, 10, 3.0, 1.0))])
def test_the_engines_stretched_rates_are_the_plain_ones(base, dims, scaling):
    from shrike_amd.parts.rotary import yarn_rates

    rates, magnitude = yarn_rates(base, dims, *scaling)
    want, factor = P.turn_rates({"base": base, "dims": dims, "scaling": dict(zip(("factor", "original", "fast", "slow"), scaling))})
    assert torch.allclose(torch.tensor(rates, dtype=F64), want, rtol=1e-14, atol=0) and abs(magnitude - factor) < 1e-15


def test_rotation_is_a_complex_turn_of_neighbours_times_a_factor():
    x, pos = rnd(5, 3, 10), torch.tensor([0, 1, 7, 100, 3])
    rot = {"base": 50.0, "dims": 10, "scaling": {"factor": 3.0, "original": 40, "fast": 4.0, "slow": 1.0}}
    rates, factor = P.turn_rates(rot)
    z = torch.complex(x[..., 0::2], x[..., 1::2]) * torch.polar(torch.full((5, 1, 5), factor, dtype=F64), pos[:, None, None] * rates)
    got = P.rotate_pairs(x, pos, rot)
    assert torch.allclose(got[..., 0::2], z.real) and torch.allclose(got[..., 1::2], z.imag)


def test_one_head_of_latent_attention_by_hand():
    m = {"heads": 2, "dim": 3, "rot_dim": 2, "vdim": 4, "q_rank": 5, "kv_rank": 6, "scale": 0.7,
         "rot": {"base": 10.0, "dims": 2, "scaling": {"factor": 2.0, "original": 100, "fast": 8.0, "slow": 1.0}}}
    n, width, eps = 5, 7, 1e-2
    w = {"p.dq": rnd(5, width), "p.dq.norm": rnd(5) + 2, "p.uq": rnd(10, 5), "p.dkv": rnd(8, width), "p.dkv.norm": rnd(6) + 2,
         "p.uk": rnd(6, 6), "p.uv": rnd(8, 6), "p.o": torch.eye(8, dtype=F64)}
    h = rnd(n, width, seed=3)
    got = P.latent_attention(h, torch.arange(n), w, "p", m, eps)
    rms = lambda x: x / math.sqrt(float((x * x).mean()) + eps)  # noqa: E731
    rates, factor = P.turn_rates(m["rot"])

    def turned(v, t):
        c, s = math.cos(t * float(rates[0])) * factor, math.sin(t * float(rates[0])) * factor
        return torch.stack([v[0] * c - v[1] * s, v[1] * c + v[0] * s])

    head, i = 1, 4
    q = w["p.uq"][5:10] @ (rms(w["p.dq"] @ h[i]) * w["p.dq.norm"])
    e = []
    for j in range(i + 1):
        down = w["p.dkv"] @ h[j]
        c = rms(down[:6]) * w["p.dkv.norm"]
        score = float(q[:3] @ (w["p.uk"][3:6] @ c) + turned(q[3:], i) @ turned(down[6:], j)) * 0.7
        e.append((math.exp(score), w["p.uv"][4:8] @ c))
    want = sum(x * v for x, v in e) / sum(x for x, _ in e)
    assert torch.allclose(got[i, 4:8], want)


def test_causal_convolution_by_hand():
    x = torch.tensor([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0]], dtype=F64)
    taps = torch.tensor([[100.0, 10.0, 1.0, 1000.0], [0.0, 0.0, 0.0, 2.0]], dtype=F64)  # the last meets the current token
    got = P.causal_convolution(x, taps, torch.tensor([0.5, -1.0], dtype=F64))
    assert got[:, 0].tolist() == [1000.5, 2001.5, 3012.5] and got[:, 1].tolist() == [19.0, 39.0, 59.0]


def test_gated_recurrence_position_by_position():
    m = {"width": 6, "blocks": 3, "conv": 3}
    n, width = 7, 4
    w = {"p.y": rnd(6, width), "p.y.b": rnd(6), "p.x": rnd(6, width, seed=1), "p.x.b": rnd(6, seed=1), "p.conv": rnd(6, 3), "p.conv.b": rnd(6, seed=2),
         "p.ra": rnd(3, 2, 2), "p.ra.b": rnd(3, 2), "p.ri": rnd(3, 2, 2, seed=1), "p.ri.b": rnd(3, 2, seed=1), "p.lam": rnd(6, seed=3) - 2,
         "p.o": torch.eye(6, dtype=F64)}
    h = rnd(n, width, seed=4)
    got = P.gated_recurrence(h, w, "p", m)
    sig = lambda z: 1 / (1 + math.exp(-z))  # noqa: E731
    x = h @ w["p.x"].T + w["p.x.b"]
    u = torch.stack([w["p.conv.b"] + sum(w["p.conv"][:, 2 - k] * x[t - k] for k in range(3) if t >= k) for t in range(n)])
    for c in (0, 3, 5):
        b, o, S = c // 2, c % 2, 0.0
        for t in range(n):
            r = sig(float(w["p.ra"][b, o] @ u[t, 2 * b : 2 * b + 2] + w["p.ra.b"][b, o]))
            i = sig(float(w["p.ri"][b, o] @ u[t, 2 * b : 2 * b + 2] + w["p.ri.b"][b, o]))
            a = math.exp(-8.0 * r * math.log(1 + math.exp(float(w["p.lam"][c]))))
            S = a * S + math.sqrt(1 - a * a) * i * float(u[t, c])  # (the first token too)
            y = float(P.gelu_tanh(w["p.y"][c] @ h[t] + w["p.y.b"][c]))
            assert abs(float(got[t, c]) - S * y) < 1e-12


def test_expert_by_hand():
    w = {"p.gate": torch.tensor([[1.0, 0.0], [0.0, 1.0]], dtype=F64), "p.up": torch.tensor([[0.0, 1.0], [1.0, 0.0]], dtype=F64),
         "p.down": torch.tensor([[1.0, 10.0]], dtype=F64)}
    got = float(P.expert(torch.tensor([[5.0, -4.0]], dtype=F64), w, "p", 2.0))
    act = lambda g: g / (1 + math.exp(-1.702 * g))  # noqa: E731
    # g = (2, -4): bounded from above alone; u = (-2, 2): from both sides
    assert abs(got - (act(2.0) * (-2.0 + 1.0) + 10 * act(-4.0) * (2.0 + 1.0))) < 1e-12


def test_choice_among_groups_by_hand():
    scores = torch.tensor([0.30, 0.01, 0.20, 0.19, 0.10, 0.20], dtype=F64)
    none = torch.zeros(6, dtype=F64)
    assert P.choose(scores, none, 2, 1, 1) == [0, 2]  # one group: the largest, of equal ones the first
    assert P.choose(scores, none, 2, 3, 1) == [0, 1]  # only the best entry's group, however small its other
    assert P.choose(scores, none, 3, 3, 2) == [0, 2, 3]
    correction = torch.tensor([-1.0, -1.0, -0.5, -2.0, -0.9, -3.0], dtype=F64)
    # negative choice scores all over: entries of other groups are out, not zero
    assert P.choose(scores, correction, 2, 3, 1) == [2, 3]
    assert P.choose(scores, correction, 2, 1, 1) == [2, 0]


def test_mixture_weights_and_identity_experts_by_hand():
    m = {"router": {"experts": 1, "identity": 2, "top": 2, "scale": 3.0, "groups": {"count": 1, "keep": 1}}, "expert": {"ff": 1, "limit": 9.0}}
    w = {"p.router": torch.tensor([[0.0, 0.0], [1.0, 0.0], [0.0, 1.0]], dtype=F64), "p.correction": torch.tensor([5.0, 0.0, 0.0], dtype=F64),
         "p.e0.gate": torch.tensor([[1.0, 0.0]], dtype=F64), "p.e0.up": torch.tensor([[0.0, 1.0]], dtype=F64),
         "p.e0.down": torch.tensor([[1.0], [-1.0]], dtype=F64)}
    h = torch.tensor([[2.0, 1.0]], dtype=F64)
    s = torch.softmax(torch.tensor([0.0, 2.0, 1.0], dtype=F64), 0)
    # the correction brings the expert in, its weight is its small score; the better identity is the other
    y = 2.0 / (1 + math.exp(-1.702 * 2.0)) * 2.0
    want = 3.0 * (s[0] * torch.tensor([y, -y]) + s[1] * h[0]) / (s[0] + s[1])
    assert torch.allclose(P.mixture(h, w, "p", m)[0], want)
    w["p.shared.gate"], w["p.shared.up"], w["p.shared.down"] = w["p.e0.gate"], w["p.e0.up"], w["p.e0.down"]
    got = P.mixture(h, w, "p", {**m, "shared": {"ff": 1, "limit": 0.5}})[0]
    bounded = 0.5 / (1 + math.exp(-1.702 * 0.5)) * 1.5
    assert torch.allclose(got, want + torch.tensor([bounded, -bounded]))


def _random_model(cfg, seed=3):
    from shrike_amd.models import DecoderModel
    from shrike_amd.models.bevovik import BevovikConfig, build_spec
    from shrike_amd.weights.random_init import random_tensors

    model = DecoderModel(build_spec(BevovikConfig.from_dict(cfg)))
    return model, {k: v.to(F64) for k, v in random_tensors(model.params(), seed, torch.float32, mode="unit").items()}


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_the_model_is_causal_and_every_layer_moves_the_stream(name):
    cfg = CONFIGS[name]
    _model, w = _random_model(cfg)
    ids = [i * 7 % cfg["vocab"] for i in range(30)]
    logits, streams = P.forward(cfg, w, ids, return_layers=True)
    changed = list(ids)
    changed[20] = (changed[20] + 1) % cfg["vocab"]
    other = P.forward(cfg, w, changed)
    assert torch.allclose(other[:20], logits[:20]) and float((other[20:] - logits[20:]).abs().max()) > 1e-3
    assert float((other[29] - logits[29]).abs().max()) > 1e-4 * float(logits[29].abs().max()), "nine tokens on it still shows"
    assert streams.shape[0] == len(cfg["layers"])
    for a, b in zip(streams[:-1], streams[1:]):
        assert float((b - a).abs().mean()) > 1e-2 * float(a.abs().mean())


def test_a_layer_adds_its_normed_and_scaled_outputs():
    cfg = {**BEV_A, "layers": BEV_A["layers"][:1]}
    _model, w = _random_model(cfg)
    ids = [3, 1, 4, 1, 5]
    _, streams = P.forward(cfg, w, ids, return_layers=True)
    x = w["embed"][torch.tensor(ids)]
    y = P.gated_recurrence(x, w, "l0.mix", cfg["layers"][0]["mixer"])
    x = x + y / torch.sqrt((y * y).mean(-1, keepdim=True) + 1e-5) * w["l0.norm1"] * w["l0.ls1"]
    f = P.mixture(x, w, "l0.mlp", cfg["layers"][0]["mlp"])
    assert torch.allclose(streams[0], x + f / torch.sqrt((f * f).mean(-1, keepdim=True) + 1e-5) * w["l0.norm2"] * w["l0.ls2"])


def test_configuration_round_trip_and_names():
    from shrike_amd.config import get_architecture
    from shrike_amd.models.bevovik import BevovikConfig

    for cfg in CONFIGS.values():
        parsed = BevovikConfig.from_dict(cfg)
        assert BevovikConfig.from_dict(parsed.to_dict()) == parsed
    assert get_architecture("Bevovik").config_cls is BevovikConfig
    model, _ = _random_model(BEV_A)
    names = {p.name: tuple(p.shape) for p in model.params()}
    assert names["embed"] == (211, 70) and names["head"] == (211, 70) and names["final.norm"] == (70,)
    assert names["l0.mix.y"] == (96, 70) and names["l0.mix.x.b"] == (96,) and names["l0.mix.conv"] == (96, 4)
    assert names["l0.mix.ra"] == (3, 32, 32) and names["l0.mix.ri.b"] == (3, 32) and names["l0.mix.lam"] == (96,)
    assert names["l0.mlp.router"] == (6, 70) and names["l0.mlp.correction"] == (6,) and "l0.mlp.e5.up" not in names
    assert names["l0.mlp.e4.down"] == (70, 24) and names["l0.mlp.shared.gate"] == (40, 70) and names["l0.ls2"] == (70,)
    assert names["l1.mix.a1"] == (5, 70) and names["l1.mix.a2"] == (60, 5) and names["l1.mix.a2.b"] == (60,) and names["l1.mix.norm"] == (12,)
    assert names["l2.mix.uq"] == (3 * 32, 40) and names["l2.mix.dkv"] == (40, 70) and "l2.mix.g" not in names
    loose = {p.name for p in model.params() if p.optional}
    assert loose == {"l2.norm2", "l2.ls2"}, "a layer without a feed-forward needs no second norm"
    assert model.launches_follow_shape() and model.graph_safe()


def test_the_rank_of_the_decays_product_is_the_files():
    """Without decay_rank the two matrices' common size is whatever the tensors have."""
    from shrike_amd.models import DecoderModel
    from shrike_amd.models.bevovik import BevovikConfig, build_spec

    cfg = copy.deepcopy(BEV_A)
    del cfg["layers"][1]["mixer"]["decay_rank"]
    params = {p.name: p for p in DecoderModel(build_spec(BevovikConfig.from_dict(cfg))).params()}
    assert params["l1.mix.a1"].matches((9, 70)) and params["l1.mix.a2"].matches((60, 9)) and not params["l1.mix.a1"].matches((9, 71))


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0]["mixer"].pop("conv"), "conv"),
    (lambda c: c["layers"][0]["mixer"].update(blocks=7), "multiple"),
    (lambda c: c["layers"][1]["mixer"].update(tau=0), "positive"),
    (lambda c: c["layers"][2]["mixer"].update(rot_dim=7), "even"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=4), "equal to rot_dim"),
    (lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][2]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "equal groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "kept"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "can be chosen"),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0), "positive"),
    (lambda c: c["layers"][0]["mlp"]["shared"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1), "negative"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "unknown feed-forward"),
    (lambda c: c["layers"][0].update(type="attention"), "unknown mixer"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_configuration_errors_say_what_is_wrong(change, text):
    from shrike_amd.config import ConfigError
    from shrike_amd.models.bevovik import BevovikConfig

    cfg = copy.deepcopy(BEV_A)
    change(cfg)
    with pytest.raises(ConfigError, match=text):
        BevovikConfig.from_dict(cfg)


def test_what_the_caches_keep():
    from shrike_amd.cache import CacheManager
    from shrike_amd.parts import PagedSpec, StateSpec

    for cfg in (BEV_A, BEV_B, BEV_C):
        model, _ = _random_model(cfg)
        for spec, layer in zip(model.cache_specs(), cfg["layers"]):
            m = layer["mixer"]
            if layer["type"] == "gla":
                assert spec == StateSpec((m["heads"] * m["dim"] * m["vdim"],))
            elif layer["type"] == "rglru":
                assert spec == StateSpec((m["width"] * m["conv"],)), "the state and the convolution's last inputs"
            else:
                assert isinstance(spec, PagedSpec) and spec.window is None and spec.tensors[0].dims[1] == m["kv_rank"] + m["rot_dim"]
    manager = CacheManager(_random_model(BEV_B)[0].cache_specs(), 4, 8, max_slots=2)
    assert len(manager.groups) == 2 and len(manager.state_groups) == 3 and not manager.enable_prefix_caching


def test_random_weights_reach_every_tensor_and_long_memories():
    """Rates of the recurrence are small enough that a state outlives hundreds of tokens in some channels."""
    _model, w = _random_model(BEV_C)
    slow = P.softplus(w["l1.mix.lam"]) * 8 * 0.5
    assert float(slow.min()) < 5e-3 and float(slow.max()) > 5e-2
