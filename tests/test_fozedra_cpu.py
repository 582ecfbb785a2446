"""What pins the plain form of Fozedra (tests/plain/fozedra.py) without any library's model code, and
the parts of the framework that need no GPU: each mechanism against numbers worked out by hand or a
second writing, the whole model's causality, the configuration reader, the tensor names, the schedule,
what the caches keep and give back."""

import copy
import math

import pytest
import torch

from .plain import fozedra as P
from .tiny_fozedra import CONFIGS, FOZ_A, FOZ_B, FOZ_C

torch.manual_seed(0)
F64 = torch.float64


def test_dynamic_tanh_by_hand():
    w = {"n": torch.tensor([2.0, 3.0], dtype=F64), "n.b": torch.tensor([0.5, -1.0], dtype=F64), "n.alpha": torch.tensor(0.25, dtype=F64)}
    got = P.dynamic_tanh(torch.tensor([[4.0, -8.0]], dtype=F64), w, "n")
    assert torch.allclose(got, torch.tensor([[2 * math.tanh(1.0) + 0.5, -3 * math.tanh(2.0) - 1.0]], dtype=F64))


def test_masks_written_out():
    vis = P.visible(6, {"size": 2, "keep_first": 1}).int().tolist()
    assert vis == [[1, 0, 0, 0, 0, 0], [1, 1, 0, 0, 0, 0], [1, 1, 1, 0, 0, 0], [1, 0, 1, 1, 0, 0], [1, 0, 0, 1, 1, 0],
                   [1, 0, 0, 0, 1, 1]]
    assert P.visible(4, {"size": 1, "keep_first": 0}).int().tolist() == torch.eye(4, dtype=torch.int).tolist()
    assert torch.equal(P.visible(5, None), P.visible(5, {"size": 1, "keep_first": 9}))


def test_short_convolution_by_hand():
    u = torch.tensor([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0], [4.0, 40.0]], dtype=F64)
    taps = torch.tensor([[100.0, 10.0, 1.0], [0.0, 0.0, 2.0]], dtype=F64)  # the last meets the current token
    got = P.short_convolution(u, taps)
    assert got[:, 0].tolist() == [1.0, 12.0, 123.0, 234.0] and got[:, 1].tolist() == [20.0, 40.0, 60.0, 80.0]
    wide = torch.nn.functional.conv1d(torch.nn.functional.pad(u.T[None], (2, 0)), taps[:, None], groups=2)[0].T
    assert torch.allclose(got, wide)


def test_rotation_rates_by_hand():
    rates, factor = P.rotation_rates({"base": 10000.0, "dims": 8})
    assert factor == 1.0 and torch.allclose(rates, torch.tensor([1.0, 0.1, 0.01, 0.001], dtype=F64))
    # 8 elements, base 10^4, 1,000 positions: 16 turns at 2 i = 8 ln(1000 / (32 pi)) / ln(10^4) -> pair 0.998,
    # down to 0; one turn at pair 2.20, up to 3: pairs 0 .. 3 pass in thirds
    rates, factor = P.rotation_rates({"base": 10000.0, "dims": 8,
                                      "scaling": {"factor": 4.0, "original": 1000, "fast": 16.0, "slow": 1.0}})
    assert abs(factor - (0.1 * math.log(4.0) + 1.0)) < 1e-15
    plain = [1.0, 0.1, 0.01, 0.001]
    assert torch.allclose(rates, torch.tensor([p / 4 * r + p * (1 - r) for p, r in zip(plain, (0, 1 / 3, 2 / 3, 1))], dtype=F64))
    # both ends beyond the pairs there are: clamped to 0 and dims - 1, and a span of nothing is a step
    rates, _ = P.rotation_rates({"base": 10000.0, "dims": 4, "scaling": {"factor": 2.0, "original": 4, "fast": 64.0, "slow": 32.0}})
    assert torch.allclose(rates, torch.tensor([1.0, 0.005], dtype=F64))


@pytest.mark.parametrize("base, dims, scaling", [(10000.0, 8, (4.0, 1000, 16.0, 1.0)), (500.0, 20, (2.0, 64, 8.0, 2.0)),
                                                 (1e6, 64, (8.0, 4096, 32.0, 1.0)), (30.0, 6, (1.0, 10, 3.0, 1.0)),
                                                 (10000.0, 4, (2.0, 4, 64.0, 32.0))])
def test_the_engines_stretched_rates_are_the_plain_ones(base, dims, scaling):
    from shrike_amd.parts.rotary import yarn_rates

    rates, magnitude = yarn_rates(base, dims, *scaling)
    want, factor = P.rotation_rates({"base": base, "dims": dims, "scaling": dict(zip(("factor", "original", "fast", "slow"), scaling))})
    assert torch.allclose(torch.tensor(rates, dtype=F64), want, rtol=1e-14, atol=0) and abs(magnitude - factor) < 1e-15


def test_rotation_is_a_complex_turn_of_halves():
    x = torch.randn(5, 3, 10, dtype=F64)
    pos = torch.tensor([0, 1, 7, 100, 3])
    rot = {"base": 50.0, "dims": 6}
    got = P.rotate_halves(x, pos, rot)
    z = torch.complex(x[..., :3], x[..., 3:6]) * torch.polar(torch.ones(5, 1, 3, dtype=F64), (pos[:, None] * 50.0 ** (-torch.arange(3, dtype=F64) / 3))[:, None])
    assert torch.allclose(got, torch.cat([z.real, z.imag, x[..., 6:]], -1))
    assert torch.equal(P.rotate_halves(x, pos, None), x)


def _weights(m, width=8, seed=0):
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=F64)  # noqa: E731
    w, rows = {}, {"q": m["heads"] * 2 * m["dim"], "k": m["kv_heads"] * 2 * m["dim"], "v": m["kv_heads"] * m["vdim"]}
    for r, n in rows.items():
        w[f"p.{r}"], w[f"p.{r}.b"] = rnd(n, width), rnd(n)
        if m.get("conv"):
            w[f"p.{r}.conv"] = rnd(n, m["conv"])
    for r in ("lq1", "lk1", "lq2", "lk2"):
        w[f"p.{r}"] = rnd(m["dim"]) * 0.3
    w["p.g"], w["p.o"] = rnd(m["heads"], width), torch.eye(m["heads"] * m["vdim"], dtype=F64)
    return w


def test_one_head_of_differential_attention_position_by_position():
    m = {"heads": 4, "kv_heads": 2, "dim": 3, "vdim": 5, "scale": 0.6, "diff": 0.3, "conv": 2, "mask": {"size": 3, "keep_first": 1},
         "rot": {"base": 20.0, "dims": 2}}
    w, n, eps = _weights(m), 7, 1e-3
    h = torch.randn(n, 8, dtype=F64)
    got, (k, v) = P.differential_attention(h, torch.arange(n), w, "p", m, eps)

    def channel(name, row, t):  # projection with its bias, two taps
        y = lambda s: float(w[f"p.{name}"][row] @ h[s] + w[f"p.{name}.b"][row]) if s >= 0 else 0.0  # noqa: E731
        return float(w[f"p.{name}.conv"][row, 1]) * y(t) + float(w[f"p.{name}.conv"][row, 0]) * y(t - 1)

    def turned(name, head, mp, t):  # 3 elements, the first two a pair that turns by the position
        a = [channel(name, head * 6 + mp * 3 + e, t) for e in range(3)]
        c, s = math.cos(t), math.sin(t)
        return torch.tensor([a[0] * c - a[1] * s, a[1] * c + a[0] * s, a[2]], dtype=F64)

    lam = math.exp(float(w["p.lq1"] @ w["p.lk1"])) - math.exp(float(w["p.lq2"] @ w["p.lk2"])) + 0.3
    head, i = 3, 5  # key/value head 1; reads keys 0 (kept), 3, 4, 5
    maps = []
    for mp in (0, 1):
        q = turned("q", head, mp, i)
        e = {j: math.exp(0.6 * float(q @ turned("k", 1, mp, j))) for j in (0, 3, 4, 5)}
        maps.append(sum(x / sum(e.values()) * torch.tensor([channel("v", 5 + d, j) for d in range(5)], dtype=F64) for j, x in e.items()))
    o = maps[0] - lam * maps[1]
    o = o / math.sqrt(float((o * o).mean()) + eps) * 0.7
    gate = 1 / (1 + math.exp(-float(w["p.g"][head] @ h[i])))
    assert torch.allclose(got[i, head * 5 : head * 5 + 5], o * gate)
    assert torch.allclose(k[4, 1, 1], turned("k", 1, 1, 4)) and k.shape == (n, 2, 2, 3) and v.shape == (n, 2, 5)
    # a reader of these keys and values: its own queries and mask, the other's keys and values
    other = {**m, "mask": {"size": 1, "keep_first": 0}, "diff": 0.0}
    again, _ = P.differential_attention(h, torch.arange(n), w, "p", other, eps, kv=(k, v))
    o = v[i, 1] * (1 - (lam - 0.3))  # one key: both maps return its value
    assert torch.allclose(again[i, head * 5 : head * 5 + 5], o / torch.sqrt((o * o).mean() + eps) * gate)


def test_lightning_against_the_unrolled_sum():
    m = {"heads": 2, "dim": 3, "vdim": 4, "decay": [0.5, 0.9]}
    n, eps = 6, 1e-5
    w = {f"p.{r}": torch.randn(s, 5, dtype=F64) for r, s in (("q", 6), ("k", 6), ("v", 8), ("g", 8))}
    w["p.norm"], w["p.o"] = torch.rand(8, dtype=F64) + 0.5, torch.eye(8, dtype=F64)
    h = torch.randn(n, 5, dtype=F64)
    act = torch.nn.functional.silu
    q, k, v = (act(h @ w[f"p.{r}"].T).view(n, 2, -1) for r in ("q", "k", "v"))
    o = torch.zeros(n, 2, 4, dtype=F64)
    for a, d in enumerate(m["decay"]):
        for t in range(n):
            o[t, a] = sum(d ** (t - s) * float(q[t, a] @ k[s, a]) * v[s, a] for s in range(t + 1))
    flat = o.reshape(n, 8)
    want = flat / torch.sqrt((flat * flat).mean(-1, keepdim=True) + eps) * w["p.norm"] * torch.sigmoid(h @ w["p.g"].T)
    assert torch.allclose(P.lightning(h, w, "p", m, eps), want)


def test_feed_forward_by_hand():
    w = {"p.up": torch.tensor([[1.0, 0.0], [0.0, -1.0]], dtype=F64), "p.down": torch.tensor([[1.0, 10.0]], dtype=F64)}
    assert P.feed_forward(torch.tensor([[3.0, 2.0], [-1.0, -4.0]], dtype=F64), w, "p", {"kind": "dense"}).flatten().tolist() == [9.0, 160.0]


def _random_model(cfg, seed=3):
    from shrike_amd.models import DecoderModel
    from shrike_amd.models.fozedra import FozedraConfig, build_spec
    from shrike_amd.weights.random_init import random_tensors

    model = DecoderModel(build_spec(FozedraConfig.from_dict(cfg)))
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
    assert streams.shape[0] == len(cfg["layers"])
    for a, b in zip(streams[:-1], streams[1:]):
        assert float((b - a).abs().mean()) > 1e-2 * float(a.abs().mean())


def test_configuration_round_trip_names_and_schedule():
    from shrike_amd.config import get_architecture
    from shrike_amd.models.fozedra import FozedraConfig

    for cfg in CONFIGS.values():
        parsed = FozedraConfig.from_dict(cfg)
        assert FozedraConfig.from_dict(parsed.to_dict()) == parsed
    assert get_architecture("Fozedra").config_cls is FozedraConfig
    model, w = _random_model(FOZ_A)
    names = {p.name: tuple(p.shape) for p in model.params()}
    assert names["l0.norm1.alpha"] == () and names["l0.norm1.b"] == (70,) and names["final.norm.alpha"] == ()
    assert names["l0.mix.q"] == (4 * 2 * 16, 70) and names["l0.mix.k"] == (2 * 2 * 16, 70) and names["l0.mix.v"] == (2 * 40, 70)
    assert names["l0.mix.q.b"] == (128,) and names["l0.mix.v.conv"] == (80, 3) and names["l0.mix.lq2"] == (16,)
    assert names["l0.mix.g"] == (4, 70) and names["l0.mix.o"] == (70, 160) and names["l0.mlp.up"] == (80, 70)
    assert names["l1.mix.norm"] == (36,) and "l1.norm2" not in names and "l1.mlp.up" not in names
    assert names["l2.mix.q.conv"] == (128, 5) and not any(n.startswith(("l2.mix.k", "l2.mix.v")) for n in names)
    assert "l3.mix.q.conv" not in names and names["l3.mix.q.b"] == (42,) and "head.weight" not in names
    assert [e.cache_of for e in model.spec.schedule] == [None, None, 0, None, 3]
    assert model.launches_follow_shape() and model.graph_safe()


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0]["mixer"].pop("diff"), "diff"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "more than dim"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "positive"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("fast"), "fast"),
    (lambda c: c["layers"][1]["mixer"].update(decay=[0.5]), "decays"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "earlier"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "of its own"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=8), "other sizes"),
    (lambda c: c["layers"][0].update(type="memory"), "unknown mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "unknown feed-forward"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_configuration_errors_say_what_is_wrong(change, text):
    from shrike_amd.config import ConfigError
    from shrike_amd.models.fozedra import FozedraConfig

    cfg = copy.deepcopy(FOZ_A)
    change(cfg)
    with pytest.raises(ConfigError, match=text):
        FozedraConfig.from_dict(cfg)


def test_what_the_caches_keep():
    from shrike_amd.models.fozedra import FozedraConfig, cache_reach
    from shrike_amd.parts import CompositeSpec, StateSpec

    a, b, c = (FozedraConfig.from_dict(x) for x in (FOZ_A, FOZ_B, FOZ_C))
    assert cache_reach(a) == {0: (37, 7), 3: (None, 0)}
    assert cache_reach(b) == {1: (16, 16), 2: (None, 3)}
    assert cache_reach(c) == {0: (37, 20), 2: (1000, 5), 4: (70, 33), 5: (None, 0)}
    model, _ = _random_model(FOZ_A)
    specs = model.cache_specs()
    pages = dict(specs[0].parts)["kv"]
    assert (pages.window, pages.keep_first) == (37, 7) and dict(specs[0].parts)["conv"] == StateSpec((2 * (128 + 64 + 80),))
    assert specs[1] == StateSpec((3 * 20 * 12,))
    assert specs[2] == CompositeSpec((("conv", StateSpec((4 * 128,))),)), "a reader keeps its own queries' inputs only"
    assert [name for name, _ in specs[3].parts] == ["kv"] and specs[4] is None
    # convolutions of one tap keep nothing
    model, _ = _random_model(FOZ_B)
    assert [name for name, _ in model.cache_specs()[1].parts] == ["kv"]


def test_a_reading_run_gets_the_pages_it_reads_and_the_state_it_owns():
    from shrike_amd.cache import CacheManager

    model, _ = _random_model(FOZ_A)
    cm = CacheManager(model.cache_specs(), 4, 20, max_slots=3)
    own, read = cm.layer_cache(0), cm.reading_cache(2, 0)
    assert own.parts["kv"].owned and not read.parts["kv"].owned and read.parts["kv"].group == own.parts["kv"].group
    assert set(read.parts) == {"kv", "conv"} and read.parts["conv"].owned
    assert read.parts["conv"].group != own.parts["conv"].group, "the reader's inputs are its own"
    assert set(cm.reading_cache(4, 3).parts) == {"kv"}


def test_pages_of_the_first_tokens_stay_when_the_window_passes():
    """A window of 6 that keeps 5 tokens, pages of 4: pages 0 and 1 stay, the others go back as the window
    passes them; everything comes back at the end, and pages are used again."""
    from shrike_amd.cache import CacheManager
    from shrike_amd.parts import PAGE, PagedSpec, PageTensor

    spec = PagedSpec((PageTensor("k", (2, PAGE)),), window=6, keep_first=5)
    cm = CacheManager([spec], 4, 7, max_slots=2, enable_prefix_caching=True)
    assert not cm.enable_prefix_caching
    seq = cm.new_sequence()
    for p in range(60):
        cm.append(seq, p, 1)
        cm.trim(seq, p + 1)
        held = [i for i, page in enumerate(seq.tables[0]) if page >= 0]
        oldest = max(0, p + 1 - 6 + 1) // 4
        assert held == sorted(set(range(min(2, p // 4 + 1))) | set(range(min(oldest, p // 4 + 1), p // 4 + 1))), p
        cm.check([seq])
    assert cm.num_free >= 2
    cm.free(seq)
    cm.check([])
    assert cm.num_free == 7
    # more kept tokens than the window has passed: nothing goes back yet
    few = CacheManager([PagedSpec((PageTensor("k", (2, PAGE)),), window=2, keep_first=100)], 4, 30)
    seq = few.new_sequence()
    few.append(seq, 0, 90)
    assert few.trim(seq, 90) == 0 and all(page >= 0 for page in seq.tables[0])
