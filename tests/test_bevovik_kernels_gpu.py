"""The kernels and options that the Bevovik decoder brought, each alone against a plain computation
(tests/plain/bevovik.py): the stream's sum with a normed output; rotation with a factor; batched products
with float32 results; the convolution without activation and the decays' logarithms; gated linear attention
token by token and in chunks, in pieces and in used slots, with gentle and steep decays, a far token that
stays and one that fades; the gated recurrence in single tokens and portions; the router's groups; experts
with bounds, a shift and identity experts in every kernel of their products."""

import math

import pytest
import torch

from .plain import bevovik as plain

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.6e-2}


@pytest.fixture(scope="module")
def ops():
    from shrike_amd.kernels import ops

    return ops


def dev(t, dtype=None):
    return t.to("cuda", dtype).contiguous() if dtype else t.to("cuda").contiguous()


def i32(x):
    return torch.as_tensor(x, dtype=torch.int32).to("cuda")


def close(got, want, dtype, what="", tol=None):
    want = want.double().cpu()
    err = float((got.double().cpu() - want).abs().max() / want.abs().max().clamp_min(1e-30))
    tol = TOL[dtype] if tol is None else tol
    assert err <= tol, f"{what} rel err {err:.3e} > {tol}"


def step_arrays(starts, lens):
    positions, token_seq, cu = [], [], [0]
    for s, (st, n) in enumerate(zip(starts, lens)):
        positions += list(range(st, st + n))
        token_seq += [s] * n
        cu.append(cu[-1] + n)
    return i32(positions), i32(token_seq), i32(cu)


# ------------------------------------------------------------------ the stream

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n, width, splits", [(3, 70, 0), (5, 128, 0), (2, 130, 3), (9, 3584, 4), (1, 5120, 0)])
def test_a_normed_output_joins_the_stream_which_is_left_in_the_compute_dtype(ops, dtype, n, width, splits):
    torch.manual_seed(width)
    eps = 1e-3
    resid, weight = torch.randn(n, width), torch.randn(width)
    if splits:
        parts = torch.randn(splits, n, width)
        delta, total = ops.SplitSum(dev(parts)), parts.double().sum(0)
    else:
        x = torch.randn(n, width).to(dtype)
        delta, total = dev(x), x.double()
    got, out = dev(resid), torch.full((n, width), float("nan"), dtype=dtype, device="cuda")
    ops.add_normed_rmsnorm(got, delta, dev(weight), eps, out=out)
    want = resid.double() + plain.unit_rms(total, eps) * weight.double()
    close(got, want, torch.float32)
    assert torch.equal(out, got.to(dtype))


# ------------------------------------------------------------------ latent attention's rotation

@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_with_stretched_rates_and_a_factor(ops, dtype):
    torch.manual_seed(5)
    n, heads, rot_dim, q_rank, kv_rank, page = 7, 3, 12, 20, 24, 4
    rot = {"base": 777.0, "dims": rot_dim, "scaling": {"factor": 5.0, "original": 90, "fast": 6.0, "slow": 1.5}}
    rates, factor = plain.turn_rates(rot)
    assert factor > 1.1
    pos = [0, 1, 2, 300, 301, 4000, 4001]
    src = torch.randn(n, heads * (rot_dim + 5)).to(dtype)
    dst = torch.zeros(n, heads * (rot_dim + 9), dtype=dtype, device="cuda")
    ops.rotate_heads(dev(src), rot_dim + 5, 5, dst, rot_dim + 9, 9, heads, rot_dim, dev(rates.float()), i32(pos), magnitude=factor)
    want = plain.rotate_pairs(src.double().view(n, heads, -1)[..., 5:], torch.tensor(pos), rot)
    # (float32 angles of some thousand radians are off by their rounding)
    close(dst.view(n, heads, -1)[..., 9:], want, dtype, tol=1e-3 if dtype == torch.float32 else None)
    close(dst.view(n, heads, -1)[:5, :, 9:], want[:5], dtype)
    down = torch.randn(n, q_rank + kv_rank + rot_dim).to(dtype)
    tables = torch.arange(1001, dtype=torch.int32).view(1, -1)
    pool = torch.zeros(1001, page, kv_rank + rot_dim, dtype=dtype, device="cuda")
    c_q = torch.empty(n, q_rank, dtype=dtype, device="cuda")
    ops.latent_prepare(dev(down), q_rank, kv_rank, rot_dim, dev(torch.ones(q_rank)), dev(torch.ones(kv_rank)), 1e-5, dev(rates.float()),
                       i32(pos), i32([0] * n), dev(tables), c_q, pool, page, magnitude=factor)
    rows = torch.stack([pool[p // page, p % page] for p in pos])
    want = plain.rotate_pairs(down.double()[:, q_rank + kv_rank :], torch.tensor(pos), rot)
    close(rows[:5, kv_rank:], want[:5], dtype)
    close(rows[:, :kv_rank], plain.unit_rms(down.double()[:, q_rank : q_rank + kv_rank], 1e-5), dtype, "the latent has no factor")


# ------------------------------------------------------------------ products

@pytest.mark.parametrize("n, batch, m, k", [(1, 3, 64, 32), (70, 2, 40, 24), (33, 4, 30, 15), (5, 2, 14, 7), (2, 14, 512, 256), (300, 3, 130, 72)])
def test_batched_product_of_bfloat16_rows_keeps_float32_results(ops, n, batch, m, k):
    torch.manual_seed(k)
    a = torch.randn(n, batch * k).to(torch.bfloat16)
    w = (torch.randn(batch, m, k) / k**0.5).to(torch.bfloat16)
    out = torch.full((n, batch * m), float("nan"), device="cuda")
    ops.gemm_batched(dev(a), dev(w), out, batch, k, m)
    want = torch.einsum("nbk,bmk->nbm", a.double().view(n, batch, k), w.double()).reshape(n, -1)
    close(out, want, torch.float32)


@pytest.mark.parametrize("n, rank, inner", [(1, 16, 128), (40, 1, 70), (9, 24, 300), (100, 5, 60)])
def test_logarithms_of_decays(ops, n, rank, inner):
    """log sigmoid(z) / tau, from z far below zero (the logarithm is z itself) to far above (tiny numbers)."""
    torch.manual_seed(rank)
    low, w, b = torch.randn(n, rank + 3) * 4, torch.randn(inner, rank) * 3, torch.randn(inner)
    b[0], b[1] = -60.0, 12.0
    got = torch.empty(n, inner, device="cuda")
    ops.dt_softplus(dev(low)[:, :rank], dev(w.t()), dev(b), got, sign=-1.0, mult=-1.0 / 7.0)
    z = low[:, :rank].double() @ w.double().T + b.double()
    want = plain.log_sigmoid(z) / 7.0
    close(got, want, torch.float32)
    assert float(got.max()) <= 0.0
    small = want[want.abs() < 1e-3]
    if small.numel():
        assert float(((got.cpu().double()[want.abs() < 1e-3] - small) / small.abs().clamp_min(1e-12)).abs().max()) < 1e-2


# ------------------------------------------------------------------ gated linear attention

def chunk_lists(counts, first_seq):
    seqs, t0, base = [], [], []
    for i, c in enumerate(counts):
        base.append(len(seqs))
        for at in range(0, c, 64):
            seqs.append(first_seq + i)
            t0.append(at)
    return i32(seqs + t0 + base)


def run_gla(ops, kernel, x, log_decay, plan, lens, heads, dim, v_dim, q_scale, state):
    """plan: steps of [(sequence, slot, start, count)], single tokens first; x[s] the projections of a
    sequence (queries, keys, values side by side)."""
    qk, vv = heads * dim, heads * v_dim
    got = {s: torch.zeros(n, vv, device="cuda") for s, n in lens.items()}
    for step in plan:
        starts, counts = [e[2] for e in step], [e[3] for e in step]
        singles = sum(c == 1 for c in counts)
        assert all(c == 1 for c in counts[:singles])
        positions, _, cu = step_arrays(starts, counts)
        rows = dev(torch.cat([x[s][st : st + c] for s, _, st, c in step]))
        g = dev(torch.cat([log_decay[s][st : st + c] for s, _, st, c in step]))
        slots, out = i32([slot for _, slot, _, _ in step]), torch.full((rows.shape[0], vv), float("nan"), device="cuda")
        in_order = len(step)
        if kernel == "chunk" and len(step) > singles:
            in_order = singles
            lists = chunk_lists(counts[singles:], singles)
            chunks = (lists.numel() - len(step) + singles) // 2
            scratch = torch.full((ops.gla_chunk_scratch_bytes(rows.shape[0] - singles, chunks, heads, dim, v_dim),), 255, dtype=torch.uint8,
                                 device="cuda")  # (not numbers, where nothing is written)
            ops.gla_chunk(rows, 0, qk, 2 * qk, g, q_scale, singles, len(step) - singles, singles, heads, dim, v_dim, lists, positions, cu,
                          slots, state, scratch, out)
        if in_order:
            ops.retention_scan(rows, 0, qk, 2 * qk, None, in_order, heads, dim, v_dim, positions, cu, slots, state, out, log_decay=g,
                               q_scale=q_scale)
        at = 0
        for s, _, st, c in step:
            got[s][st : st + c] = out[at : at + c]
            at += c
    return got


GLA_PLAN = [[("a", 0, 0, 2), ("b", 1, 0, 64)], [("a", 0, 2, 1)], [("c", 1, 0, 1), ("a", 0, 3, 100)], [("c", 1, 1, 1), ("a", 0, 103, 1)],
            [("c", 1, 2, 65), ("a", 0, 104, 64)], [("c", 1, 67, 64), ("a", 0, 168, 37)]]
GLA_LENS = {"a": 205, "b": 64, "c": 131}
GLA_CASES = [(2, 64, 32), (1, 32, 64), (3, 128, 32), (2, 96, 96), (1, 192, 32), (1, 256, 64)]


@pytest.mark.parametrize("spread, shift", [(1.0, 0.05), (3.0, 2.0), (0.01, 1e-4)])
@pytest.mark.parametrize("kernel, heads, dim, v_dim", [(k, *c) for c in GLA_CASES for k in ("scan_f32", "scan_bf16", "chunk")]
                         + [(k, *c) for c in ((2, 20, 12), (3, 7, 5)) for k in ("scan_f32", "scan_bf16")])
def test_gated_linear_attention_in_pieces_and_in_used_slots(ops, kernel, heads, dim, v_dim, spread, shift):
    """Three sequences in portions and single tokens over slots that earlier holders left full.  Decays from
    nearly 1 (a memory longer than the sequences) to e^-12 a token in places: products of their inverses
    over a chunk would leave float32."""
    assert kernel != "chunk" or ops.gla_chunk_supports(dim, v_dim)
    torch.manual_seed(dim + v_dim)
    qk, vv = heads * dim, heads * v_dim
    dtype = torch.float32 if kernel == "scan_f32" else torch.bfloat16
    x = {s: torch.randn(n, -(-(2 * qk + vv) // 8) * 8 + 8).to(dtype) for s, n in GLA_LENS.items()}
    g = {s: -(torch.randn(n, qk) * spread).abs() - shift * torch.rand(qk) for s, n in GLA_LENS.items()}
    q_scale = dim**-0.5
    state = torch.full((3, ops.retention_state_floats(heads, dim, v_dim)), -3.0, device="cuda")
    got = run_gla(ops, kernel, x, g, GLA_PLAN, GLA_LENS, heads, dim, v_dim, q_scale, state)
    for s, rows in x.items():
        p = rows.double()
        split = lambda o, w, n=rows.shape[0]: p[:, o : o + w].reshape(n, heads, -1)  # noqa: E731
        want = plain.decayed_outer_sums(split(0, qk) * q_scale, split(qk, qk), split(2 * qk, vv),
                                        torch.exp(g[s].double()).view(-1, heads, dim)).reshape(-1, vv)
        close(got[s], want, torch.float32, f"sequence {s}", tol=5e-5)


def test_chunks_of_gated_linear_attention_keep_a_far_token_and_forget_others(ops):
    """Without decay the first token's value comes back whole 600 tokens later in one key channel; beside
    it, in the same head, a channel that fades by e^-20 a token sees itself alone; and one token that
    forgets everything empties the first channel."""
    heads, dim, v_dim, n = 2, 32, 32, 700
    qk = heads * dim
    rows = torch.zeros(n, 2 * qk + heads * v_dim, dtype=torch.bfloat16)
    g = torch.zeros(n, qk)
    g[:, 1::dim] = -20.0
    g[650, 0::dim] = -200.0
    rows[:, 0:qk:dim], rows[:, 1:qk:dim] = 1.0, 1.0  # every query reads channels 0 and 1
    rows[0, qk : 2 * qk : dim], rows[0, 2 * qk :] = 1.0, 2.0
    rows[600, qk + 1 : 2 * qk : dim], rows[600, 2 * qk :] = 0.5, 3.0
    lens, cuts = {"a": n}, [130, 2, 300, 64, 95] + [1] * 9 + [40, 60]
    assert sum(cuts) == n
    plan, at = [], 0
    for c in cuts:
        plan.append([("a", 0, at, c)])
        at += c
    state = torch.full((1, ops.retention_state_floats(heads, dim, v_dim)), 9.0, device="cuda")
    o = run_gla(ops, "chunk", {"a": rows}, {"a": g}, plan, lens, heads, dim, v_dim, 1.0, state)["a"].cpu()
    assert torch.allclose(o[599], torch.full((heads * v_dim,), 2.0)) and torch.isfinite(o).all()
    assert torch.allclose(o[600], torch.full((heads * v_dim,), 3.5)) and torch.allclose(o[602], torch.full((heads * v_dim,), 2.0))
    assert torch.allclose(o[649], torch.full((heads * v_dim,), 2.0)) and float(o[650:].abs().max()) < 1e-30


# ------------------------------------------------------------------ the gated recurrence

def run_rglru(ops, seqs, w, blocks, taps, dtype, state, plan, lone=True):
    """plan: steps of [(sequence, slot, start, count)], single tokens first; seqs[s]: rows [y | x] after
    their biases.  lone False: single tokens run as portions."""
    width = w["lam"].numel()
    part = width // blocks
    got = {s: torch.full((x.shape[0], width), float("nan"), dtype=dtype, device="cuda") for s, x in seqs.items()}
    gates_w = dev(torch.cat([w["ra"], w["ri"]], dim=1), dtype)
    rate = dev((8.0 * plain.softplus(w["lam"].double())).float())
    for step in plan:
        starts, counts = [e[2] for e in step], [e[3] for e in step]
        singles = sum(c == 1 for c in counts) if lone else 0
        positions, token_seq, cu = step_arrays(starts, counts)
        slots = i32([slot for _, slot, _, _ in step])
        rows = dev(torch.cat([seqs[s][st : st + c] for s, _, st, c in step]), dtype)
        n, raw = rows.shape[0], rows[:, width:]
        u = torch.full((n, width), float("nan"), dtype=dtype, device="cuda")
        ops.short_conv(raw, dev(w["conv"]), dev(w["conv.b"]), positions, token_seq, cu, slots, state, 1, u)
        gates = torch.empty(n, 2 * width, device="cuda")
        ops.gemm_batched(u, gates_w, gates, blocks, part, 2 * part)
        out = torch.full((n, width), float("nan"), dtype=dtype, device="cuda")
        ops.rglru(gates, blocks, dev(w["ra.b"].reshape(-1)), dev(w["ri.b"].reshape(-1)), rate, u, rows, raw, taps, positions, cu, slots, state,
                  out, singles, len(step))
        at = 0
        for s, _, st, c in step:
            got[s][st : st + c] = out[at : at + c]
            at += c
    return got


def recurrence_weights(width, blocks, taps, dtype, slow=True):
    part = width // blocks
    round_ = lambda t: t.to(dtype).float()  # noqa: E731
    return {"ra": round_(torch.randn(blocks, part, part) * part**-0.5), "ri": round_(torch.randn(blocks, part, part) * part**-0.5),
            "ra.b": torch.randn(blocks, part) * 0.5, "ri.b": torch.randn(blocks, part) * 0.5,
            "lam": torch.randn(width) * 1.5 - (5.0 if slow else 0.0), "conv": torch.randn(width, taps), "conv.b": torch.randn(width) * 0.3}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width, blocks, taps, slow", [(40, 2, 4, True), (96, 3, 2, False), (70, 7, 1, True), (33, 1, 5, True),
                                                       (264, 11, 3, False), (512, 2, 4, True)])
def test_gated_recurrence_in_pieces_and_in_used_slots(ops, dtype, width, blocks, taps, slow):
    torch.manual_seed(width)
    w = recurrence_weights(width, blocks, taps, dtype, slow)
    lens = {"a": 300, "b": 9, "c": 1, "d": 600, "e": 2}
    seqs = {s: torch.randn(n, 2 * width).to(dtype).float() for s, n in lens.items()}
    floats = ops.rglru_state_floats(width, taps)
    assert floats == width * taps
    plan = [[("c", 2, 0, 1), ("a", 0, 0, 2), ("b", 1, 0, 5)], [("a", 0, 2, 1), ("b", 1, 5, 1), ("d", 2, 0, 258)],
            [("b", 1, 6, 3), ("a", 0, 3, 40)], [("e", 1, 0, 2), ("a", 0, 43, 256), ("d", 2, 258, 7)], [("a", 0, 299, 1), ("d", 2, 265, 335)]]

    def run(plan, lone=True):
        state = torch.full((3, floats), 7.0, device="cuda")  # what earlier holders left behind
        return run_rglru(ops, seqs, w, blocks, taps, dtype, state, plan, lone)

    got = run(plan)
    double = {f"p.{k}": v.double() for k, v in w.items()}
    for s, rows in seqs.items():
        x = rows.double()
        u = plain.causal_convolution(x[:, width:], double["p.conv"], double["p.conv.b"])
        if dtype == torch.bfloat16:
            u = u.to(dtype).double()  # the convolution's output has the compute dtype
        r, i = plain.block_gate(u, double, "p.ra", blocks), plain.block_gate(u, double, "p.ri", blocks)
        S = plain.recurrent_sums(-8.0 * r * plain.softplus(double["p.lam"]), i * u)
        close(got[s], S * plain.gelu_tanh(x[:, :width]), dtype, f"sequence {s}", tol=5e-5 if dtype == torch.float32 else None)
    # every token is one multiply-add on the state before it: the same bits in any cutting, alone or as a portion
    whole = [[(s, 0, 0, n)] for s, n in lens.items()]
    one_by_one = [[("b", 0, p, 1)] for p in range(9)]
    for other in (run(whole), run(plan, lone=False)):
        for s in lens:
            # (bfloat16: the gates' products of few rows may run in another kernel)
            assert torch.equal(other[s], got[s]) or dtype == torch.bfloat16, s
            close(other[s], got[s], dtype)
    assert torch.equal(run(one_by_one)["b"], got["b"]) or dtype == torch.bfloat16


def test_gated_recurrence_keeps_a_far_input_where_its_rate_is_small(ops):
    """Channels with rates of e^-12 and e^3: the first token's input is there 700 tokens later, or gone at
    the next; sqrt(1 - a^2) of a rate that small is not lost in rounding."""
    width, taps = 64, 1
    w = {"ra": torch.zeros(1, width, width), "ri": torch.zeros(1, width, width), "ra.b": torch.full((1, width), 30.0),
         "ri.b": torch.full((1, width), 30.0), "lam": torch.tensor([-12.0, 3.0]).repeat(width // 2), "conv": torch.ones(width, 1),
         "conv.b": torch.zeros(width)}
    x = torch.zeros(701, 2 * width)
    x[:, :width] = 20.0  # gelu(20) = 20
    x[0, width:] = 1000.0
    state = torch.full((1, width), 5.0, device="cuda")
    cuts = [1, 299, 2, 1, 300, 97, 1]
    plan, at = [], 0
    for c in cuts:
        plan.append([("a", 0, at, c)])
        at += c
    o = run_rglru(ops, {"a": x}, w, 1, taps, torch.float32, state, plan)["a"].double().cpu()
    log_a = -8.0 * math.log1p(math.exp(-12.0))
    want = 20.0 * math.sqrt(-math.expm1(2 * log_a)) * 1000.0 * math.exp(700 * log_a)
    assert abs(float(o[700, 0]) / want - 1) < 1e-4 and float(o[2, 1]) < 1e-10 and float(o[0, 1]) > 1.9e4


# ------------------------------------------------------------------ router

@pytest.mark.parametrize("outputs, top, count, keep", [(6, 2, 3, 1), (10, 4, 2, 1), (12, 6, 6, 3), (12, 3, 4, 4), (128, 8, 64, 9),
                                                       (200, 20, 8, 3), (512, 64, 32, 7), (5, 5, 1, 1), (6, 3, 2, 1)])
def test_router_chooses_among_the_best_groups(ops, outputs, top, count, keep):
    torch.manual_seed(outputs + top)
    n = 61
    logits = torch.randn(n, outputs + 3)
    chosen, weights = torch.empty(n, top, dtype=torch.int32, device="cuda"), torch.empty(n, top, device="cuda")
    for shift in (0.0, -4.0):  # choice scores of both signs, and none above zero
        correction = torch.randn(outputs) * 0.2 + shift
        ops.moe_route(dev(logits)[:, :outputs], dev(correction), top, chosen, weights, groups=(count, keep), scale=2.5)
        s = torch.softmax(logits[:, :outputs].double(), -1)
        want = torch.tensor([plain.choose(row, correction.double(), top, count, keep) for row in s])
        assert torch.equal(chosen.cpu().long(), want)
        picked = s.gather(1, want)
        close(weights, picked / picked.sum(-1, keepdim=True) * 2.5, torch.float32)


def test_equal_groups_and_equal_scores_take_the_lowest(ops):
    chosen, weights = torch.empty(1, 2, dtype=torch.int32, device="cuda"), torch.empty(1, 2, device="cuda")
    ops.moe_route(dev(torch.zeros(1, 6)), None, 2, chosen, weights, groups=(3, 1))
    assert chosen.cpu().tolist() == [[0, 1]]
    ops.moe_route(dev(torch.zeros(1, 6)), dev(torch.tensor([0.0, 0.1, 0.1, 0.0, 0.1, 0.1])), 2, chosen, weights, groups=(2, 1))
    assert chosen.cpu().tolist() == [[1, 2]]
    with pytest.raises(Exception, match="groups"):
        ops.moe_route(dev(torch.zeros(1, 6)), None, 2, chosen, weights, groups=(4, 1))
    with pytest.raises(Exception, match="chosen"):
        ops.moe_route(dev(torch.zeros(1, 6)), None, 2, chosen, weights, groups=(6, 1))


# ------------------------------------------------------------------ experts

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n, width, ff, experts, identity, top, limit, shared", [
    (1, 64, 24, 5, 2, 3, 0.7, True), (7, 100, 30, 3, 1, 4, 2.0, False), (40, 128, 64, 6, 3, 1, 0.3, True),
    (130, 72, 24, 4, 4, 3, 1.0, False), (300, 256, 96, 3, 1, 2, 0.5, True), (200, 128, 136, 2, 1, 2, 1.5, True)])
def test_bounded_experts_and_identity_experts(ops, dtype, n, width, ff, experts, identity, top, limit, shared):
    """Few and many pairs an expert (all kernels of the products), rows in and not in multiples of 8, tokens
    of identity experts alone, bounds that bite on both sides."""
    torch.manual_seed(n + width)
    x = torch.randn(n, width).to(dtype)
    wg, wu = ((torch.randn(experts, ff, width) * width**-0.5).to(dtype) for _ in range(2))
    wd = (torch.randn(experts, width, ff) * ff**-0.5).to(dtype)
    chosen = torch.stack([torch.randperm(experts + identity)[:top] for _ in range(n)]).to(torch.int32)
    chosen[n // 2] = torch.arange(experts, experts + top) if identity >= top else chosen[n // 2]
    weights = torch.rand(n, top) + 0.1
    add = torch.randn(n, width).to(dtype) if shared else None
    want = torch.zeros(n, width, dtype=torch.float64) if add is None else add.double().clone()
    bounded = 0
    for t in range(n):
        for j in range(top):
            e = int(chosen[t, j])
            if e >= experts:
                want[t] += weights[t, j].double() * x[t].double()
                continue
            g, u = wg[e].double() @ x[t].double(), wu[e].double() @ x[t].double()
            bounded += int((g > limit).sum()) + int((u.abs() > limit).sum())
            g, u = g.clamp(max=limit), u.clamp(-limit, limit)
            hidden = g * torch.sigmoid(1.702 * g) * (u + 1.0)
            if dtype == torch.bfloat16:
                hidden = hidden.to(dtype).double()  # the activations between the two products have the compute dtype
            want[t] += weights[t, j].double() * (wd[e].double() @ hidden)
    assert bounded > 0 or n == 1
    kw = dict(activation="quick_gelu", add=None if add is None else dev(add), identity=identity, limit=limit, up_shift=1.0)
    scratches = [None]
    if ops.moe_grouped(n, width, ff, dtype):
        scratches.append(torch.full((ops.moe_grouped_scratch_bytes(n, width, experts, top),), 255, dtype=torch.uint8, device="cuda"))
    for scratch in scratches:
        act = torch.full((n * top, ff), float("nan"), dtype=dtype, device="cuda")
        out = torch.full((n, width), float("nan"), dtype=dtype, device="cuda")
        ops.moe_experts(dev(x), dev(chosen), dev(weights), dev(wg), dev(wu), dev(wd), act, out, scratch=scratch, **kw)
        close(out, want, dtype, f"scratch {scratch is not None}", tol=None if dtype == torch.float32 else 2e-2)


def test_what_the_kernels_do_not_take_is_refused(ops):
    assert not ops.gla_chunk_supports(48, 32) and not ops.gla_chunk_supports(64, 20)
    one = i32([0, 1])
    x = torch.zeros(1, 24, device="cuda")
    state = torch.zeros(1, 64, device="cuda")
    out = torch.zeros(1, 8, device="cuda")
    with pytest.raises(Exception, match="decay"):
        ops.retention_scan(x, 0, 8, 16, None, 1, 1, 8, 8, one, one, one, state, out)
    with pytest.raises(Exception, match="blocks"):
        ops.rglru(torch.zeros(1, 16, device="cuda"), 3, *[torch.zeros(8, device="cuda")] * 3, out, out, out, 2, one, one, one, state,
                  torch.zeros_like(out), 0, 1)
    with pytest.raises(Exception, match="hold the state"):
        ops.rglru(torch.zeros(1, 16, device="cuda"), 2, *[torch.zeros(8, device="cuda")] * 3, out, out, out, 20, one, one, one, state,
                  torch.zeros_like(out), 0, 1)
