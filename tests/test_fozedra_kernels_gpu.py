"""The kernels and options that the Fozedra decoder brought, each alone against a plain computation
(tests/plain/fozedra.py): the bounded map around the stream; the products' plain activations; convolution,
rotation and cache write in portions down to single tokens, in slots that are used again; differential
attention in the general kernel and on the matrix units, with keys made to stand out among the kept first
tokens, just behind them, just inside and just outside a window and far back; lightning attention token
by token and in chunks; the norm over many heads."""

import math

import pytest
import torch

from .plain import fozedra as plain

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
    positions = torch.cat([torch.arange(s, s + l) for s, l in zip(starts, lens)])
    token_seq = torch.cat([torch.full((l,), i) for i, l in enumerate(lens)])
    cu = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)))
    return i32(positions), i32(token_seq), i32(cu)


def tables_for(ctx_lens, page_size, num_pages, seed=0):
    g = torch.Generator().manual_seed(seed)
    perm = torch.randperm(num_pages, generator=g).tolist()
    width = max(-(-n // page_size) for n in ctx_lens)
    rows = []
    for n in ctx_lens:
        need = -(-n // page_size)
        rows.append([perm.pop() for _ in range(need)] + [0] * (width - need))
    return torch.tensor(rows, dtype=torch.int32)


def runs(lens, singles, run):
    """Sequences, then first queries, of the runs of `run` tokens that prompt portions are cut into."""
    seqs, q0 = [], []
    for s, l in enumerate(lens):
        if s >= singles:
            for q in range(0, l, run):
                seqs.append(s), q0.append(q)
    return i32(seqs + q0) if seqs else None


# ------------------------------------------------------------------ the bounded map around the stream

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n, hidden, splits", [(5, 64, 0), (3, 70, 0), (40, 1024, 3), (2, 4097, 6), (300, 132, 1), (1, 5, 2)])
def test_dynamic_tanh_around_the_stream(ops, dtype, n, hidden, splits):
    torch.manual_seed(4)
    resid = torch.randn(n, hidden) * 3
    weight, bias, alpha, scale = torch.rand(hidden) + 0.5, torch.randn(hidden), 0.7, 0.3
    if splits:
        parts = torch.randn(splits, n, hidden)
        delta, total = ops.SplitSum(dev(parts)), parts.double().sum(0)
    else:
        d = (torch.randn(n, hidden) * 2).to(dtype)
        delta, total = dev(d), d.double()
    x = resid.double() + scale * total
    w = {"n": weight.double(), "n.b": bias.double(), "n.alpha": torch.tensor(alpha, dtype=torch.float64)}
    want = plain.dynamic_tanh(x, w, "n")
    got, out = dev(resid.clone()), torch.empty(n, hidden, dtype=dtype, device="cuda")
    ops.add_dynamic_tanh(got, delta, scale, alpha, dev(weight), dev(bias), out)
    close(got, x, torch.float32, "stream", tol=1e-6)
    close(out, want, dtype, "mapped")
    # chosen rows, the stream left alone
    rows = i32([n - 1, 0, n // 2])
    kept, few = dev(resid.clone()), torch.empty(3, hidden, dtype=dtype, device="cuda")
    ops.add_dynamic_tanh(kept, delta, scale, alpha, dev(weight), dev(bias), few, rows=rows, write_resid=False)
    assert torch.equal(kept.cpu(), resid) and torch.equal(few, out[rows.long()])
    # the addition alone, and the map alone
    only = dev(resid.clone())
    ops.add_dynamic_tanh(only, delta, scale, dtype=dtype)
    assert torch.equal(only, got)
    ops.add_dynamic_tanh(only, None, 1.0, alpha, dev(weight), dev(bias), out)
    close(out, want, dtype)
    # far from zero the map is weight + bias
    big = torch.full((1, hidden), 1e4, device="cuda")
    one = torch.empty(1, hidden, dtype=dtype, device="cuda")
    ops.add_dynamic_tanh(big, None, 1.0, alpha, dev(weight), dev(bias), one)
    close(one[0], weight + bias, dtype)


@pytest.mark.parametrize("norm", ["rmsnorm", "layernorm"])
def test_other_norms_take_a_scaled_addend_too(ops, norm):
    from shrike_amd.config.specs import LayerNormSpec, RMSNormSpec
    from shrike_amd.parts.base import HiddenState, build_part

    class Ctx:
        dtype = torch.float32

        def buffer(self, name, shape, dtype):
            return torch.empty(shape, dtype=dtype, device="cuda")

    torch.manual_seed(1)
    x, d, w, b = torch.randn(4, 48), torch.randn(4, 48), torch.rand(48), torch.randn(48)
    part = build_part("norm", RMSNormSpec(1e-5) if norm == "rmsnorm" else LayerNormSpec(1e-5), 48, "n")
    part.load({"n.weight": dev(w), "n.bias": dev(b)}, None)
    hidden = HiddenState(dev(x), dev(d))
    hidden.pending_scale = 0.25
    out = part.forward(Ctx(), hidden)
    s = (x + 0.25 * d).double()
    want = plain.unit_rms(s, 1e-5) * w if norm == "rmsnorm" else torch.nn.functional.layer_norm(s, (48,), w.double(), b.double(), 1e-5)
    close(out, want, torch.float32)
    close(hidden.resid, s, torch.float32)
    assert hidden.pending is None and hidden.pending_scale == 1.0


@pytest.mark.parametrize("n", [1, 8, 40, 64, 300, 700])
@pytest.mark.parametrize("m, k", [(200, 96), (131, 40)])
def test_plain_products_with_an_activation(ops, n, m, k):
    """The bfloat16 product's epilogue in each of its kernels: the square of ReLU of everything, SiLU of the
    first columns alone (an edge inside a block of 16 and inside the last one), with a bias before it."""
    torch.manual_seed(n + m)
    x, w = torch.randn(n, k).to(torch.bfloat16), (torch.randn(m, k) * k**-0.5).to(torch.bfloat16)
    bias, wt = torch.randn(m), ops.retile_weight(dev(w))
    v = x.double() @ w.double().T
    out = torch.empty(n, m, dtype=torch.bfloat16, device="cuda")
    ops.gemm_tiled_weight(dev(x), wt, m, k, out, activation="relu_squared")
    close(out, torch.relu(v) ** 2, torch.bfloat16)
    ops.gemm_tiled_weight(dev(x), wt, m, k, out, bias=dev(bias), activation="relu_squared")
    close(out, torch.relu(v + bias.double()) ** 2, torch.bfloat16)
    for rows in (1, 37, m - 1, m):
        for dtype in DTYPES:
            res = torch.empty(n, m, dtype=dtype, device="cuda")
            ops.gemm_tiled_weight(dev(x), wt, m, k, res, activation=("silu", rows))
            want = torch.cat([v[:, :rows] * torch.sigmoid(v[:, :rows]), v[:, rows:]], 1)
            close(res[:, :rows], want[:, :rows], torch.bfloat16, f"SiLU of {rows}")
            if rows < m:
                close(res[:, rows:], want[:, rows:], torch.bfloat16, f"behind {rows}")
    with pytest.raises(Exception, match="activation"):
        ops.gemm_tiled_weight(dev(x), wt, m, k, out, activation="tanh")


def test_a_product_in_two_launches_applies_its_activation_to_the_right_columns(ops):
    n, m, k = 1024, 16640, 1024
    assert ops.gemm_parts(n, m, k) == 2, "this shape was meant to run as two launches"
    torch.manual_seed(2)
    x, w = torch.randn(n, k).to(torch.bfloat16), (torch.randn(m, k) * k**-0.5).to(torch.bfloat16)
    v = dev(x).double() @ dev(w).double().T
    wt = ops.retile_weight(dev(w))
    for rows in (100, 16384 + 30, m - 3):  # an edge in the first launch's columns, and in the second's
        out = torch.empty(n, m, dtype=torch.bfloat16, device="cuda")
        ops.gemm_tiled_weight(dev(x), wt, m, k, out, activation=("silu", rows))
        want = torch.cat([v[:, :rows] * torch.sigmoid(v[:, :rows]), v[:, rows:]], 1)
        assert float((out.double() - want).abs().max()) <= 1e-2 * float(want.abs().max())


# ------------------------------------------------------------------ convolution, rotation, cache write

CONV_CASES = [
    # heads, kv_heads, maps, dim, vdim, taps, rot, page_size, gates, splits
    (4, 2, 2, 16, 40, 3, 8, 16, True, 0),
    (3, 3, 2, 7, 9, 0, 0, 4, True, 0),
    (6, 1, 2, 24, 20, 1, 24, 8, True, 0),
    (2, 2, 2, 40, 64, 12, 2, 4, False, 0),
    (8, 2, 2, 32, 64, 4, 32, 32, True, 3),
    (5, 1, 1, 48, 32, 2, 16, 16, True, 0),
    (2, 0, 2, 20, 1, 5, 20, 16, True, 2),
    (4, 0, 2, 8, 1, 4, 0, 16, True, 0),
    (2, 1, 2, 12, 8, 33, 12, 16, True, 0),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, kv_heads, maps, dim, vdim, taps, rot, page_size, gated, splits", CONV_CASES)
def test_convolution_rotation_and_cache_write(ops, dtype, heads, kv_heads, maps, dim, vdim, taps, rot, page_size, gated, splits):
    """Three sequences cut into portions and single tokens, mixed in one step, in slots and pages that hold
    what others left: queries, cached keys and values and gates are the whole sequence's, the same bits
    however it was cut; the slots hold the last inputs."""
    torch.manual_seed(dim + taps)
    qw, kw, vw = heads * maps * dim, kv_heads * maps * dim, kv_heads * vdim
    channels, gates = qw + kw + vw, heads if gated else 0
    width = -(-(channels + gates) // 16) * 16
    lens = {"a": 53, "b": 9, "c": 40}
    proj = {s: torch.randn(n, width).to(dtype if not splits else torch.float32) for s, n in lens.items()}
    w_taps = torch.randn(channels, taps) if taps else None
    inv = None
    spec = {"base": 50.0, "dims": rot, "scaling": {"factor": 3.0, "original": 40, "fast": 4.0, "slow": 1.0}} if rot else None
    magnitude = 1.0
    if rot:
        rates, magnitude = plain.rotation_rates(spec)
        inv = dev(rates.float())
    order = list(lens)
    tables = tables_for([lens[s] for s in order], page_size, 60, seed=dim)
    slab = 32 if (maps * dim) % 32 == 0 else maps * dim

    def run(plan):
        state = torch.full((5, max(1, ops.conv_store_state_floats(channels, taps) + 3) // 4 * 4 + 4), 7.0, device="cuda")
        k_pool = torch.full((61, kv_heads, maps * dim // slab, page_size, slab), 50.0, dtype=dtype, device="cuda") if kv_heads else None
        v_pool = torch.full((61, kv_heads, vdim, page_size), 50.0, dtype=dtype, device="cuda") if kv_heads else None
        got_q = {s: torch.zeros(n, qw, dtype=dtype, device="cuda") for s, n in lens.items()}
        got_g = {s: torch.zeros(n, max(1, gates), device="cuda") for s, n in lens.items()}
        for step in plan:
            step = sorted(step, key=lambda e: e[3] > 1)  # single tokens first
            starts, counts = [e[2] for e in step], [e[3] for e in step]
            singles = sum(c == 1 for c in counts)
            positions, _, cu = step_arrays(starts, counts)
            rows = torch.cat([proj[s][st : st + c] for s, _, st, c in step])
            n = rows.shape[0]
            if splits:
                parts = torch.randn(splits, n, width)
                parts[-1] = rows - parts[:-1].sum(0)
                arg = ops.SplitSum(dev(parts))
            else:
                arg = dev(rows)
            q = torch.empty(n, qw, dtype=dtype, device="cuda")
            g = torch.empty(n, gates, device="cuda") if gates else None
            tab = dev(torch.stack([tables[order.index(s)] for s, *_ in step]))
            ops.conv_store(arg, heads, kv_heads, maps, dim, vdim, gates, dev(w_taps.t()) if taps else None, rot, inv, magnitude,
                           positions, cu, i32([slot for _, slot, _, _ in step]), tab, state,
                           runs(counts, singles, ops.conv_store_tile(max(1, taps))), singles, q, g, k_pool, v_pool, page_size)
            at = 0
            for s, _, st, c in step:
                got_q[s][st : st + c] = q[at : at + c]
                if gates:
                    got_g[s][st : st + c] = g[at : at + c]
                at += c
        return got_q, got_g, k_pool, v_pool, state

    whole = [[("a", 0, 0, 53), ("b", 1, 0, 9), ("c", 2, 0, 40)]]
    cut = [[("a", 3, 0, 2), ("b", 1, 0, 9)], [("a", 3, 2, 1)], [("a", 3, 3, 30), ("c", 1, 0, 1)], [("c", 1, 1, 1), ("a", 3, 33, 1)],
           [("c", 1, 2, 3), ("a", 3, 34, 2)], [("c", 1, 5, 33), ("a", 3, 36, 1)], [("c", 1, 38, 2), ("a", 3, 37, 16)]]
    ones = [[(s, i, t, 1)] for i, s in enumerate(order) for t in range(lens[s])]
    first = run(whole)
    for s in order:
        x = proj[s].double()
        y = plain.short_convolution(x[:, :channels], w_taps.double()) if taps else x[:, :channels]
        pos = torch.arange(lens[s])
        q = plain.rotate_halves(y[:, :qw].reshape(lens[s], heads * maps, dim), pos, spec)
        close(first[0][s].view(lens[s], heads * maps, dim), q, dtype, f"queries of {s}")
        if gates:
            close(first[1][s], torch.sigmoid(x[:, channels : channels + gates]), torch.float32, "gates", tol=1e-6)
        if kv_heads:
            k = plain.rotate_halves(y[:, qw : qw + kw].reshape(lens[s], kv_heads * maps, dim), pos, spec).reshape(lens[s], kv_heads, maps * dim)
            v = y[:, qw + kw :].reshape(lens[s], kv_heads, vdim)
            for t in range(lens[s]):
                page, slot = int(tables[order.index(s), t // page_size]), t % page_size
                close(first[2][page, :, :, slot, :].reshape(kv_heads, maps * dim), k[t], dtype, f"keys of {s} at {t}")
                close(first[3][page, :, :, slot], v[t], dtype, f"values of {s} at {t}")
    for plan, tol in ((cut, None), (ones, None)):
        again = run(plan)
        for s in order:
            if splits:  # (the partial sums themselves differ from step to step)
                close(again[0][s], first[0][s], dtype, tol=2e-5 if dtype == torch.float32 else 1e-2)
            else:
                assert torch.equal(again[0][s], first[0][s]) and torch.equal(again[1][s], first[1][s])
        if kv_heads and not splits:
            assert torch.equal(again[2], first[2]) and torch.equal(again[3], first[3])
    if taps > 1:
        kept = first[4][:3, : (taps - 1) * channels].view(3, taps - 1, channels).cpu()
        for i, s in enumerate(order):
            want = torch.zeros(taps - 1, channels)
            have = min(taps - 1, lens[s])
            want[taps - 1 - have :] = proj[s][lens[s] - have :, :channels].float()
            close(kept[i], want, torch.float32, "kept inputs", tol=1e-5)
        assert torch.equal(first[4][3:].cpu(), torch.full_like(first[4][3:].cpu(), 7.0)), "a slot that nobody holds was written"


# ------------------------------------------------------------------ differential attention

def plain_attention(q, k, v, pos_q, scale, window, keep, diff, lam, eps):
    """One head: q [n, maps, d] at positions pos_q over keys [ctx, maps, d] and values [ctx, v]."""
    out = []
    for r, p in enumerate(pos_q):
        j = torch.arange(p + 1)
        vis = torch.ones(p + 1, dtype=torch.bool) if window is None else (p - j < window) | (j < keep)
        maps = [plain.one_map(q[r : r + 1, m], k[: p + 1, m], v[: p + 1], scale, vis[None])[0] for m in range(q.shape[1])]
        out.append(maps[0] if diff is None else plain.combine_maps(maps[0], maps[1], lam, diff, eps))
    return torch.stack(out)


def fill_pools(keys, values, tables, page_size, dtype, pages):
    """keys [ctx, kv_heads, row], values [ctx, kv_heads, vdim] per sequence; whatever no token holds is large."""
    kv_heads, row, vdim = keys[0].shape[1], keys[0].shape[2], values[0].shape[2]
    slab = 32 if row % 32 == 0 else row
    k_pool = torch.full((pages, kv_heads, row // slab, page_size, slab), 1e4, dtype=dtype, device="cuda")
    v_pool = torch.full((pages, kv_heads, vdim, page_size), 1e4, dtype=dtype, device="cuda")
    for s, (kk, vv) in enumerate(zip(keys, values)):
        for first in range(0, kk.shape[0], page_size):
            page, m = int(tables[s, first // page_size]), min(page_size, kk.shape[0] - first)
            k_pool[page, :, :, :m, :] = kk[first : first + m].to("cuda").view(m, kv_heads, row // slab, slab).permute(1, 2, 0, 3)
            v_pool[page, :, :, :m] = vv[first : first + m].to("cuda").permute(1, 2, 0)
    return k_pool, v_pool


def run_attention(ops, q, sizes, positions, token_seq, cu, tables, ctx, lens, pools, page_size, mask, gate, units):
    """All rows through the general kernel, or single tokens through the decode kernel (with and without
    shared keys) and portions through the prompt kernel (both workgroup sizes, with and without shared keys)."""
    heads, kv_heads, maps, dim, vdim = sizes
    n = q.shape[0]
    out = torch.full((n, heads * vdim), float("nan"), dtype=q.dtype, device="cuda")
    if not units:
        ops.diff_attention(q, out, *sizes, positions, token_seq, tables, *pools, page_size, *mask, gate=gate)
        return [out]
    singles = sum(1 for l in lens if l == 1)
    results = []
    for small in (True, False):
        tiles = ops.diff_attention_tiles(heads, kv_heads, small)
        if not tiles:
            continue
        for nsplit in (1, 3):
            out = torch.full((n, heads * vdim), float("nan"), dtype=q.dtype, device="cuda")
            if singles:
                partial = torch.full((singles * heads * maps * nsplit * (vdim + 2),), float("nan"), device="cuda")
                ops.diff_attention_decode(q, out, singles, *sizes, positions, tables, *pools, page_size, *mask, gate, partial, nsplit,
                                          streaming=small)
            if singles < len(lens):
                rows = n - singles
                partial = torch.full((rows * heads * maps * nsplit * (vdim + 2),), float("nan"), device="cuda") if nsplit > 1 else None
                ops.diff_attention_prefill(q, out, runs(lens, singles, 16 * tiles), *sizes, cu, i32(ctx), tables, *pools, page_size,
                                           *mask, gate, small=small, partial=partial, nsplit=nsplit, first_token=singles)
            results.append(out)
    return results


ATTENTION_CASES = [
    # heads, kv_heads, dim, vdim, page_size, window, keep, diff
    (4, 2, 16, 40, 16, 21, 3, 0.3),
    (3, 3, 7, 9, 4, None, 0, 0.5),
    (6, 1, 24, 20, 8, 1, 1, 0.7),
    (2, 2, 40, 64, 4, 37, 0, 0.4),
    (8, 2, 32, 64, 32, 37, 5, 0.5),
    (10, 1, 16, 32, 16, 300, 40, 0.25),
    (16, 1, 16, 96, 16, 16, 16, 0.6),
    (2, 1, 48, 32, 16, 70, 33, 0.65),
    (4, 4, 64, 128, 16, 100, 2, 0.9),
    (6, 2, 64, 64, 16, None, 0, 0.35),
    (3, 1, 64, 64, 16, 50, 7, None),
    (4, 4, 128, 128, 32, 33, 1, None),
    (5, 1, 12, 30, 8, 50, 9, None),
]


def attention_runs():
    """Every case with every key that its mask has, in the general kernel in both precisions and, where they
    take the sizes (rows and values in 32s up to 128, pages in 16s), on the matrix units."""
    out = []
    for case in ATTENTION_CASES:
        heads, kv_heads, dim, vdim, page_size, window, keep, diff = case
        row = dim * (1 if diff is None else 2)
        units = row % 32 == 0 and row <= 128 and vdim % 32 == 0 and vdim <= 128 and page_size % 16 == 0 and \
            (diff is not None or row == vdim)
        for shows in (["far"] if window is None else ["window"] + (["kept"] if keep else [])):
            out += [(torch.float32, False, shows, *case), (torch.bfloat16, False, shows, *case)]
            if units:
                out.append((torch.bfloat16, True, shows, *case))
    return out


@pytest.mark.parametrize("dtype, units, shows, heads, kv_heads, dim, vdim, page_size, window, keep, diff", attention_runs())
def test_differential_attention(ops, dtype, heads, kv_heads, dim, vdim, page_size, window, keep, diff, units, shows):
    """Two single tokens and two portions (one of two tokens, one that crosses pages) over up to 700 keys.
    For every sequence's last query one key is made to stand out: the last kept one of the first tokens
    ("kept"), the oldest inside the window ("window"), or, without a window, one far back; the key just
    behind the kept ones, and the one just outside the window, are stronger copies of it that must not
    show.  The query before the last points at the key just outside its own window.  Map 2 points elsewhere,
    at the newest key, so that a map that reads the other's keys shows too."""
    maps = 1 if diff is None else 2
    assert not units or ops.diff_attention_supports_mfma(heads, kv_heads, maps, dim, vdim, page_size)
    torch.manual_seed(8)
    ctx, lens = [700, 333, 2, 420], [1, 1, 2, 39]
    starts = [c - l for c, l in zip(ctx, lens)]
    scale, eps, lam = dim**-0.5, 1e-3, 0.8
    tables = tables_for(ctx, page_size, 400, seed=dim)
    keys = [torch.randn(c, kv_heads, maps, dim) * 0.3 for c in ctx]
    values = [torch.randn(c, kv_heads, vdim) for c in ctx]
    n = sum(lens)
    q = torch.randn(n, heads, maps, dim) * 0.3
    gate = torch.rand(n, heads) + 0.2
    row = 0
    for s, (c, l) in enumerate(zip(ctx, lens)):
        last = row + l - 1
        special = {"kept": keep - 1, "window": c - (window or 0), "far": 3}[shows]
        if c > 2 and 0 <= special < c:
            for behind in ([keep] if window is not None and keep < c - window else []) + \
                    ([c - window - 1] if window is not None and c - window - 1 >= keep else []):
                if behind != special:
                    keys[s][behind] = 1.5 * keys[s][special]
            for h in range(heads):
                g = h // (heads // kv_heads)
                k = keys[s][special, g, 0]
                q[last, h, 0] = k / k.norm() ** 2 * 12.0 / scale
                if maps == 2:
                    k = keys[s][c - 1, g, 1]
                    q[last, h, 1] = k / k.norm() ** 2 * 12.0 / scale
                if l > 1 and window is not None and c - window - 2 >= keep:
                    k = keys[s][c - window - 2, g, 0]
                    q[last - 1, h, 0] = k / k.norm() ** 2 * 12.0 / scale
        row += l
    q, keys, values = q.to(dtype), [k.to(dtype) for k in keys], [v.to(dtype) for v in values]
    pools = fill_pools([k.reshape(k.shape[0], kv_heads, maps * dim) for k in keys], values, tables, page_size, dtype, 400)
    positions, token_seq, cu = step_arrays(starts, lens)
    want = torch.zeros(n, heads, vdim, dtype=torch.float64)
    row = 0
    for s, (c, l) in enumerate(zip(ctx, lens)):
        for h in range(heads):
            g = h // (heads // kv_heads)
            want[row : row + l, h] = plain_attention(q[row : row + l, h].double(), keys[s][:, g].double(), values[s][:, g].double(),
                                                     list(range(c - l, c)), scale, window, keep, diff, lam, eps)
        row += l
    want *= gate.double()[:, :, None]
    rest = 1.0 if diff is None else 1.0 - diff
    for out in run_attention(ops, dev(q.reshape(n, -1)), (heads, kv_heads, maps, dim, vdim), positions, token_seq, cu, dev(tables), ctx,
                             lens, pools, page_size, (window, keep, scale, lam, rest, eps), dev(gate), units):
        close(out.view(n, heads, vdim), want, dtype, tol=2.5e-2 if dtype == torch.bfloat16 else None)


@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_in_portions_and_single_tokens(ops, dtype):
    """The same sequence whole, in portions down to two tokens and token by token: the same bits in the
    general kernel; on the matrix units within rounding.  Pages that the window has passed are gone (their
    table entries name no page), those of the kept first tokens are not."""
    torch.manual_seed(9)
    heads, kv_heads, dim, vdim, page_size, window, keep, length = 4, 2, 32, 64, 16, 21, 18, 150
    keys, values = torch.randn(length, kv_heads, 2 * dim).to(dtype), torch.randn(length, kv_heads, vdim).to(dtype)
    tables = tables_for([length], page_size, 40)
    pools = fill_pools([keys], [values], tables, page_size, dtype, 40)
    q, gate = torch.randn(length, heads * 2 * dim).to(dtype), torch.rand(length, heads)

    def run(cuts, units):
        out, at = [], 0
        for c in cuts:
            positions, token_seq, cu = step_arrays([at], [c])
            held = tables.clone()
            held[0, -(-keep // page_size) : max(0, at - window + 1) // page_size] = -1
            out.append(run_attention(ops, dev(q[at : at + c]), (heads, kv_heads, 2, dim, vdim), positions, token_seq, cu, dev(held),
                                     [at + c], [c], pools, page_size, (window, keep, dim**-0.5, 0.5, 0.6, 1e-5), dev(gate[at : at + c]),
                                     units))
            at += c
        return [torch.cat([o[i] for o in out]) for i in range(min(map(len, out)))]

    whole = run([length], False)[0]
    cuts = [2, 30, 1, 1, 17, 2, 22, 40, 1, 3, 31]
    assert torch.equal(run(cuts, False)[0], whole) and torch.equal(run([1] * length, False)[0], whole)
    if dtype == torch.bfloat16:
        for way in ([length], cuts, [1] * length):
            for got in run(way, True):
                close(got, whole, dtype, tol=2.5e-2)


# ------------------------------------------------------------------ lightning attention

LIGHT_CASES = [(2, 64, 32), (1, 32, 64), (3, 128, 32), (2, 96, 96), (1, 192, 32), (1, 256, 64)]


def _plain_lightning(p, heads, dim, v_dim, decay, off):
    qk, vv = heads * dim, heads * v_dim
    q, k, v = (plain.silu(p[:, o : o + w]).view(p.shape[0], heads, -1) for o, w in ((off, qk), (off + qk, qk), (off + 2 * qk, vv)))
    return torch.stack([plain.lightning_recurrence(q[:, a], k[:, a], v[:, a], decay[a]) for a in range(heads)], 1).reshape(-1, vv)


@pytest.mark.parametrize("kernel, heads, dim, v_dim", [(k, *c) for c in LIGHT_CASES for k in ("scan_f32", "scan_bf16", "chunk")]
                         + [(k, *c) for c in ((2, 20, 12), (3, 7, 5)) for k in ("scan_f32", "scan_bf16")])
def test_lightning_in_pieces_and_in_used_slots(ops, kernel, heads, dim, v_dim):
    """Three sequences in portions and single tokens over slots that earlier holders left full; the scan
    applies SiLU itself, the chunked kernel takes activated rows (and leaves single tokens to the scan)."""
    assert kernel != "chunk" or ops.retention_chunk_supports(dim, v_dim)
    torch.manual_seed(dim + v_dim)
    decay = [1.0, 0.4, 0.97][:heads]
    lens = {"a": 205, "b": 64, "c": 131}
    qk, vv = heads * dim, heads * v_dim
    ld = -(-(2 * qk + vv) // 8) * 8 + 8
    dtype = torch.float32 if kernel == "scan_f32" else torch.bfloat16
    proj = {s: torch.randn(n, ld).to(dtype) for s, n in lens.items()}
    if kernel == "chunk":
        rows = {s: plain.silu(p.float()).to(dtype) for s, p in proj.items()}
        want = {}
        for s, p in rows.items():  # the plain recurrence over the activated rows as they are rounded
            x = p.double()
            q, k, v = x[:, :qk].view(-1, heads, dim), x[:, qk : 2 * qk].view(-1, heads, dim), x[:, 2 * qk : 2 * qk + vv].view(-1, heads, v_dim)
            want[s] = torch.stack([plain.lightning_recurrence(q[:, a], k[:, a], v[:, a], decay[a]) for a in range(heads)], 1).reshape(-1, vv)
    else:
        rows = proj
        want = {s: _plain_lightning(p.double(), heads, dim, v_dim, decay, 0) for s, p in proj.items()}
    state = torch.full((3, ops.retention_state_floats(heads, dim, v_dim)), -3.0, device="cuda")
    plan = [[("a", 0, 0, 2), ("b", 1, 0, 64)], [("a", 0, 2, 1)], [("c", 1, 0, 1), ("a", 0, 3, 100)], [("c", 1, 1, 1), ("a", 0, 103, 1)],
            [("c", 1, 2, 65), ("a", 0, 104, 64)], [("c", 1, 67, 64), ("a", 0, 168, 37)]]
    got = {s: torch.zeros(n, vv, device="cuda") for s, n in lens.items()}
    for step in plan:
        starts, counts = [e[2] for e in step], [e[3] for e in step]
        singles = sum(c == 1 for c in counts)
        assert all(c == 1 for c in counts[:singles])
        positions, _, cu = step_arrays(starts, counts)
        x = dev(torch.cat([rows[s][st : st + c] for s, _, st, c in step]))
        slots, out = i32([slot for _, slot, _, _ in step]), torch.full((x.shape[0], vv), float("nan"), device="cuda")
        args = (heads, dim, v_dim, positions, cu, slots, state, out)
        if kernel == "chunk":
            ops.retention_chunk(x, 0, qk, 2 * qk, dev(torch.tensor(decay)), singles, len(step) - singles, *args)
            if singles:
                ops.retention_scan(x, 0, qk, 2 * qk, dev(torch.tensor(decay)), singles, *args)
        else:
            ops.retention_scan(x, 0, qk, 2 * qk, dev(torch.tensor(decay)), len(step), *args, activation="silu")
        at = 0
        for s, _, st, c in step:
            got[s][st : st + c] = out[at : at + c]
            at += c
    for s in lens:
        # (decayed operands of the chunk's products are sums of two bfloat16 numbers)
        close(got[s], want[s], torch.float32, f"sequence {s}", tol=3e-5 if kernel == "chunk" else 2e-5)


def test_lightning_chunks_keep_a_far_token_and_forget(ops):
    """With decay 1 the first token's value comes back whole 600 tokens later, through chunks and single
    tokens; with decay 0.5 it is gone; with decay 0 a token sees itself alone."""
    heads, dim, v_dim, n = 3, 32, 32, 640
    qk = heads * dim
    rows = torch.zeros(n, 2 * qk + heads * v_dim, dtype=torch.bfloat16)
    rows[0, qk : 2 * qk] = 1.0
    rows[0, 2 * qk :] = 2.0
    rows[:, :qk] = 1.0 / dim  # every q: q . k_0 = 1
    rows[600, qk : 2 * qk], rows[600, 2 * qk :] = 0.5, 3.0  # o_600 = S_600 q: 0.5 * 3 for a decay of 0
    state = torch.full((1, ops.retention_state_floats(heads, dim, v_dim)), 9.0, device="cuda")
    decay, res = dev(torch.tensor([1.0, 0.5, 0.0])), []
    for start, count in [(0, 130), (130, 2), (132, 300), (432, 64), (496, 95)] + [(591 + i, 1) for i in range(9)] + [(600, 40)]:
        positions, _, cu = step_arrays([start], [count])
        out = torch.empty(count, heads * v_dim, device="cuda")
        args = (heads, dim, v_dim, positions, cu, i32([0]), state, out)
        x = dev(rows[start : start + count])
        if count > 1:
            ops.retention_chunk(x, 0, qk, 2 * qk, decay, 0, 1, *args)
        else:
            ops.retention_scan(x, 0, qk, 2 * qk, decay, 1, *args)
        res.append(out)
    o = torch.cat(res).view(n, heads, v_dim).cpu()
    assert torch.allclose(o[599, 0], torch.full((v_dim,), 2.0)) and float(o[599, 1].abs().max()) < 1e-30
    assert torch.allclose(o[600], torch.tensor([3.5, 1.5, 1.5])[:, None].expand(3, v_dim)) and float(o[601, 2].abs().max()) == 0.0
    assert torch.allclose(o[639, 0], torch.full((v_dim,), 3.5)) and torch.isfinite(o).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n, heads, size, gate_dtype", [(3, 1, 700, "float32"), (600, 1, 640, "same"), (2, 1, 5000, "same"), (9, 4, 48, "same"),
                                                        (4, 2, 513, "float32")])
def test_norm_and_gate_over_many_heads(ops, dtype, n, heads, size, gate_dtype):
    torch.manual_seed(3)
    o, w = torch.randn(n, heads * size) * 4, torch.rand(heads * size) + 0.5
    g = torch.randn(n, heads * size + 8).to(torch.float32 if gate_dtype == "float32" else dtype)
    out = torch.empty(n, heads * size, dtype=dtype, device="cuda")
    for act in ("sigmoid", "silu"):
        ops.headnorm_gate(dev(o), dev(g)[:, 8:], dev(w), 1e-3, out, heads, size, gate_act=act)
        z = g[:, 8:].double()
        want = plain.unit_rms(o.double().view(n, heads, size), 1e-3).reshape(n, -1) * w.double() * torch.sigmoid(z)
        close(out, want * z if act == "silu" else want, dtype)


def test_sizes_that_the_kernels_do_not_take_are_refused(ops):
    q = torch.zeros(1, 2 * 2 * 300, device="cuda")
    pool = torch.zeros(1, 1, 1, 16, 600, device="cuda")
    v = torch.zeros(1, 1, 8, 16, device="cuda")
    one = i32([0])
    with pytest.raises(Exception, match="256"):
        ops.diff_attention(q, torch.zeros(1, 16, device="cuda"), 2, 1, 2, 300, 8, one, one, i32([[0]]), pool, v, 16, None, 0, 1.0, 0.0, 1.0,
                           1e-5)
    assert not ops.diff_attention_supports_mfma(4, 2, 2, 80, 128, 16) and not ops.diff_attention_supports_mfma(4, 2, 2, 32, 64, 8)
    assert not ops.retention_chunk_supports(48, 32) and not ops.retention_chunk_supports(64, 20)
    assert math.isclose(ops.conv_store_tile(4), 8) and ops.conv_store_tile(33) == 32
