"""The Bevovik decoder in the engine against its plain implementation (tests/plain/bevovik.py), on tiny
models with random weights (tests/tiny_bevovik.py): the stream after every layer; whole prompts, single
tokens from the very first, portions down to two tokens and mixed batches over so few pages that they are
used again (all pages that nobody holds poisoned with NaN); a far token that must be found in a prompt and
while decoding; long decoding; a single state slot for several requests in turn; greedy generation through
the entry point and its scheduler, with preemption; graphs and recorded launches against kernel-by-kernel
steps; the command line."""

import random

import numpy as np
import pytest
import torch

from .compare import GreedyCheck
from .plain.bevovik import PlainBevovik
from .tiny_bevovik import CONFIGS, PAGE_SIZES, make_model_dir
from .traces import (TraceBuilder, changing_portions, check_pages, last_one_by_one, mixed, read_pages,
                     run_trace, whole)

pytestmark = pytest.mark.gpu

TOL = {"float32": 1e-4, "bfloat16": 3e-2}
# lengths on both sides of a page, of a convolution's taps and of the chunks of 64 tokens that prompts run in
LENGTHS = {"A": [1, 6, 49, 97, 130, 10], "B": [3, 41, 38, 29, 8, 150], "C": [2, 64, 17, 65, 300]}


@pytest.fixture(scope="module")
def model_root(tmp_path_factory):
    return tmp_path_factory.mktemp("bevovik_models")


def requests_for(name: str, lengths=None, seed: int = 0) -> dict[str, list[int]]:
    rng = random.Random(sum(map(ord, name)) + seed)
    vocab = CONFIGS[name]["vocab"]
    return {f"r{i}": [rng.randrange(vocab) for _ in range(n)] for i, n in enumerate(lengths or LENGTHS[name])}


def engine_parts(model_dir, dtype, page_size, pages, graphs=True, slots=4):
    from shrike_amd.cache import CacheManager
    from shrike_amd.engine.loading import load_model
    from shrike_amd.engine.runner import ModelRunner

    model, rt, _cfg = load_model(model_dir, dtype)
    cache = CacheManager(model.cache_specs(), page_size, pages, max_slots=slots, enable_prefix_caching=False)
    cache.allocate(rt.dtype, rt.device)
    return model, cache, ModelRunner(model, cache, rt, graphs=graphs)


def rel_errors(got, want):
    return (got.double() - want).abs().amax(-1) / want.abs().max()


def check_errors(err, dtype):
    """float32: every row.  bfloat16: where a head's readout is nearly nothing (q . k close to zero among a
    sequence's first tokens, say) its norm carries the rounding of its inputs undamped: such rows are few,
    and bounded."""
    assert float(err.max()) <= (TOL[dtype] if dtype == "float32" else 0.5), f"row {int(err.argmax())}: {float(err.max()):.3e}"
    assert float((err > TOL[dtype]).double().mean()) <= 0.03, float((err > TOL[dtype]).double().mean())


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_the_stream_after_every_layer(name, model_root):
    """float32: the stream that every layer leaves against the plain model's, for a prompt of
    more than one chunk."""
    from shrike_amd.engine.runner import StepEntry

    model_dir = make_model_dir(name, model_root, dtype="float32")
    ids = requests_for(name, [75])["r0"]
    want = PlainBevovik(model_dir).layers(ids)
    model, cache, runner = engine_parts(model_dir, "float32", 16, 16, graphs=False)
    runner.use_call_lists = False
    seen = []
    for block in model.blocks:
        def wrapped(ctx, hidden, layer_cache, inner=block.forward):
            inner(ctx, hidden, layer_cache)
            hidden.settle(ctx)
            seen.append(hidden.resid.detach().cpu().double().clone())

        block.forward = wrapped
    seq = cache.new_sequence()
    cache.append(seq, 0, len(ids))
    runner.step([StepEntry(seq, ids, 0, [len(ids) - 1])])
    assert len(seen) == want.shape[0] == len(CONFIGS[name]["layers"])
    for i, (got, ref) in enumerate(zip(seen, want)):
        err = float((got - ref).abs().max() / ref.abs().max())
        assert err <= 2e-5, f"layer {i} ({CONFIGS[name]['layers'][i]['type']}): rel err {err:.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name, page_size", [("A", 16), ("B", 4), ("B", 16), ("C", 32), ("A", 8), ("C", 16)])
def test_four_cuttings_agree_with_the_plain_implementation(name, page_size, dtype, model_root, tmp_path):
    model_dir = make_model_dir(name, model_root, dtype=dtype)
    vocab = CONFIGS[name]["vocab"]
    seqs = requests_for(name)
    plain = PlainBevovik(model_dir)
    want = {rid: plain.logits(ids).numpy() for rid, ids in seqs.items()}

    tb = TraceBuilder()
    budget = max(-(-len(ids) // 64) * 64 for ids in seqs.values())
    whole(tb, "w_", seqs)
    last_one_by_one(tb, "d_", seqs, tail=45)
    changing_portions(tb, "p_", seqs)
    mixed_budget = budget + 128
    mixed(tb, "m_", seqs, mixed_budget, seed=5)
    outputs = run_trace(model_dir, dtype, tb.steps, mixed_budget, tmp_path / "out", vocab,
                        block_size=page_size, poison=True, pages=True)
    got = tb.collect(outputs)
    assert all(np.isfinite(rows).all() for rows in outputs.values()), "a page that nobody holds was read"
    reused = check_pages(tb.steps, read_pages(tmp_path / "out", tb.steps), page_size, mixed_budget // page_size)
    assert reused > 0, "the pool was meant to be so small that pages are used again"

    worst, errors = {}, []
    for (rid, pos), row in got.items():
        cut, name_ = rid.split("_", 1)
        err = np.abs(row.astype(np.float64) - want[name_][pos]).max() / np.abs(want[name_]).max()
        worst[cut] = max(worst.get(cut, 0.0), err)
        errors.append(err)
        if dtype == "float32":  # every float32 kernel sums a row in one order whatever the step holds
            assert np.array_equal(row, got[(f"w_{name_}", pos)]), f"{rid} position {pos} differs from the whole prompt's"
    check_errors(torch.tensor(errors), dtype)
    assert set(worst) == {"w", "d", "p", "m"}
    for cut in "wdp":
        assert all((f"{cut}_{rid}", p) in got for rid, ids in seqs.items() for p in range(len(ids)))
    print(f"{name} page {page_size} {dtype}: worst rel err per cutting {worst}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_long_decoding_from_the_first_token(name, dtype, model_root):
    """Every token on the single-token path (graphs included)."""
    from shrike_amd.engine.runner import StepEntry

    model_dir = make_model_dir(name, model_root, dtype=dtype)
    model, cache, runner = engine_parts(model_dir, dtype, PAGE_SIZES[name], 64)
    ids = requests_for(name, [230], seed=3)["r0"]
    seq = cache.new_sequence()
    rows = []
    for p, tok in enumerate(ids):
        cache.append(seq, p, 1)
        rows.append(runner.step([StepEntry(seq, [tok], p, [0])]).cpu().clone())
        cache.trim(seq, p + 1)
    check_errors(rel_errors(torch.cat(rows), PlainBevovik(model_dir).logits(ids)), dtype)
    assert runner.graph_replays > 100
    cache.free(seq)
    cache.check([])


@pytest.mark.parametrize("kind", ["latent_attention", "gla", "rglru"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_token_moves_the_last_positions(dtype, kind, tmp_path):
    """Models of one mixer in which a marked token, far back, matters at the end: steep attention scores,
    decays of nearly one, a token of a large embedding.  The engine's logits move by it as the plain model's
    do, whether the last tokens come in the prompt or are decoded."""
    from safetensors.torch import load_file, save_file

    from shrike_amd.engine.runner import StepEntry
    from shrike_amd.weights import write_model_folder

    layer = next({**x, "mlp": None} for x in CONFIGS["C"]["layers"] if x["type"] == kind)
    cfg = {**CONFIGS["C"], "layers": [layer]}
    model_dir = write_model_folder(cfg, tmp_path / "model", seed=5, dtype=dtype, mode="unit")
    w = load_file(str(model_dir / "model.safetensors"))
    marked = cfg["vocab"] - 1
    w["embed"][marked] *= 12.0
    if kind == "latent_attention":
        w["l0.mix.uk"] *= 4.0
    elif kind == "gla":
        w["l0.mix.a2.b"] += 9.0
    else:
        w["l0.mix.lam"].fill_(-9.0)
    save_file(w, str(model_dir / "model.safetensors"))
    plain = PlainBevovik(model_dir)
    rng = random.Random(8)
    ids = [rng.randrange(marked) for _ in range(333)]
    other = ids[:2] + [marked] + ids[3:]
    want = torch.stack([plain.logits(x)[-3:] for x in (ids, other)])
    moved = float((want[1] - want[0]).abs().max())
    assert moved > 3 * TOL[dtype] * float(want.abs().max()), moved
    for decoded in (0, 40):
        model, cache, runner = engine_parts(model_dir, dtype, 16, 64)
        got = []
        for seq_ids in (ids, other):
            seq, rows = cache.new_sequence(), []
            cuts = [len(seq_ids) - decoded] + [1] * decoded
            at = 0
            for n in cuts:
                cache.append(seq, at, n)
                rows.append(runner.step([StepEntry(seq, seq_ids[at : at + n], at, list(range(n)))]).cpu().clone())
                at += n
            cache.free(seq)
            got.append(torch.cat(rows)[-3:].double())
        diff = (got[1] - got[0]) - (want[1] - want[0])
        assert float(diff.abs().max()) <= (1e-3 if dtype == "float32" else 0.3) * moved, (decoded, float(diff.abs().max()), moved)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_one_state_slot_for_requests_in_turn(name, dtype, model_root):
    """Convolution inputs and recurrent state that an earlier request left in the only slot do not reach
    the next one, whether it starts with one token or with a portion."""
    from shrike_amd.engine.runner import StepEntry

    model_dir = make_model_dir(name, model_root, dtype=dtype)
    plain = PlainBevovik(model_dir)
    model, cache, runner = engine_parts(model_dir, dtype, 16, 8, slots=1)
    for state in cache.state_groups:
        state.padded.fill_(1e3)
    errors = []
    for ids, first in zip(requests_for(name, [40, 3, 25, 1, 60], seed=6).values(), (7, 1, 25, 1, 2)):
        seq, rows, at = cache.new_sequence(), [], 0
        for group in cache.state_groups:
            group.tensor[:, seq.state_slot] = -50.0  # (the slot is not even cleared)
        while at < len(ids):
            n = min(first if at == 0 else 5, len(ids) - at)
            cache.append(seq, at, n)
            rows.append(runner.step([StepEntry(seq, ids[at : at + n], at, list(range(n)))]).cpu().clone())
            at += n
        errors.append(rel_errors(torch.cat(rows), plain.logits(ids)))
        cache.free(seq)
    check_errors(torch.cat(errors), dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name, lengths, new, budget", [("A", [1, 20, 47, 30], 40, 16), ("B", [5, 13, 2], 30, 512),
                                                        ("C", [70, 3], 25, 68)])
def test_greedy_generation_through_the_entry_point(name, lengths, new, budget, dtype, model_root):
    """Prompts in portions under a small token budget beside decoding requests, through
    LLM.generate and its scheduler; float32: the plain model's greedy tokens exactly."""
    from shrike_amd import LLM, SamplingParams

    model_dir = make_model_dir(name, model_root, dtype=dtype)
    prompts = list(requests_for(name, lengths, seed=9).values())
    llm = LLM(str(model_dir), dtype=dtype, block_size=PAGE_SIZES[name], num_kv_blocks=96, max_tokens_per_step=budget)
    outs = llm.generate(prompts, SamplingParams(max_new_tokens=new, ignore_eos=True))
    assert [len(o) for o in outs] == [new] * len(prompts)
    check = GreedyCheck(PlainBevovik(model_dir), dtype)
    for prompt, out in zip(prompts, outs):
        check.request(prompt, out)
    check.finish()
    assert len({tok for out in outs for tok in out}) > new // 3, "the tokens were meant to vary"
    assert llm.engine.cache.num_free == llm.engine.cache.num_pages


def test_generation_survives_preemption_when_pages_run_out(model_root):
    """So few pages that the newest request is preempted, gives its pages and state back and recomputes
    from its first token: the tokens are the plain model's all the same."""
    from shrike_amd import LLM, SamplingParams

    model_dir = make_model_dir("A", model_root, dtype="float32")
    plain = PlainBevovik(model_dir)
    prompts = list(requests_for("A", [30, 28, 33], seed=2).values())
    llm = LLM(str(model_dir), dtype="float32", block_size=16, num_kv_blocks=9, max_tokens_per_step=64)
    outs = llm.generate(prompts, SamplingParams(max_new_tokens=40, ignore_eos=True))
    assert llm.engine.metrics()["preemptions"] > 0
    for prompt, out in zip(prompts, outs):
        assert out == plain.greedy(prompt, 40)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_graphs_and_recorded_launches_equal_kernel_by_kernel_steps(name, dtype, model_root):
    """The same steps with and without HIP graphs and recorded launch lists: the same bits."""
    from shrike_amd.engine.runner import StepEntry

    model_dir = make_model_dir(name, model_root, dtype=dtype)
    ids = requests_for(name, [90, 41], seed=4)
    results = []
    for graphs in (True, False):
        model, cache, runner = engine_parts(model_dir, dtype, 16, 32, graphs=graphs)
        a, b = cache.new_sequence(), cache.new_sequence()
        rows = []
        pa = pb = 0
        for step in range(40):
            entries = []
            na = 7 if pa < 60 else 1  # portions of a first, then single tokens
            na = min(na, len(ids["r0"]) - pa)
            if na:
                cache.append(a, pa, na)
                entries.append(StepEntry(a, ids["r0"][pa : pa + na], pa, [na - 1]))
            nb = 1 if pb < len(ids["r1"]) else 0
            if nb:
                cache.append(b, pb, 1)
                entries.append(StepEntry(b, [ids["r1"][pb]], pb, [0]))
            if not entries:
                break
            rows.append(runner.step(entries).cpu().clone())
            pa, pb = pa + na, pb + nb
            cache.trim(a, pa), cache.trim(b, pb)
        if graphs:
            assert runner.graph_replays > 0 and runner.list_replays > 0
        results.append(torch.cat(rows))
    assert torch.equal(results[0], results[1])


def test_command_line_generates_with_a_model_folder(model_root, capsys):
    from shrike_amd.__main__ import main

    model_dir = make_model_dir("A", model_root, dtype="float32")
    rc = main(["--model", str(model_dir), "--prompt-ids", "5,6,7,8,140,2", "--max-tokens", "9", "--dtype", "fp32",
               "--block-size", "4", "--num-kv-blocks", "16", "--ignore-eos", "--metrics"])
    assert rc == 0
    out = capsys.readouterr()
    assert [int(t) for t in out.out.split()] == PlainBevovik(model_dir).greedy([5, 6, 7, 8, 140, 2], 9)
    assert "tokens_generated" in out.err
