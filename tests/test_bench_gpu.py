"""bench.py's own runs on a tiny model: the offline run hands out what it was asked
for, and a decode run counts its tokens (the numbers themselves are the bench's)."""

import importlib.util
from pathlib import Path

import pytest

from .tiny import CONFIGS

pytestmark = pytest.mark.gpu

spec_ = importlib.util.spec_from_file_location("bench", Path(__file__).resolve().parent.parent / "bench.py")
bench = importlib.util.module_from_spec(spec_)
spec_.loader.exec_module(bench)


def test_offline_run_and_decode_run_on_a_tiny_model():
    import shrike_amd.models  # noqa: F401
    from shrike_amd.models.qwen2 import Qwen2Config, build_spec

    cfg = Qwen2Config.from_dict(dict(CONFIGS["B"], torch_dtype="bfloat16"))
    spec = build_spec(cfg)
    got = bench.run_offline(cfg, spec, 12, seed=3)
    assert got["tokens"] >= 12 * 32 and got["tok_s"] > 0 and got["preemptions"] == 0
    assert got["steps"] >= 32 and got["token_budget"] == 512 and got["page_size"] == 16
    engine = bench.make_engine(cfg, spec, 4, seed=1)
    run = bench.run_decode(engine, cfg, 4, steps=10, warmup=2, seed=5, prompt_len=40)
    assert run["context_end"] - run["context_start"] == 10 and run["tok_s"] > 0
    sampled = bench.run_decode(engine, cfg, 4, steps=10, warmup=2, seed=6, prompt_len=40, temperature=0.8, top_p=0.9)
    assert sampled["context_end"] - sampled["context_start"] == 10


def test_products_mode_times_every_product_of_a_layer_both_ways():
    import shrike_amd.models  # noqa: F401
    from shrike_amd.models.qwen2 import Qwen2Config

    cfg = Qwen2Config.from_dict(dict(CONFIGS["D"], torch_dtype="bfloat16"))
    got = bench.run_products(cfg, [8, 200])
    assert set(got) == {f"{name}_n{n}" for n in (8, 200) for name in ("qkv", "o", "gate_up", "down")} | {"lm_head_n8"}
    for entry in got.values():
        assert entry["own_us"] > 0 and entry["library_us"] > 0 and entry["k_shares"] >= 1


def test_the_second_design_of_the_comparison_is_built_from_the_first_ones_sizes_and_decodes():
    """bench.py --minilorn: a Minilorn with a Qwen2 configuration's width, heads, feed-forward width and
    number of layers, every mixer in the pattern's order; it takes prompts in and decodes like the other."""
    import shrike_amd.models  # noqa: F401
    from shrike_amd.models import minilorn
    from shrike_amd.models.qwen2 import Qwen2Config

    qcfg = Qwen2Config.from_dict(dict(CONFIGS["B"], torch_dtype="bfloat16"))
    mcfg, sizes = bench.minilorn_like(qcfg, window=48, pattern="lma")
    assert [layer.type for layer in mcfg.layers][:3] == ["latent_attention", "mlstm", "attention"][: len(mcfg.layers)]
    assert len(mcfg.layers) == qcfg.num_hidden_layers and mcfg.width == qcfg.hidden_size
    assert all(layer.ff == qcfg.intermediate_size for layer in mcfg.layers)
    assert sizes.layer_elements > 2 * qcfg.hidden_size * qcfg.intermediate_size and sizes.kv_elements_per_token > 0
    engine = bench.make_engine(sizes, minilorn.build_spec(mcfg), 4, seed=1)
    run = bench.run_decode(engine, sizes, 4, steps=10, warmup=2, seed=5, prompt_len=70)
    assert run["context_end"] - run["context_start"] == 10 and run["tok_s"] > 0


def test_the_bevovik_of_the_comparison_is_built_from_the_first_ones_sizes_and_decodes():
    """bench.py --bevovik: a Qwen2 configuration's width, vocabulary and number of layers, every mixer in the
    pattern's order, experts that together are as large as its feed-forward."""
    import shrike_amd.models  # noqa: F401
    from shrike_amd.models import bevovik
    from shrike_amd.models.qwen2 import Qwen2Config

    qcfg = Qwen2Config.from_dict(dict(CONFIGS["B"], hidden_size=256, num_hidden_layers=4, torch_dtype="bfloat16"))
    bcfg, sizes = bench.bevovik_like(qcfg, "grl", experts=6, top=2)
    assert [layer.type for layer in bcfg.layers] == ["gla", "rglru", "latent_attention", "gla"]
    assert bcfg.width == 256 and bcfg.vocab == qcfg.vocab_size and sizes.kv_elements_per_token > 0
    router = bcfg.layers[0].mlp
    assert (router.experts, router.identity, router.groups, router.top) == (6, 2, (2, 1), 2)
    few = sizes.layer_elements
    sizes.at_batch(64)
    assert sizes.layer_elements > few, "many tokens touch more experts than one token's"
    engine = bench.make_engine(sizes, bevovik.build_spec(bcfg), 4, seed=1)
    run = bench.run_decode(engine, sizes, 4, steps=10, warmup=2, seed=5, prompt_len=70)
    assert run["context_end"] - run["context_start"] == 10 and run["tok_s"] > 0
