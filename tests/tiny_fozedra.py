"""Tiny Fozedra configurations for tests.  They differ from each other in every size and option: both
mixers in several orders and more than once; grouped, ungrouped and single key/value heads, more than
eight heads of one key/value head; values smaller and larger than a map's queries; map sizes that are and
are not multiples of 16 or 32, odd ones too; convolutions of none, 1, 2, 3, 4, 5 and 12 taps; windows of
1, 5, 16, 20, 37 and 1,000 positions (smaller than a page, exactly a page, across page edges, larger
than any test sequence) that keep none, one, some, a page's worth and more of the first tokens, and no
window; rotation of none, some and all elements, with and without stretched rates; layers that read an
earlier layer's keys and values with masks of their own, wider and narrower than the owner's, with more
and fewer kept tokens, and more than one reader of one cache; lightning heads with decays from 0.3 to 1;
layers without a feed-forward; widths that are multiples of nothing."""

from __future__ import annotations

import tempfile
from pathlib import Path


def _attn(heads, kv_heads, dim, vdim, diff, conv=None, mask=None, rot=None, scaling=None, kv_from=None, scale=None, ff=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff,
             "scale": dim**-0.5 if scale is None else scale}
    if conv is not None:
        mixer["conv"] = conv
    if mask is not None:
        mixer["mask"] = {"size": mask[0], "keep_first": mask[1]}
    if rot is not None:
        mixer["rot"] = {"base": rot[0], "dims": rot[1]}
        if scaling is not None:
            mixer["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _light(heads, dim, vdim, decay, ff=None):
    assert len(decay) == heads
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


FOZ_A = {
    "architecture": "Fozedra", "vocab": 211, "width": 70, "norm": {"eps": 1e-6}, "residual_mult": 0.5,
    "layers": [
        _attn(4, 2, 16, 40, 0.3, conv=3, mask=(5, 2), rot=(500.0, 8), scaling=(4.0, 64, 16.0, 1.0), ff=80),
        _light(3, 20, 12, (1.0, 0.5, 0.97)),
        # reads a windowed layer's cache with a wider window that keeps more
        _attn(4, 2, 16, 40, 0.8, conv=5, mask=(37, 7), rot=(500.0, 8), scaling=(4.0, 64, 16.0, 1.0), kv_from=0, ff=30),
        _attn(3, 3, 7, 9, 0.5, ff=44),
        _attn(3, 3, 7, 9, 0.2, mask=(1, 0), kv_from=3),
    ],
}

FOZ_B = {
    "architecture": "Fozedra", "vocab": 97, "width": 100, "norm": {"eps": 1e-4}, "residual_mult": 1.3,
    "layers": [
        _light(2, 32, 64, (0.999, 0.3), ff=50),
        _attn(6, 1, 24, 20, 0.7, conv=1, mask=(16, 16), rot=(90.0, 24), ff=60),
        _attn(2, 2, 40, 64, 0.4, conv=12, mask=(20, 1), rot=(1.0e5, 2), scale=0.3),
        # a causal layer that reads a windowed layer's cache: that cache keeps everything
        _attn(2, 2, 40, 64, 0.6, conv=2, rot=(1.0e5, 2), kv_from=2, ff=33),
        _light(1, 64, 32, (0.9,)),
        _attn(2, 2, 40, 64, 0.1, conv=12, mask=(5, 3), rot=(1.0e5, 2), kv_from=2),
    ],
}

FOZ_C = {  # (bfloat16: the kernels on the matrix units, maps that share operand slices among them)
    "architecture": "Fozedra", "vocab": 300, "width": 128, "norm": {"eps": 2e-5}, "residual_mult": 0.4,
    "layers": [
        _attn(8, 2, 32, 64, 0.5, conv=4, mask=(37, 3), rot=(1.0e4, 32), scaling=(2.5, 200, 8.0, 2.0), ff=256),
        _light(2, 64, 96, (0.99, 0.8), ff=96),
        _attn(10, 1, 16, 32, 0.25, conv=2, mask=(1000, 5), rot=(300.0, 8)),
        _attn(8, 2, 32, 64, 0.35, conv=3, mask=(16, 20), rot=(1.0e4, 32), scaling=(2.5, 200, 8.0, 2.0), kv_from=0, ff=64),
        _attn(2, 1, 48, 32, 0.65, conv=4, mask=(70, 33), ff=128),
        _attn(3, 3, 64, 128, 0.9, conv=4, rot=(1.0e6, 64)),
    ],
}

CONFIGS = {"A": FOZ_A, "B": FOZ_B, "C": FOZ_C}
SEEDS = {"A": 11, "B": 23, "C": 37}
PAGE_SIZES = {"A": 16, "B": 4, "C": 32}


def make_model_dir(name: str, root=None, dtype: str = "float32", mode: str = "unit") -> Path:
    """Writes the tiny model `name` with seeded random weights (stored in `dtype`) into
    `root` (or a fresh temporary folder) and returns the folder.  The last map's weight is drawn
    around zero and the embedding is small beside what the layers add: else, the output matrix being
    the embedding, every token's best successor would be itself, whatever the layers do."""
    import torch
    from safetensors.torch import load_file, save_file

    from shrike_amd.weights import write_model_folder

    if root is None:
        root = tempfile.mkdtemp(prefix="shrike_tiny_")
    path = Path(root) / f"fozedra_{name}_{dtype}_{mode}"
    if not (path / "model.safetensors").is_file():
        write_model_folder(dict(CONFIGS[name]), path, seed=SEEDS[name], dtype=dtype, mode=mode)
        tensors = load_file(str(path / "model.safetensors"))
        last = tensors["final.norm"]
        gen = torch.Generator().manual_seed(SEEDS[name])
        tensors["final.norm"] = torch.randn(last.shape, generator=gen).to(last.dtype)
        tensors["embed"] = tensors["embed"] * 0.25
        save_file(tensors, str(path / "model.safetensors"))
    return path
