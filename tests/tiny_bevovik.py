"""Tiny Bevovik configurations for tests.  They differ from each other in every size and option: the
three mixers in several orders and more than once; 1 to 6 heads, values smaller than, equal to and
larger than keys, head sizes that are and are not multiples of 32; decays with tau from 0.5 (steep) to 200
(a memory of thousands of tokens) through products of rank 1 to 24; latent attention rotated whole, with and
without stretched rates, and not at all, with latents wider and narrower than the heads; recurrent
widths smaller and larger than the model's, in 1 to 6 blocks, behind convolutions of 1 to 5 taps;
3 to 12 experts of which 1 to 6 are chosen, in 1 to 6 groups of which one to all are kept, with none
to five identity experts (a whole group of them too), limits of 0.3 to 7 that differ between routed and
shared experts, shared experts wider and narrower than the routed ones and none; router scales on both
sides of 1; layers without a feed-forward; widths that are multiples of nothing."""

from __future__ import annotations

import tempfile
from pathlib import Path


def _gla(heads, dim, vdim, tau, rank):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}}


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=10000.0, scaling=None, scale=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
             "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}
    if rot_dim:
        mixer["rot"] = {"base": base, "dims": rot_dim}
        if scaling is not None:
            mixer["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mixer": mixer}


def _rec(width, blocks, conv):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def _moe(experts, top, ff, limit, identity=0, groups=None, scale=1.0, shared=None):
    router = {"experts": experts, "top": top, "identity": identity, "scale": scale}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}
    if shared is not None:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def _with(layer, mlp):
    return {**layer, "mlp": mlp}


BEV_A = {
    "architecture": "Bevovik", "vocab": 211, "width": 70, "norm": {"eps": 1e-5},
    "layers": [
        _with(_rec(96, 3, 4), _moe(5, 2, 24, 2.0, identity=1, groups=(3, 2), scale=1.5, shared=(40, 0.7))),
        _with(_gla(3, 20, 12, 8.0, 5), _moe(7, 3, 16, 0.5, identity=5, groups=(2, 1), scale=0.8)),
        _with(_latent(3, 24, 8, 20, 40, 32, base=500.0, scaling=(4.0, 64, 8.0, 1.0)), None),
        _with(_rec(60, 5, 1), _moe(3, 3, 20, 3.0, identity=0, shared=(12, 3.0))),
    ],
}

BEV_B = {
    "architecture": "Bevovik", "vocab": 97, "width": 100, "norm": {"eps": 1e-4},
    "layers": [
        _with(_latent(5, 12, 6, 30, 20, 50, base=90.0), _moe(6, 4, 12, 0.3, identity=2, groups=(4, 2), scale=2.5, shared=(25, 7.0))),
        _with(_gla(1, 7, 40, 200.0, 24), None),
        _with(_latent(1, 40, 0, 12, 8, 16), _moe(4, 1, 30, 1.0, identity=4, groups=(2, 2), scale=3.0)),
        _with(_rec(44, 1, 5), _moe(12, 6, 8, 7.0, identity=0, groups=(6, 3), scale=1.0, shared=(8, 0.4))),
        _with(_gla(6, 16, 5, 0.5, 1), _moe(9, 2, 20, 1.2, identity=1, scale=1.0)),
    ],
}

BEV_C = {  # (bfloat16: the kernels on the matrix units)
    "architecture": "Bevovik", "vocab": 300, "width": 128, "norm": {"eps": 2e-5},
    "layers": [
        _with(_gla(2, 64, 96, 12.0, 16), _moe(6, 4, 48, 1.7, identity=2, groups=(2, 1), scale=1.2, shared=(96, 2.0))),
        _with(_rec(192, 6, 3), _moe(8, 8, 32, 4.0, identity=0, shared=(32, 1.0))),
        _with(_latent(4, 32, 32, 64, 64, 96, base=1.0e5, scaling=(8.0, 96, 16.0, 2.0)), _moe(3, 2, 64, 0.9, identity=1, groups=(2, 1))),
        _with(_gla(3, 32, 32, 1.0, 8), _moe(4, 1, 128, 2.5, identity=2, groups=(3, 2), scale=2.0)),
        _with(_rec(64, 2, 4), None),
    ],
}

CONFIGS = {"A": BEV_A, "B": BEV_B, "C": BEV_C}
SEEDS = {"A": 7, "B": 19, "C": 33}
PAGE_SIZES = {"A": 16, "B": 4, "C": 32}


def settle_routes(model_dir, classes: int = 4, size: float = 4.0) -> None:
    """Rewrites a model folder so that no router's choice is a close call in bfloat16: the stream's first
    `classes` elements name a class of the token (the embedding holds `size` at token % classes, no
    layer's output reaches them), and routers read those elements alone.  Tokens of different classes take
    different experts, in every layer others."""
    import torch
    from safetensors.torch import load_file, save_file

    path = Path(model_dir) / "model.safetensors"
    w = load_file(str(path))
    ids = torch.arange(w["embed"].shape[0])
    w["embed"][:, :classes] = 0.0
    w["embed"][ids, ids % classes] = size
    for name, t in w.items():
        if name.endswith((".norm1", ".norm2")):
            t[:classes] = 0.0
        elif name.endswith(".router"):
            gen = torch.Generator().manual_seed(sum(map(ord, name)))
            t.zero_()
            t[:, :classes] = (torch.randn(t.shape[0], classes, generator=gen) * 2.0 / size).to(t.dtype)
    save_file(w, str(path))


def make_model_dir(name: str, root=None, dtype: str = "float32", mode: str = "unit") -> Path:
    """Writes the tiny model `name` with seeded random weights (stored in `dtype`) into
    `root` (or a fresh temporary folder) and returns the folder; bfloat16 ones with settled routes."""
    from shrike_amd.weights import write_model_folder

    if root is None:
        root = tempfile.mkdtemp(prefix="shrike_tiny_")
    path = Path(root) / f"bevovik_{name}_{dtype}_{mode}"
    if not (path / "model.safetensors").is_file():
        write_model_folder(dict(CONFIGS[name]), path, seed=SEEDS[name], dtype=dtype, mode=mode)
        if dtype == "bfloat16":
            settle_routes(path)
    return path
