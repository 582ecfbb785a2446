"""Grouped-query attention behind a short convolution, whose heads may each be the difference of two
attentions over the same values, under a window that keeps a sequence's first tokens."""

from __future__ import annotations

import math
from dataclasses import dataclass

import numpy as np
import torch

from ..kernels import ops
from .attention import (QUERY_TILE, compute_units, decode_splits, decode_streams, heavy_first, kv_cache_spec, portion_runs,
                        portion_splits)
from .base import CompositeSpec, Mixer, ParamSpec, PositionEncoding, StateSpec, build_part, register_mixer

ROW_MULTIPLE = 16  # the stacked projections' rows are padded to this many


@dataclass
class DiffPlan:
    """How one step's attention is launched for a (heads, kv heads, maps, sizes, mask)."""

    mfma: bool = False
    nsplit: int = 1  # key splits of the single-token rows
    streaming: bool = False  # single-token rows: non-temporal loads of keys and values
    small: bool = False  # prompt portions: half as many wavefronts per workgroup
    portion_splits: int = 1
    count: int = 0  # workgroups' runs of queries
    lists: str = ""  # name of the runs' list among the step's extras


class DifferentialAttention(Mixer):
    """One product yields a token's queries, keys, values and the heads' gates (stacked, with the biases);
    `conv_store` convolves, rotates, writes keys and values into their pages and queries and gates into
    tensors of their own; attention forms both maps of a head from one read of the values, and its last
    kernel the difference, its norm and the gate; then the output product.

    Caches: pages of keys (a head's maps side by side in one row) and values, and, with a convolution of
    more than one tap, a state slot with its last inputs.  A layer that reads another run's keys and values
    keeps the inputs of its own queries' convolution all the same."""

    state_graph_safe = True

    def __init__(self, spec, width, name):
        super().__init__(spec, width, name)
        self.position = build_part("position", spec.position, width, name) if spec.position is not None else None

    @property
    def launches_follow_shape(self):
        return self.position is None or self.position.launches_follow_shape

    @property
    def maps(self) -> int:
        return 1 if self.spec.diff is None else 2

    @property
    def kv_heads(self) -> int:
        """Key/value heads whose projections the layer has."""
        return 0 if self.spec.shared_kv else self.spec.num_kv_heads

    def _widths(self) -> dict:
        s = self.spec
        return {"q": s.num_heads * self.maps * s.head_dim, "k": self.kv_heads * self.maps * s.head_dim,
                "v": self.kv_heads * s.value_dim, "g": s.num_heads if s.head_gate else 0}

    @property
    def channels(self) -> int:
        w = self._widths()
        return w["q"] + w["k"] + w["v"]

    def _roles(self):
        return ("q",) if self.spec.shared_kv else ("q", "k", "v")

    def _t(self, role: str) -> str:
        return self.tensor_name(role)

    def params(self):
        s, h, w = self.spec, self.width, self._widths()
        out = []
        for role in self._roles():
            out.append(ParamSpec(self._t(role), (w[role], h)))
            if s.qkv_bias:
                out.append(ParamSpec(self._t(role + "_bias"), (w[role],), init="bias", keep_float32=True))
            if s.conv:
                out.append(ParamSpec(self._t(role + "_conv"), (w[role], s.conv), init="taps", keep_float32=True))
        if s.diff is not None:
            out += [ParamSpec(self._t(r), (s.head_dim,), init="vector", keep_float32=True) for r in ("lq1", "lk1", "lq2", "lk2")]
        if s.head_gate:
            out.append(ParamSpec(self._t("g"), (s.num_heads, h)))
        out.append(ParamSpec(self._t("o"), (h, s.num_heads * s.value_dim)))
        return out

    # ------------------------------------------------------------ caches

    def _conv_state(self) -> tuple:
        floats = max(0, self.spec.conv - 1) * self.channels
        return (("conv", StateSpec((floats,), "float32")),) if floats else ()

    def cache_spec(self):
        s = self.spec
        own = s.cache_window == "own"
        window = s.window if own else s.cache_window
        keep = s.keep_first if own or s.cache_keep is None else s.cache_keep
        pages = kv_cache_spec(s.num_kv_heads, self.maps * s.head_dim, window, None, s.value_dim,
                              keep_first=keep if window is not None else 0)
        return CompositeSpec((("kv", pages),) + self._conv_state())

    def reader_spec(self):
        parts = self._conv_state()
        return CompositeSpec(parts) if parts else None

    def check(self, runtime):
        s = self.spec
        if min(s.num_heads, s.num_kv_heads, s.head_dim, s.value_dim) < 1 or s.num_heads % s.num_kv_heads:
            raise ValueError(f"{self.name}: heads {s.num_heads} must be a positive multiple of kv_heads {s.num_kv_heads}, and "
                             f"the heads' sizes {s.head_dim}, {s.value_dim} positive")
        if s.head_dim > 256 or s.value_dim > 256:
            raise ValueError(f"{self.name}: head sizes {s.head_dim}, {s.value_dim} are more than 256")
        if not 0 <= s.conv <= 33:
            raise ValueError(f"{self.name}: a convolution of {s.conv} taps is outside 0..33")
        if (s.window is not None and s.window < 1) or s.keep_first < 0:
            raise ValueError(f"{self.name}: bad mask, window {s.window} and keep_first {s.keep_first}")
        if s.diff is not None and not s.eps > 0:
            raise ValueError(f"{self.name}: eps must be positive, got {s.eps}")
        if s.cache_window != "own" and s.cache_window is not None and (
                s.window is None or s.cache_window < s.window or (s.cache_keep is not None and s.cache_keep < s.keep_first)):
            raise ValueError(f"{self.name}: the cache keeps fewer keys than the layer's own mask reads")
        if self.position is not None and (type(self.position).rotary_table is PositionEncoding.rotary_table
                                          or getattr(self.position, "adjacent_pairs", False)):
            raise ValueError(f"{self.name}: the cache-write kernel rotates pairs (i, i + rot_dim / 2) only")
        rotated = 0 if s.position is None else int(s.position.rotary_dim)
        if rotated % 2 or not 0 <= rotated <= s.head_dim:
            raise ValueError(f"{self.name}: {rotated} rotated elements must be even and at most head_dim {s.head_dim}")

    def load(self, tensors, runtime):
        s, t, w = self.spec, self._t, self._widths()
        rows = [tensors[t(r)] for r in self._roles()] + ([tensors[t("g")]] if s.head_gate else [])
        used = sum(w.values())
        self.row_width = -(-used // ROW_MULTIPLE) * ROW_MULTIPLE
        if self.row_width > used:
            rows.append(torch.zeros(self.row_width - used, self.width, dtype=rows[0].dtype, device=rows[0].device))
        self.w_in = runtime.weight(torch.cat(rows, dim=0))
        self.b_in = None
        if s.qkv_bias:
            bias = torch.zeros(self.row_width, dtype=torch.float32, device=rows[0].device)
            bias[: self.channels] = torch.cat([tensors[t(r + "_bias")] for r in self._roles()])
            self.b_in = bias
        self.taps = None
        if s.conv:  # [taps, channels]: neighbouring channels are neighbours in memory
            self.taps = torch.cat([tensors[t(r + "_conv")] for r in self._roles()], dim=0).t().contiguous()
        self.lam, self.rest = 0.0, 1.0
        if s.diff is not None:
            lq1, lk1, lq2, lk2 = (tensors[t(r)].to(torch.float64).cpu() for r in ("lq1", "lk1", "lq2", "lk2"))
            self.lam = math.exp(float((lq1 * lk1).sum())) - math.exp(float((lq2 * lk2).sum())) + float(s.diff)
            self.rest = 1.0 - float(s.diff)
        self.w_o = runtime.weight(tensors[t("o")])
        if self.position is not None:
            self.position.load(tensors, runtime)
        self.linear_deferred = runtime.linear_deferred
        self.dtype = runtime.dtype

    # ------------------------------------------------------------ launch plans

    @property
    def plan_key(self):
        s = self.spec
        return ("differential_attention", s.num_heads, s.num_kv_heads, self.maps, s.head_dim, s.value_dim, s.window, s.keep_first)

    @property
    def tiles_key(self):
        return ("conv_store_tiles", ops.conv_store_tile(max(1, self.spec.conv)))

    def prepare(self, shape) -> None:
        """Once per step and geometry: the tiles of the prompt portions that the convolution walks, the key
        splits of single tokens, the runs of queries of prompt portions."""
        portions = shape.q_lens[shape.num_decode:]
        key = self.tiles_key
        if key not in shape.notes:
            shape.notes[key] = ""
            if portions.size:
                seqs, q0 = portion_runs(portions, shape.num_decode, key[1])
                shape.notes[key] = f"conv_store_tiles:{key[1]}"
                shape.add(shape.notes[key], np.concatenate([seqs, q0]))
            shape.launch_key.append((key, int(portions.size)))
        key = self.plan_key
        if key in shape.notes:
            return
        s = self.spec
        h, hkv = s.num_heads, s.num_kv_heads
        plan = shape.notes[key] = DiffPlan()
        plan.mfma = self.dtype == torch.bfloat16 and ops.diff_attention_supports_mfma(
            h, hkv, self.maps, s.head_dim, s.value_dim, shape.page_size)
        if not plan.mfma:
            return  # the general kernel takes every token alike
        reach = 1 << 40 if s.window is None else s.window + s.keep_first  # the most keys that a query reads
        if shape.num_decode:
            # columns of the products: sixteen (map, head) pairs a workgroup
            blocks = -(-(h // hkv) // (16 // self.maps))
            plan.nsplit = decode_splits(shape.num_decode, hkv * blocks, min(shape.max_decode_ctx, reach))
            plan.streaming = decode_streams(shape.num_decode, hkv, (self.maps * s.head_dim + s.value_dim) // 2,
                                            shape.max_decode_ctx, None if s.window is None else reach)
            shape.launch_key.append((key, plan.nsplit, plan.streaming))
        if portions.size == 0:
            return
        tiles = ops.diff_attention_tiles(h, hkv)
        small = ops.diff_attention_tiles(h, hkv, small=True)
        # workgroups of half the size: for two maps wherever they hold the heads (their registers), for one
        # while all of them find room on the chip at once
        if small and (self.maps == 2 or int((-(-portions // (QUERY_TILE * small))).sum()) * hkv <= 2 * compute_units()):
            plan.small, tiles = True, small
        run = QUERY_TILE * tiles
        seqs, q0 = portion_runs(portions, shape.num_decode, run)
        keys = np.minimum(shape.starts[seqs] + q0 + run, reach + run)
        order = heavy_first(keys)
        plan.count = int(seqs.size)
        plan.portion_splits = portion_splits(plan.count * hkv, int(keys.mean()))
        plan.lists = "diff_attention:" + ":".join(str(int(x or 0)) for x in key[1:])
        shape.add(plan.lists, np.concatenate([seqs[order], q0[order]]))
        shape.launch_key.append((key, plan.small, plan.portion_splits, plan.count))

    # ------------------------------------------------------------ forward

    def attend(self, ctx, q, gate, out, tables, cache) -> None:
        s = self.spec
        plan = ctx.notes[self.plan_key]
        sizes = (s.num_heads, s.num_kv_heads, self.maps, s.head_dim, s.value_dim)
        pools = (tables, cache.pools["k"], cache.pools["v"], cache.page_size)
        mask = (s.window, s.keep_first, s.scale, self.lam, self.rest, s.eps)
        if not plan.mfma:
            ops.diff_attention(q, out, *sizes, ctx.positions, ctx.token_seq, *pools, *mask, gate=gate)
            return
        per_row = s.num_heads * self.maps * (s.value_dim + 2)
        if ctx.num_decode:
            partial = ctx.buffer("attn_partial", (ctx.num_decode * plan.nsplit * per_row,), torch.float32)
            ops.diff_attention_decode(q, out, ctx.num_decode, *sizes, ctx.positions, *pools, *mask, gate, partial,
                                      plan.nsplit, plan.streaming)
        if plan.count:
            partial = None
            if plan.portion_splits > 1:
                partial = ctx.buffer("attn_portion_partial",
                                     ((ctx.num_tokens - ctx.num_decode) * plan.portion_splits * per_row,), torch.float32)
            ops.diff_attention_prefill(q, out, ctx.extras[plan.lists], *sizes, ctx.cu_q, ctx.ctx_lens, *pools, *mask, gate,
                                       small=plan.small, partial=partial, nsplit=plan.portion_splits,
                                       first_token=ctx.num_decode)

    def forward(self, ctx, x: torch.Tensor, cache):
        s = self.spec
        n = x.shape[0]
        kv, conv = cache.parts["kv"], cache.parts.get("conv")
        if s.shared_kv == kv.owned:
            raise RuntimeError(f"{self.name}: a layer without keys and values of its own must read another "
                               "run's cache, and only such a layer may")
        state = None if conv is None else conv.state_padded if conv.state_padded is not None else conv.state
        tables = ctx.block_tables[kv.group]
        proj = self.linear_deferred(ctx, "diff_in", x, self.w_in, bias=self.b_in, reader="position")
        q = ctx.buffer("diff_q", (n, s.num_heads * self.maps * s.head_dim), ctx.dtype)
        gate = ctx.buffer("diff_gate", (n, s.num_heads), torch.float32) if s.head_gate else None
        inv_freq, rot_dim = self.position.rotary_table() if self.position is not None else (None, 0)
        tiles = ctx.notes[self.tiles_key]
        ops.conv_store(proj, s.num_heads, self.kv_heads, self.maps, s.head_dim, s.value_dim, s.num_heads if s.head_gate else 0,
                       self.taps, rot_dim, inv_freq, float(getattr(self.position, "magnitude", 1.0)), ctx.positions, ctx.cu_q,
                       ctx.state_slots, tables, state, ctx.extras[tiles] if tiles else None, ctx.num_decode, q, gate,
                       kv.pools["k"], kv.pools["v"], kv.page_size)
        attn = ctx.buffer("attn_out", (n, s.num_heads * s.value_dim), ctx.dtype)
        self.attend(ctx, q, gate, attn, tables, kv)
        return self.linear_deferred(ctx, "attn_proj", attn, self.w_o)


register_mixer("differential_attention", DifferentialAttention)
