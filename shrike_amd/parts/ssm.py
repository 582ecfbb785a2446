"""Mixers whose cache is a state of fixed size per request: the selective scan of Mamba,
retention (linear attention with a fixed decay per head), gated linear attention (a decay per token
and key channel) and the real-gated linear recurrent unit of Griffin."""

from __future__ import annotations

import numpy as np
import torch

from ..kernels import ops
from .attention import portion_runs
from .base import Mixer, ParamSpec, PositionEncoding, StateSpec, build_part, register_mixer


class SelectiveScan(Mixer):
    """in-projection -> [u | z]; u through a short causal convolution and SiLU; W_x u -> [dt | B |
    C] in float32; dt through its own small matrix, a bias and softplus (float32); the scan;
    y * silu(z); out-projection.

    The projections, the convolution and their activations have the compute dtype; step sizes,
    decays, exponentials, B, C and the state are float32.  A request's state slot holds S
    [inner, state] and the convolution's last taps - 1 inputs; both are reached on the device
    through ctx.state_slots, and a sequence whose first row of the step is at position 0
    starts from zeros whatever the slot held."""

    launches_follow_shape = True
    state_graph_safe = True

    def _t(self, role: str) -> str:
        return self.tensor_name(role)

    def params(self):
        s, h = self.spec, self.width
        return [
            ParamSpec(self._t("in"), (2 * s.inner, h)),
            ParamSpec(self._t("conv"), (s.inner, s.conv), init="bias", keep_float32=True),
            ParamSpec(self._t("conv.b"), (s.inner,), init="bias", keep_float32=True),
            ParamSpec(self._t("x"), (s.dt_rank + 2 * s.state, s.inner)),
            ParamSpec(self._t("dt"), (s.inner, s.dt_rank), keep_float32=True),
            ParamSpec(self._t("dt.b"), (s.inner,), init="bias", keep_float32=True),
            ParamSpec(self._t("A_log"), (s.inner, s.state), init="log_rate", keep_float32=True),
            ParamSpec(self._t("D"), (s.inner,), init="norm", keep_float32=True),
            ParamSpec(self._t("o"), (h, s.inner)),
        ]

    def state_floats(self) -> int:
        s = self.spec
        return s.inner * s.state + (s.conv - 1) * s.inner

    def cache_spec(self):
        return StateSpec((self.state_floats(),), "float32")

    def check(self, runtime):
        s = self.spec
        if min(s.inner, s.state, s.dt_rank, s.conv) < 1:
            raise ValueError(f"{self.name}: inner, state, dt_rank and conv must be positive")
        if s.state > 512 or s.conv > 64 or s.dt_rank > 1024:
            raise ValueError(f"{self.name}: at most 512 states a channel, 64 taps and a step-size rank of 1024, got "
                             f"{s.state}, {s.conv} and {s.dt_rank}")
        if ops.selective_scan_state_floats(s.inner, s.state, s.conv) != self.state_floats():
            raise RuntimeError(f"{self.name}: the kernel's state layout and the cache's size disagree")

    def load(self, tensors, runtime):
        self.w_in = runtime.weight(tensors[self._t("in")])
        self.taps = tensors[self._t("conv")].contiguous()
        self.conv_bias = tensors[self._t("conv.b")].contiguous()
        self.w_x = runtime.weight(tensors[self._t("x")])
        self.w_dt = tensors[self._t("dt")].t().contiguous()  # [dt_rank, inner]: channels are neighbours in memory
        self.dt_bias = tensors[self._t("dt.b")].contiguous()
        self.a_log = tensors[self._t("A_log")].contiguous()
        self.skip = tensors[self._t("D")].contiguous()
        self.w_o = runtime.weight(tensors[self._t("o")])
        self.linear = runtime.linear
        self.linear_deferred = runtime.linear_deferred

    def forward(self, ctx, x: torch.Tensor, cache):
        s = self.spec
        n = x.shape[0]
        state = cache.state_padded if cache.state_padded is not None else cache.state
        uz = ctx.buffer("scan_in", (n, 2 * s.inner), ctx.dtype)
        self.linear(x, self.w_in, uz)
        u = ctx.buffer("scan_u", (n, s.inner), ctx.dtype)
        ops.short_conv(uz, self.taps, self.conv_bias, ctx.positions, ctx.token_seq, ctx.cu_q, ctx.state_slots,
                       state, s.state, u, activation="silu")
        low = ctx.buffer("scan_low", (n, s.dt_rank + 2 * s.state), torch.float32)
        self.linear(u, self.w_x, low)
        dt = ctx.buffer("scan_dt", (n, s.inner), torch.float32)
        ops.dt_softplus(low, self.w_dt, self.dt_bias, dt)
        gated = ctx.buffer("scan_gated", (n, s.inner), ctx.dtype)
        ops.selective_scan(dt, u, low, s.dt_rank, s.dt_rank + s.state, uz[:, s.inner:], self.a_log, self.skip,
                           s.state, s.conv, uz, ctx.positions, ctx.cu_q, ctx.state_slots, state, gated, ctx.num_seqs)
        return self.linear_deferred(ctx, "scan_out", gated, self.w_o)


register_mixer("selective_scan", SelectiveScan)


class Retention(Mixer):
    """One product yields queries, keys, values and the output gate of a token, in float32 where
    they enter the recurrence as projected, in the compute dtype where an activation comes
    between (bfloat16: prompt portions then run in chunks on the matrix units); by the spec SiLU is applied to the first three; queries and keys are rotated (the spec's position
    encoding, applied to float32 rows) and the keys scaled; the scan carries S per head in the
    request's state slot (float32); the readout is brought to unit root mean square (per head, or
    the heads together), weighted, gated by SiLU or the sigmoid of the gate projection, and
    projected."""

    launches_follow_shape = True
    state_graph_safe = True

    def __init__(self, spec, width, name):
        super().__init__(spec, width, name)
        self.position = build_part("position", spec.position, width, name) if spec.position is not None else None

    def _t(self, role: str) -> str:
        return self.tensor_name(role)

    def params(self):
        s, h = self.spec, self.width
        qk, v = s.num_heads * s.head_dim, s.num_heads * s.value_dim
        out = [ParamSpec(self._t("q"), (qk, h)), ParamSpec(self._t("k"), (qk, h)), ParamSpec(self._t("v"), (v, h)),
               ParamSpec(self._t("g"), (v, h)), ParamSpec(self._t("o"), (h, v))]
        if s.norm_weight:
            out.append(ParamSpec(self._t("norm"), (v,), init="norm", keep_float32=True))
        return out

    def state_floats(self) -> int:
        s = self.spec
        return s.num_heads * s.value_dim * s.head_dim

    def cache_spec(self):
        return StateSpec((self.state_floats(),), "float32")

    def check(self, runtime):
        s = self.spec
        if min(s.num_heads, s.head_dim, s.value_dim) < 1:
            raise ValueError(f"{self.name}: heads, head_dim and value_dim must be positive")
        if s.head_dim > 1024:
            raise ValueError(f"{self.name}: head_dim {s.head_dim} is more than the 1024 the scan kernel holds")
        if len(s.decay) != s.num_heads:
            raise ValueError(f"{self.name}: {len(s.decay)} decays for {s.num_heads} heads")
        if self.position is not None:
            if type(self.position).rotary_table is PositionEncoding.rotary_table \
                    or getattr(self.position, "adjacent_pairs", False) or getattr(s.position, "scaling", None):
                raise ValueError(f"{self.name}: retention rotates pairs (i, i + rot_dim / 2) only, without scaling")
            if s.activation is not None:
                raise ValueError(f"{self.name}: retention applies an activation to queries and keys only where "
                                 "they are not rotated")
        if s.activation not in (None, "silu") or s.gate not in ("silu", "sigmoid"):
            raise ValueError(f"{self.name}: unknown activation {s.activation!r} or gate {s.gate!r}")
        if s.activation is not None and s.key_scale != 1.0:
            raise ValueError(f"{self.name}: activated keys are not scaled (key_scale 1)")
        if ops.retention_state_floats(s.num_heads, s.head_dim, s.value_dim) != self.state_floats():
            raise RuntimeError(f"{self.name}: the kernel's state layout and the cache's size disagree")

    def load(self, tensors, runtime):
        s = self.spec
        self.w_in = runtime.weight(torch.cat([tensors[self._t(r)] for r in ("q", "k", "v", "g")], dim=0))
        qk, v = s.num_heads * s.head_dim, s.num_heads * s.value_dim
        self.offsets = {"q": 0, "k": qk, "v": 2 * qk, "g": 2 * qk + v}
        self.in_width = 2 * qk + 2 * v
        self.chunked = bool(s.activation == "silu" and self.position is None and qk % 8 == 0 and v % 8 == 0
                            and ops.retention_chunk_supports(s.head_dim, s.value_dim))
        self.decay = torch.tensor([float(d) for d in s.decay], dtype=torch.float32, device=runtime.device)
        self.w_o = runtime.weight(tensors[self._t("o")])
        self.norm_weight = tensors[self._t("norm")].contiguous() if s.norm_weight else None
        self.key_scale = float(s.head_dim) ** -0.5 if s.key_scale is None else float(s.key_scale)
        if self.position is not None:
            self.position.load(tensors, runtime)
        self.linear = runtime.linear
        self.linear_deferred = runtime.linear_deferred

    def forward(self, ctx, x: torch.Tensor, cache):
        s, off = self.spec, self.offsets
        n = x.shape[0]
        # (an activation stands between the projections and the recurrence: both have the compute dtype)
        proj = ctx.buffer("retention_proj", (n, self.in_width), ctx.dtype if s.activation else torch.float32)
        left = s.activation  # what the recurrence's kernels still have to apply
        if s.activation and proj.dtype == torch.bfloat16:
            self.linear(x, self.w_in, proj, activation=(s.activation, off["g"]))  # in the product's epilogue
            left = None
        else:
            self.linear(x, self.w_in, proj)
        inv_freq, rot_dim = self.position.rotary_table() if self.position is not None else (None, 0)
        if rot_dim:
            ops.rotate_half_rows(proj, off["q"], s.num_heads, s.head_dim, rot_dim, inv_freq, ctx.positions, 1.0)
        if rot_dim or self.key_scale != 1.0:
            ops.rotate_half_rows(proj, off["k"], s.num_heads, s.head_dim, rot_dim, inv_freq, ctx.positions, self.key_scale)
        read = ctx.buffer("retention_read", (n, s.num_heads * s.value_dim), torch.float32)
        state = cache.state_padded if cache.state_padded is not None else cache.state
        sizes = (s.num_heads, s.head_dim, s.value_dim)
        in_order = ctx.num_seqs  # sequences whose tokens are walked one by one
        if self.chunked and proj.dtype == torch.bfloat16:
            in_order = ctx.num_decode
            if ctx.num_seqs > in_order:
                ops.retention_chunk(proj, off["q"], off["k"], off["v"], self.decay, in_order, ctx.num_seqs - in_order, *sizes,
                                    ctx.positions, ctx.cu_q, ctx.state_slots, state, read)
        if in_order:
            ops.retention_scan(proj, off["q"], off["k"], off["v"], self.decay, in_order, *sizes, ctx.positions, ctx.cu_q,
                               ctx.state_slots, state, read, activation=left)
        gated = ctx.buffer("retention_gated", (n, s.num_heads * s.value_dim), ctx.dtype)
        heads, size = (s.num_heads, s.value_dim) if s.norm_heads else (1, s.num_heads * s.value_dim)
        ops.headnorm_gate(read, proj[:, off["g"]:], self.norm_weight, s.eps, gated, heads, size, gate_act=s.gate)
        return self.linear_deferred(ctx, "retention_out", gated, self.w_o)


register_mixer("retention", Retention)


class GatedLinearAttention(Mixer):
    """One product yields queries, keys, values and the output gate (in the compute dtype where bfloat16
    prompt portions run in chunks on the matrix units, else in float32); the decays come through a low-rank
    pair of matrices of their own, whose results are never rounded (float32): log alpha = -softplus(-(W_a2 (W_a1
    x) + b)) / tau.  The scan carries S per head in the request's state slot (float32); each head's readout is
    brought to unit root mean square, weighted, gated by SiLU and projected."""

    launches_follow_shape = True
    state_graph_safe = True

    def _t(self, role: str) -> str:
        return self.tensor_name(role)

    def params(self):
        s, h = self.spec, self.width
        qk, v = s.num_heads * s.head_dim, s.num_heads * s.value_dim
        free = s.decay_rank or 16
        return [
            ParamSpec(self._t("q"), (qk, h)), ParamSpec(self._t("k"), (qk, h)), ParamSpec(self._t("v"), (v, h)),
            ParamSpec(self._t("g"), (v, h)), ParamSpec(self._t("o"), (h, v)),
            ParamSpec(self._t("norm"), (s.value_dim,), init="norm", keep_float32=True),
            ParamSpec(self._t("a1"), (s.decay_rank, h), free_size=free),
            ParamSpec(self._t("a2"), (qk, s.decay_rank), keep_float32=True, free_size=free),
            ParamSpec(self._t("a2.b"), (qk,), init="bias", keep_float32=True),
        ]

    def state_floats(self) -> int:
        s = self.spec
        return s.num_heads * s.value_dim * s.head_dim

    def cache_spec(self):
        return StateSpec((self.state_floats(),), "float32")

    def check(self, runtime):
        s = self.spec
        if min(s.num_heads, s.head_dim, s.value_dim) < 1 or not s.tau > 0:
            raise ValueError(f"{self.name}: heads, head_dim, value_dim and tau must be positive")
        if s.head_dim > 1024:
            raise ValueError(f"{self.name}: head_dim {s.head_dim} is more than the 1024 the scan kernel holds")
        if ops.retention_state_floats(s.num_heads, s.head_dim, s.value_dim) != self.state_floats():
            raise RuntimeError(f"{self.name}: the kernel's state layout and the cache's size disagree")

    LISTS = "gla_chunks"  # the chunks of a step's prompt portions, the same for every such layer

    def prepare(self, shape) -> None:
        if not self.chunked or self.LISTS in shape.notes:
            return
        shape.notes[self.LISTS] = True
        portions = shape.q_lens[shape.num_decode:]
        if portions.size:
            seqs, t0 = portion_runs(portions, shape.num_decode, ops.GLA_CHUNK)
            per = -(-portions // ops.GLA_CHUNK)
            shape.add(self.LISTS, np.concatenate([seqs, t0, np.cumsum(per) - per]))

    def load(self, tensors, runtime):
        s = self.spec
        qk, v = s.num_heads * s.head_dim, s.num_heads * s.value_dim
        a1, a2 = tensors[self._t("a1")], tensors[self._t("a2")]
        self.rank = a1.shape[0]
        if a2.shape[1] != self.rank or not 1 <= self.rank <= 1024:
            raise ValueError(f"{self.name}: the decays' two matrices have ranks {self.rank} and {a2.shape[1]} (1 to 1024)")
        self.w_in = runtime.weight(torch.cat([tensors[self._t(r)] for r in ("q", "k", "v", "g")], dim=0))
        self.offsets = {"q": 0, "k": qk, "v": 2 * qk, "g": 2 * qk + v}
        self.in_width = 2 * qk + 2 * v
        self.w_a1 = runtime.weight(a1)
        self.w_a2 = a2.t().contiguous()  # [rank, heads * head_dim]: channels are neighbours in memory
        self.a2_bias = tensors[self._t("a2.b")].contiguous()
        self.norm_weight = tensors[self._t("norm")].repeat(s.num_heads).contiguous()
        self.w_o = runtime.weight(tensors[self._t("o")])
        self.q_scale = float(s.head_dim) ** -0.5
        self.chunked = bool(runtime.dtype == torch.bfloat16 and qk % 8 == 0 and v % 8 == 0
                            and ops.gla_chunk_supports(s.head_dim, s.value_dim))
        self.linear = runtime.linear
        self.linear_deferred = runtime.linear_deferred

    def forward(self, ctx, x: torch.Tensor, cache):
        s, off = self.spec, self.offsets
        n = x.shape[0]
        proj = ctx.buffer("gla_proj", (n, self.in_width), ctx.dtype if self.chunked else torch.float32)
        self.linear(x, self.w_in, proj)
        low = ctx.buffer("gla_low", (n, self.rank), torch.float32)
        self.linear(x, self.w_a1, low)
        log_decay = ctx.buffer("gla_log_decay", (n, s.num_heads * s.head_dim), torch.float32)
        ops.dt_softplus(low, self.w_a2, self.a2_bias, log_decay, sign=-1.0, mult=-1.0 / s.tau)
        read = ctx.buffer("gla_read", (n, s.num_heads * s.value_dim), torch.float32)
        state = cache.state_padded if cache.state_padded is not None else cache.state
        sizes = (s.num_heads, s.head_dim, s.value_dim)
        in_order = ctx.num_seqs  # sequences whose tokens are walked one by one
        if self.chunked and ctx.num_seqs > ctx.num_decode:
            in_order = ctx.num_decode
            lists = ctx.extras[self.LISTS]
            rows = n - in_order  # (the single tokens' rows come first)
            chunks = (lists.shape[0] - (ctx.num_seqs - in_order)) // 2
            scratch = ctx.buffer("gla_scratch", (ops.gla_chunk_scratch_bytes(rows, chunks, *sizes),), torch.uint8)
            ops.gla_chunk(proj, off["q"], off["k"], off["v"], log_decay, self.q_scale, in_order, ctx.num_seqs - in_order,
                          in_order, *sizes, lists, ctx.positions, ctx.cu_q, ctx.state_slots, state, scratch, read)
        if in_order:
            ops.retention_scan(proj, off["q"], off["k"], off["v"], None, in_order, *sizes, ctx.positions, ctx.cu_q,
                               ctx.state_slots, state, read, log_decay=log_decay, q_scale=self.q_scale)
        gated = ctx.buffer("gla_gated", (n, s.num_heads * s.value_dim), ctx.dtype)
        ops.headnorm_gate(read, proj[:, off["g"]:], self.norm_weight, s.eps, gated, s.num_heads, s.value_dim, gate_act="silu")
        return self.linear_deferred(ctx, "gla_out", gated, self.w_o)


register_mixer("gated_linear_attention", GatedLinearAttention)


class GatedRecurrence(Mixer):
    """One product yields both branches; the recurrent one passes a short causal convolution, a
    block-diagonal product gives both gates' pre-activations in float32, and one kernel forms the gates, the
    decays and the recurrence (float32) and multiplies its state by GELU of the other branch; out-projection.

    A request's state slot holds S [recurrent_width] and the convolution's last taps - 1 inputs."""

    launches_follow_shape = True
    state_graph_safe = True

    def _t(self, role: str) -> str:
        return self.tensor_name(role)

    def params(self):
        s, h = self.spec, self.width
        w, part = s.recurrent_width, s.recurrent_width // max(1, s.blocks)
        out = []
        for role in ("y", "x"):
            out += [ParamSpec(self._t(role), (w, h)), ParamSpec(self._t(role + ".b"), (w,), init="bias", keep_float32=True)]
        out += [ParamSpec(self._t("conv"), (w, s.conv), init="taps", keep_float32=True),
                ParamSpec(self._t("conv.b"), (w,), init="bias", keep_float32=True)]
        for role in ("ra", "ri"):
            out += [ParamSpec(self._t(role), (s.blocks, part, part)),
                    ParamSpec(self._t(role + ".b"), (s.blocks, part), init="bias", keep_float32=True)]
        return out + [ParamSpec(self._t("lam"), (w,), init="slow_rate", keep_float32=True), ParamSpec(self._t("o"), (h, w))]

    def state_floats(self) -> int:
        return self.spec.recurrent_width * max(1, self.spec.conv)

    def cache_spec(self):
        return StateSpec((self.state_floats(),), "float32")

    def check(self, runtime):
        s = self.spec
        if min(s.recurrent_width, s.blocks, s.conv) < 1 or s.recurrent_width % s.blocks or not s.power > 0:
            raise ValueError(f"{self.name}: recurrent_width {s.recurrent_width} must be a positive multiple of blocks {s.blocks}, "
                             f"conv ({s.conv}) and power ({s.power}) positive")
        if s.conv > 64:
            raise ValueError(f"{self.name}: at most 64 taps, got {s.conv}")
        if ops.rglru_state_floats(s.recurrent_width, s.conv) != self.state_floats():
            raise RuntimeError(f"{self.name}: the kernel's state layout and the cache's size disagree")

    def load(self, tensors, runtime):
        s = self.spec
        self.w_in = runtime.weight(torch.cat([tensors[self._t("y")], tensors[self._t("x")]], dim=0))
        self.b_in = torch.cat([tensors[self._t("y.b")], tensors[self._t("x.b")]]).contiguous()
        self.taps = tensors[self._t("conv")].contiguous()
        self.conv_bias = tensors[self._t("conv.b")].contiguous()
        # per block [r rows; i rows]: one batched product gives both gates
        self.w_gates = torch.cat([tensors[self._t("ra")], tensors[self._t("ri")]], dim=1).contiguous()
        self.r_bias = tensors[self._t("ra.b")].reshape(-1).contiguous()
        self.i_bias = tensors[self._t("ri.b")].reshape(-1).contiguous()
        lam = tensors[self._t("lam")].to(torch.float64)
        self.rate = (float(s.power) * torch.nn.functional.softplus(lam)).to(torch.float32).contiguous()
        self.w_o = runtime.weight(tensors[self._t("o")])
        self.linear = runtime.linear
        self.linear_deferred = runtime.linear_deferred

    def forward(self, ctx, x: torch.Tensor, cache):
        s = self.spec
        n, w = x.shape[0], s.recurrent_width
        part = w // s.blocks
        state = cache.state_padded if cache.state_padded is not None else cache.state
        yx = ctx.buffer("rglru_in", (n, 2 * w), ctx.dtype)
        self.linear(x, self.w_in, yx, bias=self.b_in)
        raw = yx[:, w:]
        u = ctx.buffer("rglru_u", (n, w), ctx.dtype)
        ops.short_conv(raw, self.taps, self.conv_bias, ctx.positions, ctx.token_seq, ctx.cu_q, ctx.state_slots, state, 1, u)
        gates = ctx.buffer("rglru_gates", (n, 2 * w), torch.float32)
        ops.gemm_batched(u, self.w_gates, gates, s.blocks, part, 2 * part)
        read = ctx.buffer("rglru_read", (n, w), ctx.dtype)
        ops.rglru(gates, s.blocks, self.r_bias, self.i_bias, self.rate, u, yx, raw, s.conv, ctx.positions, ctx.cu_q,
                  ctx.state_slots, state, read, ctx.num_decode, ctx.num_seqs)
        return self.linear_deferred(ctx, "rglru_out", read, self.w_o)


register_mixer("gated_recurrence", GatedRecurrence)
