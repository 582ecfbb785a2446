"""Bevovik: a decoder whose only norms stand on the sublayers' outputs (each scaled by a learned
vector as it joins the stream), whose mixers are gated linear attention, attention through latents
and Griffin's gated linear recurrence, and whose feed-forward is a routed mixture of experts in
groups, some of which have no matrices.

config.json (every size and every constant that can differ between models):

    architecture   "Bevovik"
    vocab, width
    norm           {eps}                     all norms
    layers[i]      {type, mixer: {...}, mlp: {...} | null}

    type "gla"               mixer {heads, dim, vdim, tau}
        linear attention with a decay per token, head and key channel, sigmoid(W_a2 W_a1 x + b) ** (1 / tau)
        (the tensors' shapes give the rank of that product; a config.json written for random weights
        names it as decay_rank); heads' results normed with one weight of vdim, gated by SiLU.
    type "latent_attention"  mixer {heads, dim, rot_dim, vdim, q_rank, kv_rank, scale,
                                    rot: {base, dims, scaling: {factor, original, fast, slow}}}
        queries and keys/values through normed latents, a rotated key part shared by the heads
        (neighbouring pairs, rates stretched by YaRN), causal.
    type "rglru"             mixer {width, blocks, conv}
        Griffin's recurrent block: a GELU branch times a real-gated linear recurrent unit behind a short
        causal convolution; its gates' matrices are block-diagonal.

    mlp {kind: "moe", expert: {ff, limit}, router: {experts, top, identity, scale, groups: {count, keep}},
         shared: {ff, limit} | absent}
        experts: g = min(W_gate x, limit), u = clamp(W_up x, +-limit), W_down (g sigmoid(1.702 g) (u + 1));
        scores are the softmax of W_router x over the experts and, behind them, `identity` outputs that
        stand for x itself; `top` are chosen by score + correction among the `keep` best of `count` groups
        of neighbours; their weights are their scores over the sum, times scale; the shared expert runs
        for every token.

Tensors: embed, head, final.norm, and per layer l<i>.norm1, norm2, ls1, ls2, l<i>.mix.* (by mixer),
l<i>.mlp.{e<k>.{gate, up, down}, router, correction, shared.{gate, up, down}}.
"""

from __future__ import annotations

from dataclasses import dataclass

from ..config.engine_config import canonical_dtype
from ..config.registry import ConfigError, register_architecture
from ..config.specs import (
    GatedLinearAttentionSpec,
    GatedRecurrenceSpec,
    LatentAttentionSpec,
    LinearHeadSpec,
    MoESpec,
    ModelSpec,
    OutputNormBlockSpec,
    RMSNormSpec,
    TokenEmbeddingSpec,
)

ARCHITECTURE = "Bevovik"
EXPERT_ACTIVATION = "quick_gelu"  # g * sigmoid(1.702 g)
EXPERT_UP_SHIFT = 1.0  # the gate multiplies (u + 1)
RECURRENCE_POWER = 8.0  # log a = -8 r softplus(lam)


def _get(raw, key: str, kind, where: str = "config.json"):
    if not isinstance(raw, dict) or key not in raw or raw[key] is None:
        raise ConfigError(f"{where} lacks the key {key!r}, which {ARCHITECTURE} needs")
    value = raw[key]
    if kind is int:
        if isinstance(value, bool) or not isinstance(value, int):
            raise ConfigError(f"{where}: {key} must be an integer, got {value!r}")
    elif kind is float:
        if isinstance(value, bool) or not isinstance(value, (int, float)):
            raise ConfigError(f"{where}: {key} must be a number, got {value!r}")
        value = float(value)
    elif kind is dict and not isinstance(value, dict):
        raise ConfigError(f"{where}: {key} must be an object, got {value!r}")
    return value


def _opt(raw: dict, key: str, kind, where: str, default):
    return default if raw.get(key) is None else _get(raw, key, kind, where)


def _positive(where: str, **values) -> None:
    for name, value in values.items():
        if not value > 0:
            raise ConfigError(f"{where}: {name} must be positive, got {value}")


@dataclass(frozen=True)
class KeyDecayAttention:
    heads: int
    dim: int
    vdim: int
    tau: float
    decay_rank: int | None = None  # None: as many rows as the file's tensor has

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "KeyDecayAttention":
        dim = _get(raw, "dim", int, where)
        out = cls(heads=_get(raw, "heads", int, where), dim=dim, vdim=_opt(raw, "vdim", int, where, dim),
                  tau=_get(raw, "tau", float, where), decay_rank=_opt(raw, "decay_rank", int, where, None))
        _positive(where, heads=out.heads, dim=out.dim, vdim=out.vdim, tau=out.tau)
        if out.decay_rank is not None:
            _positive(where, decay_rank=out.decay_rank)
        return out

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}
        if self.decay_rank is not None:
            out["decay_rank"] = self.decay_rank
        return out

    def spec(self, eps: float):
        return GatedLinearAttentionSpec(num_heads=self.heads, head_dim=self.dim, value_dim=self.vdim, tau=self.tau, eps=eps,
                                        decay_rank=self.decay_rank)


@dataclass(frozen=True)
class StretchedLatentAttention:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float
    rot_dims: int
    rot_scaling: tuple | None = None  # (factor, original, fast, slow)

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "StretchedLatentAttention":
        rot_dim = _get(raw, "rot_dim", int, where)
        rot = raw.get("rot") or {}
        sc = rot.get("scaling") if rot_dim else None
        inside = where + ".rot.scaling"
        out = cls(heads=_get(raw, "heads", int, where), dim=_get(raw, "dim", int, where), rot_dim=rot_dim,
                  vdim=_get(raw, "vdim", int, where), q_rank=_get(raw, "q_rank", int, where),
                  kv_rank=_get(raw, "kv_rank", int, where), scale=_get(raw, "scale", float, where),
                  rot_base=_get(rot, "base", float, where + ".rot") if rot_dim else 1.0,
                  rot_dims=_opt(rot, "dims", int, where + ".rot", rot_dim) if rot_dim else 0,
                  rot_scaling=None if sc is None else tuple(_get(sc, k, float, inside)
                                                            for k in ("factor", "original", "fast", "slow")))
        _positive(where, heads=out.heads, dim=out.dim, vdim=out.vdim, q_rank=out.q_rank, kv_rank=out.kv_rank,
                  rot_base=out.rot_base)
        if out.rot_dim < 0 or out.rot_dim % 2 or out.rot_dims < 0 or out.rot_dims % 2 or out.rot_dims > out.rot_dim:
            raise ConfigError(f"{where}: rot_dim ({out.rot_dim}) and rot.dims ({out.rot_dims}) must be even, and "
                              "rot.dims at most rot_dim")
        if out.rot_scaling is not None:
            if out.rot_dims != out.rot_dim:
                raise ConfigError(f"{where}: stretched rates need rot.dims ({out.rot_dims}) equal to rot_dim ({out.rot_dim})")
            _positive(inside, **dict(zip(("factor", "original", "fast", "slow"), out.rot_scaling)))
            if out.rot_base == 1.0:
                raise ConfigError(f"{where}: stretched rates need a rot.base other than 1")
        return out

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "q_rank": self.q_rank,
               "kv_rank": self.kv_rank, "scale": self.scale}
        if self.rot_dim:
            out["rot"] = {"base": self.rot_base, "dims": self.rot_dims}
            if self.rot_scaling is not None:
                out["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), self.rot_scaling))
        return out

    def spec(self, eps: float):
        return LatentAttentionSpec(num_heads=self.heads, head_dim=self.dim, rot_dim=self.rot_dim, value_dim=self.vdim,
                                   q_rank=self.q_rank, kv_rank=self.kv_rank, scale=self.scale, eps=eps,
                                   rot_theta=self.rot_base, rotated=self.rot_dims, rot_scaling=self.rot_scaling)


@dataclass(frozen=True)
class Recurrence:
    width: int
    blocks: int
    conv: int

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "Recurrence":
        out = cls(width=_get(raw, "width", int, where), blocks=_get(raw, "blocks", int, where),
                  conv=_get(raw, "conv", int, where))
        _positive(where, width=out.width, blocks=out.blocks, conv=out.conv)
        if out.width % out.blocks:
            raise ConfigError(f"{where}: width {out.width} is not a multiple of {out.blocks} blocks")
        return out

    def to_dict(self) -> dict:
        return {"width": self.width, "blocks": self.blocks, "conv": self.conv}

    def spec(self, eps: float):
        return GatedRecurrenceSpec(recurrent_width=self.width, blocks=self.blocks, conv=self.conv, power=RECURRENCE_POWER)


MIXERS = {"gla": KeyDecayAttention, "latent_attention": StretchedLatentAttention, "rglru": Recurrence}


@dataclass(frozen=True)
class GroupedMixture:
    experts: int
    top: int
    ff: int
    limit: float
    identity: int = 0
    groups: tuple | None = None  # (count, keep)
    scale: float = 1.0
    shared: tuple | None = None  # (ff, limit)

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "GroupedMixture":
        kind = _get(raw, "kind", str, where)
        if kind != "moe":
            raise ConfigError(f"{where}: unknown feed-forward kind {kind!r} (known: moe)")
        router, expert = _get(raw, "router", dict, where), _get(raw, "expert", dict, where)
        inside, groups, shared = where + ".router", router.get("groups"), raw.get("shared")
        out = cls(experts=_get(router, "experts", int, inside), top=_get(router, "top", int, inside),
                  ff=_get(expert, "ff", int, where + ".expert"), limit=_get(expert, "limit", float, where + ".expert"),
                  identity=_opt(router, "identity", int, inside, 0),
                  groups=None if groups is None else (_get(groups, "count", int, inside + ".groups"),
                                                      _get(groups, "keep", int, inside + ".groups")),
                  scale=_opt(router, "scale", float, inside, 1.0),
                  shared=None if shared is None else (_get(shared, "ff", int, where + ".shared"),
                                                      _get(shared, "limit", float, where + ".shared")))
        _positive(where, experts=out.experts, top=out.top, ff=out.ff, limit=out.limit)
        if out.identity < 0:
            raise ConfigError(f"{inside}: identity must not be negative, got {out.identity}")
        if out.shared is not None:
            _positive(where + ".shared", ff=out.shared[0], limit=out.shared[1])
        outputs = out.experts + out.identity
        count, keep = out.groups or (1, 1)
        if count < 1 or outputs % count or not 1 <= keep <= count:
            raise ConfigError(f"{inside}: {outputs} experts do not form {count} equal groups of which {keep} are kept")
        if out.top > keep * (outputs // count):
            raise ConfigError(f"{inside}: top {out.top} is more than the {keep * (outputs // count)} experts that can be chosen")
        return out

    def to_dict(self) -> dict:
        router = {"experts": self.experts, "top": self.top, "identity": self.identity, "scale": self.scale}
        if self.groups is not None:
            router["groups"] = {"count": self.groups[0], "keep": self.groups[1]}
        out = {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit}, "router": router}
        if self.shared is not None:
            out["shared"] = {"ff": self.shared[0], "limit": self.shared[1]}
        return out

    def spec(self):
        return MoESpec(experts=self.experts, top=self.top, expert_size=self.ff,
                       shared_size=None if self.shared is None else self.shared[0], correction=True,
                       activation=EXPERT_ACTIVATION, limit=self.limit,
                       shared_limit=None if self.shared is None else self.shared[1], up_shift=EXPERT_UP_SHIFT,
                       identity=self.identity, groups=self.groups, router_scale=self.scale)


@dataclass(frozen=True)
class BevovikLayer:
    type: str
    mixer: object
    mlp: GroupedMixture | None

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class BevovikConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: tuple[BevovikLayer, ...]
    torch_dtype: str = "bfloat16"

    def __post_init__(self):
        if self.vocab < 1 or self.width < 1 or not self.layers:
            raise ConfigError("config.json: vocab, width and the number of layers must be positive")
        if not self.norm_eps > 0:
            raise ConfigError(f"config.json: norm.eps must be > 0, got {self.norm_eps}")

    @classmethod
    def from_dict(cls, raw: dict) -> "BevovikConfig":
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: layers must be a non-empty list")
        layers = []
        for i, entry in enumerate(listed):
            where = f"config.json layers[{i}]"
            kind = _get(entry, "type", str, where)
            if kind not in MIXERS:
                raise ConfigError(f"{where}: unknown mixer type {kind!r} (known: {', '.join(MIXERS)})")
            mixer = MIXERS[kind].from_dict(_get(entry, "mixer", dict, where), where + ".mixer")
            mlp = entry.get("mlp")
            layers.append(BevovikLayer(kind, mixer, None if mlp is None else GroupedMixture.from_dict(mlp, where + ".mlp")))
        try:
            dtype = canonical_dtype(raw.get("torch_dtype") or "bfloat16")
        except ValueError as e:
            raise ConfigError(f"config.json: {e}") from None
        return cls(vocab=_get(raw, "vocab", int), width=_get(raw, "width", int),
                   norm_eps=_get(_get(raw, "norm", dict), "eps", float, "config.json norm"), layers=tuple(layers),
                   torch_dtype=dtype)

    def to_dict(self) -> dict:
        """A config.json that `from_dict` reads back to the same configuration."""
        return {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "layers": [layer.to_dict() for layer in self.layers], "torch_dtype": self.torch_dtype}


def build_spec(cfg: BevovikConfig) -> ModelSpec:
    norm = RMSNormSpec(eps=cfg.norm_eps, names=(("weight", ""),))
    blocks = [OutputNormBlockSpec(name=f"l{i}", mixer=layer.mixer.spec(cfg.norm_eps),
                                  ffn=None if layer.mlp is None else layer.mlp.spec(), mixer_norm=norm, ffn_norm=norm,
                                  layer_scale=True)
              for i, layer in enumerate(cfg.layers)]
    return ModelSpec(
        architecture=ARCHITECTURE,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        blocks=tuple(blocks),
        final_norm=norm,
        tie_word_embeddings=False,
        embed_name="embed",
        final_norm_name="final.norm",
        head_name="head",
        stored_dtype=cfg.torch_dtype,
        embedding=TokenEmbeddingSpec(cfg.vocab, names=(("weight", ""),)),
        head=LinearHeadSpec(cfg.vocab, names=(("weight", ""),)),
    )


register_architecture(ARCHITECTURE, BevovikConfig, build_spec)
