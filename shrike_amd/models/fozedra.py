"""Fozedra: a pre-norm decoder whose norms are a bounded elementwise map, whose sublayers join the
stream with a common factor, and whose mixers are differential attention behind a short convolution
(with a window that keeps a sequence's first tokens; a layer may read an earlier one's keys and values)
and lightning attention (linear attention with a fixed decay per head).

config.json (every size and every constant that can differ between models):

    architecture   "Fozedra"
    vocab, width
    norm           {eps}                     the RMS norms inside the mixers
    residual_mult                            x <- x + residual_mult * sublayer(map(x)); absent: 1
    layers[i]      {type, mixer: {...}, mlp: {...} | null}

    type "attention"   mixer {heads, kv_heads, dim, vdim, scale, diff, conv, mask: {size, keep_first},
                              rot: {base, dims, scaling: {factor, original, fast, slow}}, kv_from}
        every head two maps (queries and keys of dim each, values of vdim shared); q, k, v with biases and
        a causal convolution of `conv` taps per channel; the first rot.dims elements of each map rotated in
        pairs (i, i + dims / 2), the rates stretched as YaRN does where `scaling` is there; the query at i
        reads keys j <= i with i - j < mask.size or j < mask.keep_first (no mask: all); a1 - lambda a2 of
        the maps' results, normed, times 1 - diff, times sigmoid(W_g h), one number a head.  With kv_from: j
        the layer has no keys and values of its own and reads layer j's.
    type "lightning"   mixer {heads, dim, vdim, decay: [heads]}
        q, k, v through SiLU, S <- decay S + k v^T, o = S^T q; the heads together normed and weighted,
        times sigmoid(W_g h).

    mlp {kind: "dense", ff}                  W_down relu(W_up h)^2

Tensors: embed (also the output matrix), and per map `<name>`, `<name>.b`, `<name>.alpha`: final.norm,
l<i>.norm1, l<i>.norm2; l<i>.mix.{q, k, v}(.b, .conv), l<i>.mix.{lq1, lk1, lq2, lk2, g, o} or
l<i>.mix.{q, k, v, g, o, norm}; l<i>.mlp.{up, down}.
"""

from __future__ import annotations

from dataclasses import dataclass

from ..config.engine_config import canonical_dtype
from ..config.registry import ConfigError, register_architecture
from ..config.specs import (
    BlockSpec,
    DenseFFNSpec,
    DifferentialAttentionSpec,
    DynamicTanhSpec,
    LinearHeadSpec,
    ModelSpec,
    RetentionSpec,
    RotarySpec,
    ScheduleEntry,
    TokenEmbeddingSpec,
)

ARCHITECTURE = "Fozedra"
MIXERS = ("attention", "lightning")
DENSE_ACTIVATION = "relu_squared"


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
    elif kind in (dict, list) and not isinstance(value, kind):
        raise ConfigError(f"{where}: {key} must be {'an object' if kind is dict else 'a list'}, got {value!r}")
    return value


def _optional(raw: dict, key: str, kind, default, where: str):
    return default if raw.get(key) is None else _get(raw, key, kind, where)


def _positive(where: str, **values) -> None:
    for name, value in values.items():
        if not value > 0:
            raise ConfigError(f"{where}: {name} must be positive, got {value}")


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int
    scaling: tuple | None = None  # (factor, original, fast, slow)

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "Rotation":
        scaling = raw.get("scaling")
        if scaling is not None:
            sw = where + ".scaling"
            scaling = tuple(_get(scaling, key, float, sw) for key in ("factor", "original", "fast", "slow"))
            _positive(sw, factor=scaling[0], original=scaling[1], fast=scaling[2], slow=scaling[3])
        out = cls(_get(raw, "base", float, where), _get(raw, "dims", int, where), scaling)
        _positive(where, base=out.base)
        if out.dims < 0 or out.dims % 2:
            raise ConfigError(f"{where}: dims must be even and not negative, got {out.dims}")
        if scaling is not None and out.base == 1.0:
            raise ConfigError(f"{where}: a scaled rotation needs a base other than 1")
        return out

    def to_dict(self) -> dict:
        out = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), self.scaling))
        return out


@dataclass(frozen=True)
class MappedAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float
    conv: int = 0
    window: int | None = None
    keep_first: int = 0
    rot: Rotation | None = None
    kv_from: int | None = None

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "MappedAttention":
        mask, rot = raw.get("mask"), raw.get("rot")
        dim = _get(raw, "dim", int, where)
        out = cls(heads=_get(raw, "heads", int, where), kv_heads=_get(raw, "kv_heads", int, where), dim=dim,
                  vdim=_optional(raw, "vdim", int, dim, where), scale=_get(raw, "scale", float, where),
                  diff=_get(raw, "diff", float, where), conv=_optional(raw, "conv", int, 0, where),
                  window=None if mask is None else _get(mask, "size", int, where + ".mask"),
                  keep_first=0 if mask is None else _optional(mask, "keep_first", int, 0, where + ".mask"),
                  rot=None if rot is None else Rotation.from_dict(rot, where + ".rot"),
                  kv_from=_optional(raw, "kv_from", int, None, where))
        _positive(where, heads=out.heads, kv_heads=out.kv_heads, dim=out.dim, vdim=out.vdim)
        if out.heads % out.kv_heads:
            raise ConfigError(f"{where}: {out.heads} heads are not a multiple of {out.kv_heads} kv_heads")
        if out.window is not None:
            _positive(where + ".mask", size=out.window)
        if out.keep_first < 0 or out.conv < 0:
            raise ConfigError(f"{where}: mask.keep_first and conv must not be negative")
        if out.rot is not None and out.rot.dims > out.dim:
            raise ConfigError(f"{where}: rot.dims {out.rot.dims} is more than dim {out.dim}")
        return out

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
               "diff": self.diff, "conv": self.conv}
        if self.window is not None:
            out["mask"] = {"size": self.window, "keep_first": self.keep_first}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class Lightning:
    heads: int
    dim: int
    vdim: int
    decay: tuple

    @classmethod
    def from_dict(cls, raw: dict, where: str) -> "Lightning":
        decay = _get(raw, "decay", list, where)
        if any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
            raise ConfigError(f"{where}: decay must be a list of numbers, got {decay!r}")
        dim = _get(raw, "dim", int, where)
        out = cls(heads=_get(raw, "heads", int, where), dim=dim, vdim=_optional(raw, "vdim", int, dim, where),
                  decay=tuple(float(d) for d in decay))
        _positive(where, heads=out.heads, dim=out.dim, vdim=out.vdim)
        if len(out.decay) != out.heads:
            raise ConfigError(f"{where}: {len(out.decay)} decays for {out.heads} heads")
        return out

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}


@dataclass(frozen=True)
class FozedraLayer:
    type: str
    mixer: object
    ff: int | None  # width of the feed-forward, None: none

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(),
                "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}


def _ff_from_dict(raw, where: str) -> int | None:
    if raw is None:
        return None
    kind = _get(raw, "kind", str, where)
    if kind != "dense":
        raise ConfigError(f"{where}: unknown feed-forward kind {kind!r} (known: dense)")
    ff = _get(raw, "ff", int, where)
    _positive(where, ff=ff)
    return ff


@dataclass(frozen=True)
class FozedraConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: tuple[FozedraLayer, ...]
    residual_mult: float = 1.0
    torch_dtype: str = "bfloat16"

    def __post_init__(self):
        if self.vocab < 1 or self.width < 1 or not self.layers:
            raise ConfigError("config.json: vocab, width and the number of layers must be positive")
        if not self.norm_eps > 0:
            raise ConfigError(f"config.json: norm.eps must be > 0, got {self.norm_eps}")
        for i, layer in enumerate(self.layers):
            source = getattr(layer.mixer, "kv_from", None)
            if source is None:
                continue
            where = f"config.json layers[{i}].mixer"
            if not 0 <= source < i:
                raise ConfigError(f"{where}: kv_from {source} must name an earlier layer")
            other = self.layers[source]
            if other.type != "attention" or other.mixer.kv_from is not None:
                raise ConfigError(f"{where}: kv_from {source} names a layer without keys and values of its own")
            a, b = layer.mixer, other.mixer
            if (a.kv_heads, a.dim, a.vdim) != (b.kv_heads, b.dim, b.vdim):
                raise ConfigError(f"{where}: layer {source}'s keys and values have other sizes than this layer's")

    @classmethod
    def from_dict(cls, raw: dict) -> "FozedraConfig":
        layers = []
        for i, entry in enumerate(_get(raw, "layers", list)):
            where = f"config.json layers[{i}]"
            kind = _get(entry, "type", str, where)
            mixer = _get(entry, "mixer", dict, where)
            if kind == "attention":
                mixer = MappedAttention.from_dict(mixer, where + ".mixer")
            elif kind == "lightning":
                mixer = Lightning.from_dict(mixer, where + ".mixer")
            else:
                raise ConfigError(f"{where}: unknown mixer type {kind!r} (known: {', '.join(MIXERS)})")
            layers.append(FozedraLayer(kind, mixer, _ff_from_dict(entry.get("mlp"), where + ".mlp")))
        dtype = raw.get("torch_dtype") or "bfloat16"
        try:
            dtype = canonical_dtype(dtype)
        except ValueError as e:
            raise ConfigError(f"config.json: {e}") from None
        return cls(vocab=_get(raw, "vocab", int), width=_get(raw, "width", int),
                   norm_eps=_get(_get(raw, "norm", dict), "eps", float, "config.json norm"), layers=tuple(layers),
                   residual_mult=_optional(raw, "residual_mult", float, 1.0, "config.json"), torch_dtype=dtype)

    def to_dict(self) -> dict:
        """A config.json that `from_dict` reads back to the same configuration."""
        return {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "residual_mult": self.residual_mult, "layers": [layer.to_dict() for layer in self.layers],
                "torch_dtype": self.torch_dtype}


_ATTENTION_NAMES = tuple((role + sub, role + dotted) for role in ("q", "k", "v")
                         for sub, dotted in (("", ""), ("_bias", ".b"), ("_conv", ".conv")))


def cache_reach(cfg: FozedraConfig) -> dict:
    """For every attention layer with keys and values of its own, (window, keep_first) of what its cache
    has to keep: its own mask's, or more where a layer that reads its cache looks further (window None:
    everything)."""
    kept: dict = {}
    for i, layer in enumerate(cfg.layers):
        if layer.type != "attention":
            continue
        m = layer.mixer
        owner = i if m.kv_from is None else m.kv_from
        window, keep = kept.get(owner, (m.window, m.keep_first))
        kept[owner] = (None if window is None or m.window is None else max(window, m.window), max(keep, m.keep_first))
    return kept


def mixer_spec(layer: FozedraLayer, eps: float, reach: tuple | None = None):
    m = layer.mixer
    if layer.type == "lightning":
        return RetentionSpec(num_heads=m.heads, head_dim=m.dim, value_dim=m.vdim, decay=m.decay, eps=eps, activation="silu",
                             key_scale=1.0, norm_heads=False, norm_weight=True, gate="sigmoid")
    position = None
    if m.rot is not None and m.rot.dims:
        position = RotarySpec(theta=m.rot.base, rotary_dim=m.rot.dims, scaling=m.rot.scaling)
    wider = reach is not None and reach != (m.window, m.keep_first)
    return DifferentialAttentionSpec(
        num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim, scale=m.scale, diff=m.diff, eps=eps,
        conv=m.conv, window=m.window, keep_first=m.keep_first, position=position, shared_kv=m.kv_from is not None,
        cache_window=reach[0] if wider else "own", cache_keep=reach[1] if wider else None, names=_ATTENTION_NAMES)


def build_spec(cfg: FozedraConfig) -> ModelSpec:
    norm = DynamicTanhSpec(names=(("weight", ""), ("bias", "b")))
    kept = cache_reach(cfg)
    blocks, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        ffn = None if layer.ff is None else DenseFFNSpec(layer.ff, DENSE_ACTIVATION, names=(("up", "up"), ("down", "down")))
        blocks.append(BlockSpec(name=f"l{i}", mixer=mixer_spec(layer, cfg.norm_eps, kept.get(i)), ffn=ffn, mixer_norm=norm,
                                ffn_norm=norm, mixer_name="mix", ffn_name="mlp", mixer_norm_name="norm1",
                                ffn_norm_name="norm2", residual_scale=cfg.residual_mult))
        schedule.append(ScheduleEntry(i, cache_of=getattr(layer.mixer, "kv_from", None)))
    return ModelSpec(
        architecture=ARCHITECTURE,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        blocks=tuple(blocks),
        final_norm=norm,
        tie_word_embeddings=True,
        schedule=tuple(schedule),
        embed_name="embed",
        final_norm_name="final.norm",
        head_name="head",
        stored_dtype=cfg.torch_dtype,
        embedding=TokenEmbeddingSpec(cfg.vocab, names=(("weight", ""),)),
        head=LinearHeadSpec(cfg.vocab, names=(("weight", ""),)),
    )


register_architecture(ARCHITECTURE, FozedraConfig, build_spec)
