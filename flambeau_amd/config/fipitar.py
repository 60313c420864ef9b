"""FipitarConfig: a decoder whose config.json lists its layers one by one.

Every layer names its mixer, with the mixer's sizes and constants: ``gla`` (gated linear attention), ``latent_attention``
(attention over a cached latent with a rotated key part and a sink) or ``parallel`` (grouped-query attention and a
state-space recurrence side by side), and its feed-forward, ``dense`` (a clamped gate) or none.  Every size and constant
that the file gives is read here, with its type, and a missing or ill-typed key is named in the error; the rank of the
``gla`` decay's projection is the one size that only a tensor's shape gives.
"""
from __future__ import annotations

from dataclasses import dataclass

from .base import ConfigError, KeyReader


@dataclass(frozen=True)
class RotaryScaling:
    """A ladder of frequencies stretched for contexts beyond ``original`` positions."""
    factor: float
    original: int
    fast: float
    slow: float


@dataclass(frozen=True)
class RotaryConfig:
    base: float
    dims: int
    scaling: RotaryScaling | None = None


@dataclass(frozen=True)
class GatedLinearConfig:
    heads: int
    dim: int
    vdim: int
    tau: float
    decay_rank: int


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int            # unrotated query/key size per head
    rot_dim: int        # rotated query/key size per head
    vdim: int           # value size per head
    q_rank: int
    kv_rank: int
    scale: float
    rot: RotaryConfig


@dataclass(frozen=True)
class GroupedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float | None
    rot: RotaryConfig | None


@dataclass(frozen=True)
class StateSpaceConfig:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int


@dataclass(frozen=True)
class PairConfig:
    left: GroupedAttentionConfig
    right: StateSpaceConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class ClampedMlpConfig:
    ff: int
    limit: float


@dataclass(frozen=True)
class FipitarLayer:
    type: str                   # "gla" | "latent_attention" | "parallel"
    mixer: object
    mlp: ClampedMlpConfig | None


def _rotary(r: KeyReader, width: int, default_dims=None) -> RotaryConfig:
    dims = r.integer("dims", minimum=2) if default_dims is None else r.integer("dims", default=default_dims, minimum=2)
    if dims % 2 or dims > width:
        raise ConfigError(f"{r.where}: 'dims' {dims} must be even and within the part's {width} values")
    s = r.section("scaling", default=None)
    scaling = None
    if s is not None:
        scaling = RotaryScaling(factor=s.number("factor", positive=True), original=s.integer("original", minimum=1),
                                fast=s.number("fast", positive=True), slow=s.number("slow", positive=True))
    return RotaryConfig(base=r.number("base", positive=True), dims=dims, scaling=scaling)


def _gla(m: KeyReader) -> GatedLinearConfig:
    return GatedLinearConfig(heads=m.integer("heads", minimum=1), dim=m.integer("dim", minimum=1), vdim=m.integer("vdim", minimum=1),
                             tau=m.number("tau", positive=True), decay_rank=m.integer("decay_rank", minimum=1))


def _latent(m: KeyReader) -> LatentConfig:
    rot_dim = m.integer("rot_dim", minimum=2)
    return LatentConfig(heads=m.integer("heads", minimum=1), dim=m.integer("dim", minimum=1), rot_dim=rot_dim,
                        vdim=m.integer("vdim", minimum=1), q_rank=m.integer("q_rank", minimum=1), kv_rank=m.integer("kv_rank", minimum=1),
                        scale=m.number("scale", positive=True), rot=_rotary(m.section("rot"), rot_dim, default_dims=rot_dim))


def _pair(m: KeyReader) -> PairConfig:
    l, r = m.section("left"), m.section("right")
    heads, kv_heads, dim = l.integer("heads", minimum=1), l.integer("kv_heads", minimum=1), l.integer("dim", minimum=1)
    if heads % kv_heads:
        raise ConfigError(f"{l.where}: {heads} heads are not a multiple of {kv_heads} key/value heads")
    rot = l.section("rot", default=None)
    left = GroupedAttentionConfig(heads=heads, kv_heads=kv_heads, dim=dim, vdim=l.integer("vdim", minimum=1), scale=l.number("scale", positive=True),
                                  softcap=l.number("softcap", default=None, positive=True), rot=_rotary(rot, dim) if rot is not None else None)
    right = StateSpaceConfig(heads=r.integer("heads", minimum=1), vdim=r.integer("vdim", minimum=1), state=r.integer("state", minimum=1),
                             groups=r.integer("groups", minimum=1), conv=r.integer("conv", minimum=1), norm_groups=r.integer("norm_groups", minimum=1))
    if right.heads % right.groups:
        raise ConfigError(f"{r.where}: {right.heads} heads are not a multiple of {right.groups} groups")
    if (right.heads * right.vdim) % right.norm_groups:
        raise ConfigError(f"{r.where}: {right.heads} x {right.vdim} values do not divide into 'norm_groups' {right.norm_groups}")
    return PairConfig(left, right, left_scale=m.number("left_scale"), right_scale=m.number("right_scale"))


MIXERS = {"gla": _gla, "latent_attention": _latent, "parallel": _pair}


@dataclass(frozen=True)
class FipitarConfig:
    vocab_size: int
    width: int
    eps: float
    layers: tuple
    max_position_embeddings: int
    eos_token_id: int | None = None

    architecture = "Fipitar"
    # the design names no longest sequence; this bounds block tables and default pools
    DEFAULT_MAX_POSITION = 1 << 17

    @staticmethod
    def sizes_from_tensors(raw: dict, shapes: dict) -> dict:
        """``raw`` with the one size that only a tensor's shape gives filled in: the rank of every ``gla`` layer's decay, from
        ``l<i>.mix.a1`` ([rank, width]).  A key that the file has is left alone."""
        layers = raw.get("layers")
        if not isinstance(layers, list):
            return raw
        out = dict(raw, layers=[])
        for i, layer in enumerate(layers):
            shape = shapes.get(f"l{i}.mix.a1")
            if isinstance(layer, dict) and isinstance(layer.get("mixer"), dict) and layer.get("type") == "gla" and shape is not None \
                    and len(shape) == 2 and "decay_rank" not in layer["mixer"]:
                layer = dict(layer, mixer=dict(layer["mixer"], decay_rank=int(shape[0])))
            out["layers"].append(layer)
        return out

    @classmethod
    def from_dict(cls, raw: dict, where: str = "config.json") -> "FipitarConfig":
        r = KeyReader(raw, where)
        layers = []
        for lr in r.sections("layers"):
            kind = lr.string("type")
            if kind not in MIXERS:
                raise ConfigError(f"{lr.where}: unknown layer type '{kind}' ({', '.join(MIXERS)})")
            f = lr.section("mlp", default=None)
            mlp = None
            if f is not None:
                fk = f.string("kind")
                if fk != "dense":
                    raise ConfigError(f"{f.where}: unknown feed-forward kind '{fk}' (dense)")
                mlp = ClampedMlpConfig(ff=f.integer("ff", minimum=1), limit=f.number("limit", positive=True))
            layers.append(FipitarLayer(kind, MIXERS[kind](lr.section("mixer")), mlp))
        if not layers:
            raise ConfigError(f"{where}: 'layers' is empty")
        return cls(vocab_size=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                   eps=r.section("norm").number("eps", positive=True), layers=tuple(layers),
                   max_position_embeddings=r.integer("max_position_embeddings", default=cls.DEFAULT_MAX_POSITION, minimum=1),
                   eos_token_id=r.integer("eos_token_id", default=None, minimum=0))
