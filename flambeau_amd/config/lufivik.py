"""LufivikConfig: a decoder whose config.json lists its layers one by one.

Every layer names its mixer (``latent_attention``: attention over a cached latent with a rotated key part and a sliding
window) with the mixer's sizes and constants, and its feed-forward, ``moe`` (routed experts whose gate is clamped) or
none.  ``loop`` says which stretch of layers runs several times with the same weights; ``canon`` gives the taps of the
convolution in front of every mixer, ``embedding`` the table of token pairs.  Every size and constant that the file
gives is read here, with its type, and a missing or ill-typed key is named in the error.
"""
from __future__ import annotations

from dataclasses import dataclass

from .base import ConfigError, KeyReader


@dataclass(frozen=True)
class RotatedLatentAttentionConfig:
    heads: int
    dim: int            # unrotated query/key size per head
    rot_dim: int        # rotated query/key size per head
    vdim: int           # value size per head
    q_rank: int         # size of the queries' latent
    kv_rank: int        # size of the cached latent
    scale: float
    window: int         # 0: every earlier key
    rot_base: float
    rot_dims: int       # how many of the rot_dim values turn


@dataclass(frozen=True)
class ClampedExpertsConfig:
    experts: int
    top: int
    ff: int
    limit: float


@dataclass(frozen=True)
class LufivikLayer:
    type: str                   # "latent_attention"
    mixer: RotatedLatentAttentionConfig
    mlp: ClampedExpertsConfig | None


@dataclass(frozen=True)
class BigramConfig:
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


def _mixer(m: KeyReader) -> RotatedLatentAttentionConfig:
    mask = m.section("mask", default=None)                    # (a mixer without a mask sees every earlier token)
    rot = m.section("rot")
    rot_dim = m.integer("rot_dim", minimum=2)
    cfg = RotatedLatentAttentionConfig(
        heads=m.integer("heads", minimum=1), dim=m.integer("dim", minimum=1), rot_dim=rot_dim, vdim=m.integer("vdim", minimum=1),
        q_rank=m.integer("q_rank", minimum=1), kv_rank=m.integer("kv_rank", minimum=1), scale=m.number("scale", positive=True),
        window=mask.integer("size", minimum=1) if mask is not None else 0, rot_base=rot.number("base", positive=True),
        rot_dims=rot.integer("dims", default=rot_dim, minimum=2))
    if cfg.rot_dims % 2 or cfg.rot_dims > rot_dim:
        raise ConfigError(f"{rot.where}: 'dims' {cfg.rot_dims} must be even and within 'rot_dim' {rot_dim}")
    return cfg


def _mlp(f: KeyReader) -> ClampedExpertsConfig:
    kind = f.string("kind")
    if kind != "moe":
        raise ConfigError(f"{f.where}: unknown feed-forward kind '{kind}' (moe)")
    router, expert = f.section("router"), f.section("expert")
    cfg = ClampedExpertsConfig(experts=router.integer("experts", minimum=1), top=router.integer("top", minimum=1),
                               ff=expert.integer("ff", minimum=1), limit=expert.number("limit", positive=True))
    if cfg.top > cfg.experts:
        raise ConfigError(f"{f.where}: 'top' {cfg.top} of {cfg.experts} experts")
    return cfg


@dataclass(frozen=True)
class LufivikConfig:
    vocab_size: int
    width: int
    eps: float
    taps: int
    bigram: BigramConfig | None
    layers: tuple
    loop: LoopConfig | None
    max_position_embeddings: int
    eos_token_id: int | None = None

    architecture = "Lufivik"
    # the design names no longest sequence; this bounds block tables and default pools
    DEFAULT_MAX_POSITION = 1 << 17

    @classmethod
    def from_dict(cls, raw: dict, where: str = "config.json") -> "LufivikConfig":
        r = KeyReader(raw, where)
        layers = []
        for lr in r.sections("layers"):
            kind = lr.string("type")
            if kind != "latent_attention":
                raise ConfigError(f"{lr.where}: unknown layer type '{kind}' (latent_attention)")
            f = lr.section("mlp", default=None)
            layers.append(LufivikLayer(kind, _mixer(lr.section("mixer")), _mlp(f) if f is not None else None))
        if not layers:
            raise ConfigError(f"{where}: 'layers' is empty")
        lp = r.section("loop", default=None)
        loop = None
        if lp is not None:
            loop = LoopConfig(start=lp.integer("start", minimum=0), stop=lp.integer("stop", minimum=0), times=lp.integer("times", minimum=1))
            if not loop.start < loop.stop <= len(layers):
                raise ConfigError(f"{lp.where}: layers {loop.start}..{loop.stop - 1} are not a stretch of the {len(layers)} layers")
        emb = r.section("embedding", default=None)
        pairs = emb.section("bigram", default=None) if emb is not None else None
        bigram = None
        if pairs is not None:
            bigram = BigramConfig(buckets=pairs.integer("buckets", minimum=1), mul_prev=pairs.integer("mul_prev", minimum=0),
                                  mul_cur=pairs.integer("mul_cur", minimum=0))
        return cls(vocab_size=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                   eps=r.section("norm").number("eps", positive=True), taps=r.section("canon").integer("taps", minimum=1),
                   bigram=bigram, layers=tuple(layers), loop=loop,
                   max_position_embeddings=r.integer("max_position_embeddings", default=cls.DEFAULT_MAX_POSITION, minimum=1),
                   eos_token_id=r.integer("eos_token_id", default=None, minimum=0))
