"""Fipitar as a description of parts.

A decoder with layer norms behind its sublayers only (``outnorm`` blocks; the sublayers read the stream itself), a
feed-forward with a clamped gate (``clamped_mlp``) or none, and mixers as config.json lists them layer by layer:

* ``gla``: ``gated_linear_attention``;
* ``latent_attention``: the mixer of that name with a rotated part whose neighbouring dims are paired, a stretched ladder of
  frequencies, and a learned sink per head;
* ``parallel``: ``side_by_side`` of a ``normed_gqa_attention`` (heads normed ahead of a split-half rotation, capped scores, one
  added to the denominator, a gate per head) and a ``state_space`` recurrence, each with its factor.

Tensor names: ``embed``, ``final.norm`` (bias ``.b``), ``head`` and per layer ``l<i>.``: ``norm1``, ``norm2``, ``mix.*``, ``mlp.*``.
"""
from __future__ import annotations

from ..config.fipitar import FipitarConfig, GatedLinearConfig, GroupedAttentionConfig, LatentConfig, PairConfig, StateSpaceConfig
from ..parts import PartSpec
from ..registry import register_architecture
from .decoder import LayerSpec, ModelSpec, RunEntry

GATE_ALPHA = 1.702            # the feed-forward's gate: g sigmoid(1.702 g) (u + 1)
UP_SHIFT = 1.0


def _position(rot, dim: int, layout: str) -> PartSpec:
    if rot is None:
        return PartSpec("none", {})
    params = dict(head_dim=dim, theta=rot.base, rotated_dims=rot.dims)
    if rot.scaling is not None:
        sc = rot.scaling
        return PartSpec("rope_blended", dict(params, factor=sc.factor, original=sc.original, fast=sc.fast, slow=sc.slow, layout=layout))
    return PartSpec("rope_neox" if layout == "half" else "rope_interleaved", params)


def _gla(cfg: FipitarConfig, m: GatedLinearConfig):
    spec = PartSpec("gated_linear_attention", dict(hidden_size=cfg.width, n_heads=m.heads, head_dim=m.dim, value_dim=m.vdim,
                                                   decay_rank=m.decay_rank, tau=m.tau, eps=cfg.eps))
    return spec, {"q.weight": "q", "k.weight": "k", "v.weight": "v", "g.weight": "g", "a1.weight": "a1", "a2.weight": "a2",
                  "a2.bias": "a2.b", "norm.weight": "norm", "o.weight": "o"}


def _latent(cfg: FipitarConfig, m: LatentConfig):
    spec = PartSpec("latent_attention", dict(
        hidden_size=cfg.width, n_heads=m.heads, head_dim=m.dim, value_dim=m.vdim, q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale,
        eps=cfg.eps, gated=False, rot_dim=m.rot_dim, position=_position(m.rot, m.rot_dim, "interleaved"), sink=True))
    return spec, {"dq.weight": "dq", "dq_norm.weight": "dq.norm", "uq.weight": "uq", "dkv.weight": "dkv", "dkv_norm.weight": "dkv.norm",
                  "uk.weight": "uk", "uv.weight": "uv", "sink": "sink", "o.weight": "o"}


def _grouped(cfg: FipitarConfig, m: GroupedAttentionConfig):
    spec = PartSpec("normed_gqa_attention", dict(
        hidden_size=cfg.width, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim, scale=m.scale,
        position=_position(m.rot, m.dim, "half"), qk_norm="head_gain_first", eps=cfg.eps, softcap=m.softcap, gate="sigmoid", gate_per="head",
        sink=0.0))
    return spec, {"q.weight": "q", "k.weight": "k", "v.weight": "v", "q_norm.weight": "q.norm", "k_norm.weight": "k.norm", "g.weight": "g",
                  "o.weight": "o"}


def _state_space(cfg: FipitarConfig, m: StateSpaceConfig):
    spec = PartSpec("state_space", dict(hidden_size=cfg.width, n_heads=m.heads, value_dim=m.vdim, state_dim=m.state, n_groups=m.groups,
                                        conv_taps=m.conv, norm_parts=m.norm_groups, eps=cfg.eps))
    return spec, {"in.weight": "in", "conv.weight": "conv", "conv.bias": "conv.b", "dt_bias": "dt_bias", "A_log": "A_log", "D": "D",
                  "norm.weight": "norm", "o.weight": "o"}


def _pair(cfg: FipitarConfig, m: PairConfig):
    (left, left_names), (right, right_names) = _grouped(cfg, m.left), _state_space(cfg, m.right)
    spec = PartSpec("side_by_side", dict(hidden_size=cfg.width, left=left, right=right, factors=(m.left_scale, m.right_scale), normed=False))
    names = {"left." + k: "left." + v for k, v in left_names.items()}
    names.update({"right." + k: "right." + v for k, v in right_names.items()})
    return spec, names


MIXERS = {GatedLinearConfig: _gla, LatentConfig: _latent, PairConfig: _pair}


def _norm_names(local: str, file: str) -> dict:
    return {local + ".weight": file, local + ".bias": file + ".b"}


def fipitar_spec(cfg: FipitarConfig) -> ModelSpec:
    norm = PartSpec("layernorm", dict(hidden_size=cfg.width, eps=cfg.eps))
    layers, unread = [], []
    for l, layer in enumerate(cfg.layers):
        p = f"l{l}."
        mixer, mixer_names = MIXERS[type(layer.mixer)](cfg, layer.mixer)
        names = {"mixer." + k: p + "mix." + v for k, v in mixer_names.items()}
        names.update(_norm_names("mixer_norm", p + "norm1"))
        ffn = None
        if layer.mlp is not None:
            ffn = PartSpec("clamped_mlp", dict(hidden_size=cfg.width, intermediate_size=layer.mlp.ff, limit=layer.mlp.limit,
                                               alpha=GATE_ALPHA, shift=UP_SHIFT))
            names.update({f"ffn.{k}.weight": f"{p}mlp.{k}" for k in ("gate", "up", "down")})
            names.update(_norm_names("ffn_norm", p + "norm2"))
        else:                              # (a file may still hold the second sublayer's norm: nothing reads it)
            unread += [p + "norm2", p + "norm2.b"]
        layers.append(LayerSpec(PartSpec("outnorm", dict(mixer=mixer, feed_forward=ffn, norm=norm)), names))
    return ModelSpec(
        architecture=cfg.architecture,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab_size,
        max_position=cfg.max_position_embeddings,
        layers=layers,
        run_order=[RunEntry(l) for l in range(len(layers))],
        final_norm=norm,
        names={"embedding.weight": "embed", **_norm_names("final_norm", "final.norm"), "head.weight": "head"},
        tied_head=False,
        eos_token_id=cfg.eos_token_id,
        eos_token_ids=(cfg.eos_token_id,) if cfg.eos_token_id is not None else (),
        ignored_tensors=tuple(unread),
    )


register_architecture("Fipitar", FipitarConfig, fipitar_spec)
