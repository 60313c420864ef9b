"""Lufivik as a description of parts.

A decoder with layer norms on both sides of every sublayer (``sandwich`` blocks): x += ls * norm_out(sigmoid(W h + b) *
sublayer(norm_in(x))), the gate and the layer scale value by value, the mixer reading its input through a short
causal convolution.  The embedding adds a row per pair of neighbouring tokens and is normed.  The mixers are
``latent_attention`` with a rotated key part and a sliding window, the feed-forwards ``routed_experts`` with a softmax
router whose chosen scores weight the experts' outputs as they are, and a clamped gate, or none.  A stretch of layers
may run several times with the same weights; every pass has caches and kept inputs of its own, which is what
run-order entries give.

Tensor names: ``embed``, ``bigram``, ``embed.norm``, ``final.norm`` (biases ``.b``), ``head`` and per layer ``l<i>.``:
``norm1``, ``norm1b``, ``norm2``, ``norm2b``, ``ls1``, ``ls2``, ``rg1``, ``rg2``, ``canon1``, ``mix.*``, ``mlp.*``.
"""
from __future__ import annotations

from ..config.lufivik import ClampedExpertsConfig, LufivikConfig, RotatedLatentAttentionConfig
from ..parts import PartSpec
from ..registry import register_architecture
from .decoder import LayerSpec, ModelSpec, RunEntry

GATE_ALPHA = 1.702            # an expert's gate: g sigmoid(1.702 g) (u + 1)
UP_SHIFT = 1.0


def _mixer(cfg: LufivikConfig, m: RotatedLatentAttentionConfig, p: str):
    spec = PartSpec("latent_attention", dict(
        hidden_size=cfg.width, n_heads=m.heads, head_dim=m.dim, value_dim=m.vdim, q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale,
        eps=cfg.eps, window=m.window, rot_dim=m.rot_dim,
        position=PartSpec("rope_neox", dict(head_dim=m.rot_dim, theta=m.rot_base, rotated_dims=m.rot_dims))))
    names = {"dq.weight": "dq", "dq_norm.weight": "dq.norm", "uq.weight": "uq", "dkv.weight": "dkv",
             "dkv_norm.weight": "dkv.norm", "uk.weight": "uk", "uv.weight": "uv", "g.weight": "g", "o.weight": "o"}
    return spec, {"mixer." + k: p + "mix." + v for k, v in names.items()}


def _feed_forward(cfg: LufivikConfig, f: ClampedExpertsConfig, p: str):
    spec = PartSpec("routed_experts", dict(hidden_size=cfg.width, n_experts=f.experts, top=f.top, expert_size=f.ff, scoring="softmax",
                                           renormalise=False, weight_on="output", gate_limit=f.limit, gate_alpha=GATE_ALPHA,
                                           up_shift=UP_SHIFT))
    names = {"router.weight": "router"}
    for e in range(f.experts):
        names.update({f"e{e}.{k}.weight": f"e{e}.{k}" for k in ("gate", "up", "down")})
    return spec, {"ffn." + k: p + "mlp." + v for k, v in names.items()}


def _norm_names(local: str, file: str) -> dict:
    return {local + ".weight": file, local + ".bias": file + ".b"}


def lufivik_spec(cfg: LufivikConfig) -> ModelSpec:
    norm = PartSpec("layernorm", dict(hidden_size=cfg.width, eps=cfg.eps))
    layers, unread = [], []
    for l, layer in enumerate(cfg.layers):
        p = f"l{l}."
        mixer, names = _mixer(cfg, layer.mixer, p)
        ffn = None
        subs = [("mixer", "1")]
        if layer.mlp is not None:
            ffn, ffn_names = _feed_forward(cfg, layer.mlp, p)
            names.update(ffn_names)
            subs.append(("ffn", "2"))
        else:                              # (a file may still hold the second sublayer's norms, gate and scale: nothing reads them)
            unread += [f"{p}norm2", f"{p}norm2.b", f"{p}norm2b", f"{p}norm2b.b", f"{p}ls2", f"{p}rg2", f"{p}rg2.b"]
        for sub, i in subs:
            names.update(_norm_names(f"{sub}_norm", f"{p}norm{i}"))
            names.update(_norm_names(f"{sub}_out_norm", f"{p}norm{i}b"))
            names.update({f"{sub}_gate.weight": f"{p}rg{i}", f"{sub}_gate.bias": f"{p}rg{i}.b", f"{sub}_scale": f"{p}ls{i}"})
        names["conv.weight"] = p + "canon1"
        layers.append(LayerSpec(PartSpec("sandwich", dict(mixer=mixer, feed_forward=ffn, norm=norm, hidden_size=cfg.width, gated=True,
                                                          layer_scale=True, conv_taps=cfg.taps)), names))
    order = list(range(len(layers)))
    if cfg.loop is not None:
        lp = cfg.loop
        order = order[:lp.start] + order[lp.start:lp.stop] * lp.times + order[lp.stop:]
    names = {"embedding.weight": "embed", **_norm_names("embedding.norm", "embed.norm"), **_norm_names("final_norm", "final.norm"),
             "head.weight": "head"}
    sizes = dict(vocab_size=cfg.vocab_size, hidden_size=cfg.width, norm=norm)
    if cfg.bigram is not None:
        b = cfg.bigram
        embedding = PartSpec("bigram_token_embedding", dict(sizes, buckets=b.buckets, mul_prev=b.mul_prev, mul_cur=b.mul_cur))
        names["embedding.pairs"] = "bigram"
    else:
        embedding = PartSpec("normed_token_embedding", sizes)
    return ModelSpec(
        architecture=cfg.architecture,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab_size,
        max_position=cfg.max_position_embeddings,
        layers=layers,
        run_order=[RunEntry(l) for l in order],
        final_norm=norm,
        names=names,
        tied_head=False,
        eos_token_id=cfg.eos_token_id,
        eos_token_ids=(cfg.eos_token_id,) if cfg.eos_token_id is not None else (),
        embedding=embedding,
        ignored_tensors=tuple(unread),
    )


register_architecture("Lufivik", LufivikConfig, lufivik_spec)
