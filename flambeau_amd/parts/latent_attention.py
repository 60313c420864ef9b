"""Attention whose keys and values are both made from one cached latent per token.

With h the mixer's input: the queries pass through a normed latent, c_q = Norm(W_dq h), q = W_uq c_q;
the token's cached row is c = Norm(W_dkv h); head a has k = W_uk,a c and v = W_uv,a c, the score
(q_a . k_j) * scale over the keys j <= i (with a window: the newest of them), an ordinary softmax, and its output is
multiplied by sigmoid((W_g h)_a) before the output projection.

Positions, if any, live apart from the latent: W_dkv h has ``rot_dim`` more rows, one key part per token that all
heads share and that is not normed; every head of q has as many more values; both are rotated, and their product
joins the score.  The token's cached row is then (c, rotated part), of which only c is summed.

Options: no gate; a sink, a learned score per head that joins the softmax's denominator once (not scaled, with no key and
no value).

Only that row is cached (``PagedRowSpec``).  Since k and v are linear in c, the key expansion is applied to
the query instead (qa = W_uk,a^T q_a, then qa . c_j = q_a . k_j) and the value expansion to the
weighted sum of the rows (W_uv,a sum_j p_j c_j): no key or value is ever made for a cached token,
and the same kernels serve whole prompts, portions and single tokens.  This step's rows are stored
before attention runs; the query's rotated part is written behind the folded query by the kernel that folds.
The three projections of h (dq, dkv, g) are one joined product; scores, softmax, the weighted sum and both small products per head are 32-bit.
"""
from __future__ import annotations

import torch

from ..config.base import ConfigError
from ..kernels import latent_attention as _kernels  # noqa: F401  (registers this mixer's kernel set)
from ..kernels import ops
from .base import MIXERS, POSITION_ENCODINGS, Mixer, PagedRowSpec, PartSpec, Product, TensorSpec


@MIXERS.register("latent_attention")
class LatentAttention(Mixer):
    graph_safe = True
    replayable = True

    def __init__(self, hidden_size: int, n_heads: int, head_dim: int, value_dim: int, q_rank: int, kv_rank: int,
                 scale: float, eps: float, window: int = 0, gated: bool = True, rot_dim: int = 0, position: PartSpec | None = None,
                 sink: bool = False):
        """``rot_dim`` with ``position`` (an encoding with a table of cosines and sines and a ``layout``, split halves or
        neighbours): the size of the rotated key part and of every head's rotated query part."""
        if bool(rot_dim) != (position is not None):
            raise ValueError("latent_attention: a rotated part and its position encoding come together")
        if kv_rank > ops.latent_max_width():
            raise ConfigError(f"latent_attention: 'kv_rank' {kv_rank} is beyond what the kernel takes ({ops.latent_max_width()})")
        self.hidden_size, self.n_heads, self.head_dim, self.value_dim = hidden_size, n_heads, head_dim, value_dim
        self.q_rank, self.kv_rank = q_rank, kv_rank
        self.scale, self.eps, self.window, self.gated = float(scale), float(eps), int(window or 0), bool(gated)
        self.rot_dim = int(rot_dim)
        self.position = POSITION_ENCODINGS.create(position) if position is not None else None
        self.rotated_dims = self.position.rotated_dims if self.position is not None else 0
        layout = getattr(self.position, "layout", None)
        if self.rotated_dims > self.rot_dim or (self.position is not None and layout not in ("half", "interleaved")):
            raise ConfigError(f"latent_attention: {self.rotated_dims} rotated dims of a part of {self.rot_dim}, or a layout that pairs neither halves nor neighbours")
        self.interleaved, self.has_sink = layout == "interleaved", bool(sink)
        # what the cache holds per token: with a rotated part, latent and part in steps of 32 values with zeros between
        self.value_width = -(-kv_rank // 32) * 32 if self.rot_dim else kv_rank
        self.row_width = self.value_width + -(-self.rot_dim // 32) * 32
        if self.value_width > ops.latent_max_width():
            raise ConfigError(f"latent_attention: 'kv_rank' {kv_rank} is beyond what the kernel takes ({ops.latent_max_width()})")

    def cache_spec(self):
        return PagedRowSpec(self.row_width, self.window, self.value_width if self.rot_dim else None)

    def subparts(self):
        return [self.position] if self.position is not None else []

    def signature_group(self):
        return ("latent_attention", self.n_heads, self.window)

    def step_signature(self, batch):
        """Into how many parts the kernels deal the keys: all that this mixer decides from the contexts' lengths."""
        return self.kernels.signature(batch, self.n_heads, self.window)

    @classmethod
    def step_metadata_for(cls, batch, mixers):
        """The work lists the kernels of the mixers' runtime want for the batch."""
        return mixers[0].kernels.metadata(batch, mixers) if mixers else {}

    def tensors(self):
        W, H, D, Dv, Rq, R = self.hidden_size, self.n_heads, self.head_dim, self.value_dim, self.q_rank, self.kv_rank
        t = {"dq.weight": TensorSpec((Rq, W)), "dq_norm.weight": TensorSpec((Rq,), "vector32"),
             "uq.weight": TensorSpec((H * (D + self.rot_dim), Rq)),
             "dkv.weight": TensorSpec((R + self.rot_dim, W)), "dkv_norm.weight": TensorSpec((R,), "vector32"),
             "uk.weight": TensorSpec((H * D, R)), "uv.weight": TensorSpec((H * Dv, R)),
             "o.weight": TensorSpec((W, H * Dv))}
        if self.gated:
            t["g.weight"] = TensorSpec((H, W))
        if self.has_sink:
            t["sink"] = TensorSpec((H,), "vector32", init="normal")
        return t

    def bind(self, weights, rt):
        self.rt = rt
        joined = [weights["dq.weight"], weights["dkv.weight"]] + ([weights["g.weight"]] if self.gated else [])
        self.w_low = rt.prepare_weight(torch.cat(joined, dim=0).contiguous())
        self.dq_norm, self.dkv_norm = weights["dq_norm.weight"], weights["dkv_norm.weight"]
        self.w_uq = rt.prepare_weight(weights["uq.weight"])
        self.kernels = rt.kernels("latent_attention")
        self.expansions = self.kernels.prepare(weights["uk.weight"], weights["uv.weight"], self.n_heads)
        self.w_o = rt.prepare_weight(weights["o.weight"])
        self.sink = weights.get("sink")
        if self.position is not None:
            self.position.bind({}, rt)

    def forward(self, x, step, cache):
        rt, n = self.rt, x.shape[0]
        H, D, Dv, Rq, R, Dr = self.n_heads, self.head_dim, self.value_dim, self.q_rank, self.kv_rank, self.rot_dim
        angles = self.position.rotary_table(rt, step) if self.rotated_dims else None
        table = step.block_tables[cache.group]
        low = rt.buffer("la_low", n, self.w_low.rows, torch.float32)
        rt.gemm(x, self.w_low, low)
        cq = rt.buffer("la_cq", n, Rq)
        ops.latent_prepare(low, Rq, self.dq_norm, cq, Rq, R, self.dkv_norm, self.eps, cache.kv, step.positions, step.tok_seq, table,
                           rot_dim=Dr, rotated_dims=self.rotated_dims, angles=angles, write_cache=cache.writes,
                           interleaved=self.interleaved)
        q = rt.buffer("la_q", n, H * (D + Dr), torch.float32)
        rt.gemm(cq, self.w_uq, q)
        out = rt.buffer("la_out", n, H * Dv)
        self.kernels.attend(q, self.expansions, cache.kv, step, table, self.scale, self.window,
                            low if self.gated else None, Rq + R + Dr, out,
                            rotated=ops.RotatedPart(Dr, self.rotated_dims, angles, self.value_width, self.interleaved) if Dr else None, sink=self.sink)
        return Product(out, self.w_o)
