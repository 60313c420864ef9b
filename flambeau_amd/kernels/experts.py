"""The kernel set of a feed-forward of routed experts: both products of all experts over the router's tiles, with the
activation between them.

``PlainExperts`` is the 32-bit path (and bfloat16 with the tuned kernels switched off): two plain products and an
activation kernel.  ``TunedExperts`` runs each product on the matrix cores where its sizes allow
(``fl_moe_packed_takes``), with a gate in the first product's epilogue; a weight multiplies a product's result there,
in 32-bit, where the plain product scales and rounds its input."""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import ops
from .library import call, load
from .packing import interleave_gate_up, pack_weight
from .sets import register_kernel_set


@dataclass(frozen=True)
class ExpertActivation:
    """What stands between an expert's two products: ``act(up)`` (``gated`` false), ``silu(gate) * up``, or with ``limit``
    the clamped gate ``g sigmoid(alpha g) (u + shift)``."""
    gated: bool
    kind: str = "silu"
    limit: float | None = None
    alpha: float = 1.0
    shift: float = 0.0

    def apply(self, pre, out):
        if self.limit is not None:
            return ops.clamped_gate(pre, out, self.alpha, self.limit, self.shift)
        return ops.silu_mul(pre, out) if self.gated else ops.activation(pre, out, self.kind)

    @property
    def epilogue(self) -> tuple:
        """``(code, alpha, limit, shift)`` of the first product's epilogue."""
        return (0, 0.0, 0.0, 0.0) if not self.gated else (1, 0.0, 0.0, 0.0) if self.limit is None else (2, self.alpha, self.limit, self.shift)


@dataclass
class ExpertMatrix:
    """One matrix of every expert, ``[E, rows, cols]`` row-major or packed expert by expert; ``gated``: packed gate and up
    rows interleaved in fours."""
    rows: int
    cols: int
    rowmajor: torch.Tensor | None = None
    packed: torch.Tensor | None = None
    gated: bool = False


class PlainExperts:
    def __init__(self, rt):
        self.rt = rt

    def tile_rows(self, n_pairs: int, n_experts: int, *matrices) -> int:
        """Rows of the router's tiles in a step of ``n_pairs`` (token, expert) pairs for products with ``matrices``."""
        return ops.moe_tile_rows()

    def prepare(self, matrices, gates=None) -> ExpertMatrix:
        """``matrices`` (and ``gates`` beside them): one ``[rows, cols]`` tensor per expert."""
        both = [torch.cat([g, m], dim=0) for g, m in zip(gates, matrices)] if gates is not None else matrices
        w = torch.stack(list(both)).contiguous()
        return ExpertMatrix(w.shape[1], w.shape[2], rowmajor=w)

    def product(self, x, w: ExpertMatrix, out, tiles, tile_rows, src_row=None, src_scale=None):
        return ops.moe_gemm(x, w.rowmajor, out, tiles, src_row, src_scale)

    def first(self, x, w: ExpertMatrix, activation: ExpertActivation, act, tiles, tile_rows, most, src_row, src_scale):
        """``act[p] = activation((src_scale[p] *) x[src_row[p]] @ first matrices of p's expert)``."""
        pre = self.rt.buffer("moe_gate_up", act.shape[0], w.rows, torch.float32, max_rows=most)
        self.product(x, w, pre, tiles, tile_rows, src_row, src_scale)
        activation.apply(pre, act)
        return act


LARGE_TILE = 128
LARGE_TILE_MIN_ROWS = 48       # rows per expert from which on tiles of 128 rows cost less than tiles of 64


class TunedExperts(PlainExperts):
    def prepare(self, matrices, gates=None):
        m = matrices[0]
        N, K = (2 if gates is not None else 1) * m.shape[0], m.shape[1]
        if m.dtype != torch.bfloat16 or not load().fl_moe_packed_takes(N, K) or (gates is not None and m.shape[0] % 8):
            return super().prepare(matrices, gates)
        rows = (interleave_gate_up(g, u) for g, u in zip(gates, matrices)) if gates is not None else matrices
        return ExpertMatrix(N, K, packed=torch.cat([pack_weight(r) for r in rows]), gated=gates is not None)

    def tile_rows(self, n_pairs, n_experts, *matrices):
        large = n_pairs >= LARGE_TILE_MIN_ROWS * n_experts and all(m.packed is not None for m in matrices)      # (a plain product takes tiles of 64 only)
        return LARGE_TILE if large else ops.moe_tile_rows()

    def product(self, x, w, out, tiles, tile_rows, src_row=None, src_scale=None, epilogue=(0, 0.0, 0.0, 0.0)):
        if w.packed is None:
            return super().product(x, w, out, tiles, tile_rows, src_row, src_scale)
        P = out.shape[0]
        dtype, cols = (torch.bfloat16, w.rows // 2) if epilogue[0] else (torch.float32, w.rows)
        call("fl_moe_packed", ops._check(x, "moe_packed.x", torch.bfloat16, (None, w.cols)),
             ops._check(src_row, "moe_packed.src_row", torch.int32, (P,)) if src_row is not None else None,
             ops._check(src_scale, "moe_packed.src_scale", torch.float32, (P,)) if src_scale is not None else None,
             ops._check(w.packed, "moe_packed.w", torch.bfloat16), ops._check(out, "moe_packed.out", dtype, (P, cols)),
             ops._check(tiles, "moe_packed.tiles", torch.int32, (None, 4)), tiles.shape[0], int(tile_rows), P, w.rows, w.cols,
             *epilogue, ops.stream_handle())
        return out

    def first(self, x, w, activation, act, tiles, tile_rows, most, src_row, src_scale):
        if w.packed is None or not w.gated:
            return super().first(x, w, activation, act, tiles, tile_rows, most, src_row, src_scale)
        return self.product(x, w, act, tiles, tile_rows, src_row, src_scale, epilogue=activation.epilogue)


register_kernel_set("routed_experts", PlainExperts, TunedExperts)
