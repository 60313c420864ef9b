"""Dense SwiGLU feed-forward: d = (silu(x Wg^T) * (x Wu^T)) Wd^T
(crates/forward/src/core/composites/dense_ffn.rs:116-186).  Gate and up matrices are
joined at load so that one matrix product feeds both and applies the gate before it stores."""
from __future__ import annotations

import torch

from .base import FEED_FORWARDS, FeedForward, Product, TensorSpec


@FEED_FORWARDS.register("swiglu")
class SwiGLU(FeedForward):
    replayable = True
    lazy_input = True

    def __init__(self, hidden_size: int, intermediate_size: int):
        self.hidden_size = hidden_size
        self.intermediate_size = intermediate_size

    def tensors(self):
        H, I = self.hidden_size, self.intermediate_size
        return {"gate.weight": TensorSpec((I, H)), "up.weight": TensorSpec((I, H)),
                "down.weight": TensorSpec((H, I))}

    def bind(self, weights, rt):
        self.rt = rt
        self.w_gate_up = rt.prepare_gate_up(weights["gate.weight"], weights["up.weight"])
        self.w_down = rt.prepare_weight(weights["down.weight"])

    def forward(self, x, step):
        rt, n, I = self.rt, x.shape[0], self.intermediate_size
        act = rt.buffer("ffn_act", n, I)
        rt.gemm_swiglu(x, self.w_gate_up, act)
        return Product(act, self.w_down)


@FEED_FORWARDS.register("gated_mlp")
class GatedMlp(SwiGLU):
    """d = (act(x Wg^T) * (x Wu^T)) Wd^T with the activation as a parameter (``gelu_tanh``, ``gelu``, ``silu``).
    Gate and up are one joined product whose kernel applies the activation (in 32-bit) before it stores."""

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "gelu_tanh"):
        from ..kernels import ops
        if activation not in ops.ACTIVATIONS:
            raise ValueError(f"gated_mlp: unknown activation '{activation}'; known: {sorted(ops.ACTIVATIONS)}")
        super().__init__(hidden_size, intermediate_size)
        self.activation = activation

    def forward(self, x, step):
        rt, n, I = self.rt, x.shape[0], self.intermediate_size
        act = rt.buffer("ffn_act", n, I)
        rt.gemm_swiglu(x, self.w_gate_up, act, gate=self.activation)
        return Product(act, self.w_down)


@FEED_FORWARDS.register("clamped_mlp")
class ClampedMlp(SwiGLU):
    """d = (g sigmoid(alpha g) (u + shift)) Wd^T with g = min(x Wg^T, limit) and u = x Wu^T clamped to +-limit.  Gate and up are
    one joined product whose kernel clamps and gates (in 32-bit) before it stores."""
    lazy_input = False

    def __init__(self, hidden_size: int, intermediate_size: int, limit: float, alpha: float = 1.702, shift: float = 1.0):
        if not limit > 0.0:
            raise ValueError(f"clamped_mlp: a limit of {limit}")
        super().__init__(hidden_size, intermediate_size)
        self.limit, self.alpha, self.shift = float(limit), float(alpha), float(shift)

    def forward(self, x, step):
        rt, n, I = self.rt, x.shape[0], self.intermediate_size
        act = rt.buffer("ffn_act", n, I)
        rt.gemm_clamped(x, self.w_gate_up, act, self.alpha, self.limit, self.shift)
        return Product(act, self.w_down)
