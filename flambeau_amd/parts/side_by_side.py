"""Two mixers side by side: both read the same normed input, each output is normed over the model width
(root mean square, eps inside the root, a plain gain of its own) and the results are added with a factor
each (a half each: their mean); with ``normed=False`` the outputs are added as they are, each with its factor.
The members are any registered mixers; one of them may keep pages, the others records per slot, which the
joined cache lays side by side.

Members whose outputs are added as they are and that can be joined (``Mixer.joinable``) share two products: one
projection of the input gives the columns of both, and one product adds both outputs, its input being what the two
output projections read, side by side, each times its factor."""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import MIXERS, JoinedCacheSpec, LayerCache, Mixer, PartSpec, Product, StateSpec, TensorSpec


@MIXERS.register("side_by_side")
class SideBySide(Mixer):
    replayable = True
    graph_safe = True           # as far as it goes itself: its members are asked one by one (``mixers``)

    @property
    def lazy_input(self):
        return all(m.lazy_input for m in self._members.values())

    def __init__(self, hidden_size: int, left: PartSpec, right: PartSpec, eps: float = 0.0, factors=(0.5, 0.5), normed: bool = True):
        self.hidden_size, self.eps, self.normed = hidden_size, float(eps), bool(normed)
        self.factors = (float(factors[0]), float(factors[1]))
        self.left, self.right = MIXERS.create(left), MIXERS.create(right)
        self._members = {"left": self.left, "right": self.right}
        specs = [m.cache_spec() for m in self._members.values()]
        paged = [s for s in specs if s is not None and s.page_group() is not None]
        if len(paged) > 1:
            raise ValueError("side_by_side: at most one member may keep pages")
        states = tuple(s if isinstance(s, StateSpec) else None for s in specs)
        if any(s is not None and s.page_group() is None and not isinstance(s, StateSpec) for s in specs):
            raise ValueError("side_by_side: a member's cache is neither paged nor a record per slot")
        if sum(s is not None for s in states) > 1:
            raise ValueError("side_by_side: at most one member may keep a record per slot")
        self._spec = JoinedCacheSpec(paged[0] if paged else None, states) if any(s is not None for s in specs) else None


    def cache_spec(self):
        return self._spec

    def subparts(self):
        return list(self._members.values())

    def mixers(self):
        """The members: what keeps work lists and signatures per kind of mixer looks inside."""
        return list(self._members.values())

    def signature_group(self):
        return ("side_by_side", self.left.signature_group(), self.right.signature_group())

    def step_signature(self, batch):
        return (self.left.step_signature(batch), self.right.step_signature(batch))

    def tensors(self):
        t = {f"{p}.{name}": spec for p, m in self._members.items() for name, spec in m.tensors().items()}
        if self.normed:
            t["left_out.weight"] = TensorSpec((self.hidden_size,), "vector32")
            t["right_out.weight"] = TensorSpec((self.hidden_size,), "vector32")
        return t

    def bind(self, weights, rt):
        self.rt = rt
        own = {p: {k[len(p) + 1:]: v for k, v in weights.items() if k.startswith(p + ".")} for p in self._members}
        self.joined = not self.normed and all(m.joinable for m in self._members.values())
        if self.joined:
            ins, outs = zip(*(m.join_weights(own[p]) for p, m in self._members.items()))
            self.out_widths = [w.shape[1] for w in outs]
            # (the tuned kernels read rows in pieces of 8 values: members whose widths are out of step go alone)
            self.joined = not (rt.tuned and any(w % 8 for w in self.out_widths))
        if self.joined:
            self.col_right = sum(w.shape[0] for w in ins[0])
            self.w_in = rt.prepare_weight(torch.cat([w for member in ins for w in member], dim=0).contiguous())
            self.w_o = rt.prepare_weight(torch.cat(outs, dim=1).contiguous())
        for p, m in self._members.items():
            m.joined = self.joined
            m.bind(own[p], rt)
        self.gain_left, self.gain_right = weights.get("left_out.weight"), weights.get("right_out.weight")

    def _member_cache(self, cache: LayerCache, index: int):
        """What a member sees: the pages as they are, and its own stretch of the slot's record."""
        spec = self._spec
        own = spec.states[index] if spec is not None else None
        state = None
        if own is not None and cache.state is not None:
            offsets, _ = spec.state_offsets()
            n = 1
            for d in own.shape:
                n *= d
            assert offsets[index] == 0 and cache.state.shape[1] == n      # one record per slot, checked when built
            state = cache.state.view(cache.state.shape[0], *own.shape)
        return LayerCache(kv=cache.kv, group=cache.group, state=state, writes=cache.writes)

    def forward(self, x, step, cache):
        rt, n, W = self.rt, x.shape[0], self.hidden_size
        if self.joined:
            proj = rt.buffer("sbs_proj", n, self.w_in.rows, torch.float32)
            rt.gemm(x, self.w_in, proj)
            both = rt.buffer("sbs_both", n, sum(self.out_widths))
            at = self.out_widths[0]
            self.left.forward_joined(proj, 0, step, self._member_cache(cache, 0), both[:, :at], self.factors[0])
            self.right.forward_joined(proj, self.col_right, step, self._member_cache(cache, 1), both[:, at:], self.factors[1])
            return Product(both, self.w_o)
        outs = []
        for index, (name, m) in enumerate(self._members.items()):
            d = m.forward(x, step, self._member_cache(cache, index))
            if isinstance(d, Product):
                d = d.compute(rt, out=rt.buffer("sbs_" + name, n, W, torch.float32))
            outs.append(d)
        delta = rt.buffer("sbs_delta", n, W, torch.float32)
        if self.normed:
            ops.norm_mix(outs[0], self.gain_left, self.factors[0], outs[1], self.gain_right, self.factors[1], delta, self.eps)
        else:
            ops.scaled_sum(outs[0], self.factors[0], outs[1], self.factors[1], delta)
        return delta
