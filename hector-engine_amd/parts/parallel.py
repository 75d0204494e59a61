"""Mixers side by side: every branch reads the same input, and the result is the weighted sum
    out = sum_b scale_b * branch_b(n).
At most one branch keeps keys and values in the cache (the layer's cache group is that branch's); the
branches' per-sequence states lie one behind the other in the layer's row of the state area.

branches: a list of {"mixer": PartSpec, "scale": float, "name": suffix of the branch's prefix}; with "norm" (a PartSpec of
a norm that is a row scale and a gain, for every branch or for none) and "norm_name" (the suffix of its prefix), a branch's
result passes that norm before the sum. Two normed branches are handed to a block that takes a pair as they are
(NormedPair): it norms and adds them on the way into the stream, in 32-bit and without a launch of their own."""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import BuildEnv, LayerCache, Mixer, NormedPair, PartSpec, StepContext, build_part, param, register_part


@register_part("mixer", "parallel")
class ParallelMixers(Mixer):
    accepts_normed_rows = False

    def __init__(self, params: dict, prefix: str, env: BuildEnv):
        super().__init__(prefix, env)
        branches = param(params, "branches", list)
        if not branches:
            raise ValueError("parallel: no branches")
        self.branches: list[Mixer] = []
        self.scales: list[float] = []
        for b in branches:
            spec = b["mixer"]
            if not isinstance(spec, PartSpec):
                raise TypeError("parallel: a branch's mixer must be a PartSpec")
            self.branches.append(build_part("mixer", spec, prefix + b["name"] + ".", env))
            self.scales.append(float(b.get("scale", 1.0)))
        self.norms = [build_part("norm", b["norm"], prefix + b["norm_name"] + ".", env) for b in branches if b.get("norm")]
        self.gains: list[torch.Tensor] = []          # the norms' gains times the branches' scales, 32-bit (bind)
        if self.norms and len(self.norms) != len(branches):
            raise ValueError("parallel: either every branch has a norm or none has")
        if sum(m.kv_need() is not None for m in self.branches) > 1:
            raise ValueError("parallel: at most one branch may keep keys and values in the cache")
        self.graph_safe = all(m.graph_safe for m in self.branches)
        # each branch's span of the state row, begun on 256 bytes
        self._state_at: list[tuple[int, int]] = []
        at = 0
        for m in self.branches:
            n = m.state_bytes()
            self._state_at.append((at, n))
            at += (n + 255) // 256 * 256 if n else 0
        self._state_bytes = at

    def children(self):
        return [*self.branches, *self.norms]

    def kv_need(self):
        for m in self.branches:
            need = m.kv_need()
            if need is not None:
                return need
        return None

    def state_bytes(self) -> int:
        return self._state_bytes

    def tensor_specs(self):
        specs = {}
        for m in self.children():
            specs.update(m.tensor_specs())
        return specs

    def bind(self, tensors):
        for m in self.children():
            m.bind(tensors)
        if any(n.carried() is None or len(n.carried()) != 2 for n in self.norms):
            raise ValueError("parallel: a branch's norm must be a row scale and a gain")
        self.gains = [(n.carried()[0].float() * s).contiguous() for n, s in zip(self.norms, self.scales)]

    def forward(self, x, ctx: StepContext, cache: LayerCache):
        rows = ctx.rows
        ctx.sink = None
        takes_pair, ctx.takes_pair = ctx.takes_pair, False
        total = None
        scale_of_total = 1.0
        scales = [1.0] * len(self.branches) if self.norms else self.scales
        results = []
        for m, scale, (at, n) in zip(self.branches, scales, self._state_at):
            state = cache.state[:, at:at + n] if n and cache.state is not None else None
            mine = LayerCache(cache.kpool, cache.vpool, cache.page_table, cache.writes, state) \
                if m.kv_need() is not None else LayerCache(None, None, None, False, state)
            out = m.forward(x, ctx, mine)
            if self.norms:
                results.append(out)
                continue
            if total is None:
                total, scale_of_total = out, scale
            else:
                joined = ctx.alloc((rows, out.shape[-1]), out.dtype)
                ops.scaled_sum(joined, total, out, rows, scale_of_total, scale)
                total, scale_of_total = joined, 1.0
        if self.norms:
            eps = [n.carried()[1] for n in self.norms]
            if len(results) == 2 and eps[0] == eps[1]:
                pair = NormedPair(*results, *self.gains, eps[0], rows)
                return pair if takes_pair else pair.tensor(ctx)
            for out, gain, e in zip(results, self.gains, eps):
                D = out.shape[-1]
                normed = ctx.alloc((rows, D), out.dtype)
                ops.rmsnorm_rows(normed, out, gain, rows, D, D, D, e)
                if total is not None:
                    ops.scaled_sum(normed, total, normed, rows, 1.0, 1.0)
                total = normed
            return total
        if scale_of_total != 1.0:
            joined = ctx.alloc((rows, total.shape[-1]), total.dtype)
            ops.scaled_sum(joined, total, total, rows, scale_of_total, 0.0)
            total = joined
        return total
