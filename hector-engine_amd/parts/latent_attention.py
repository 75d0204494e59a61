"""Attention whose keys and values are one latent vector a token.

With H heads, d unrotated and r rotated query/key dims a head, values of e dims and a key/value latent of `rank`
dims, all from n, the mixer's input:
    q = W_q n, or, with a query latent of q_rank > 0 dims, c_q = rms(W_dq n) * g_q, q = W_uq c_q
                                                        a head's q is [d unrotated | r rotated]
    [c' | k_r] = W_dkv n,      c = rms(c') * g_kv           k_r: r dims, one rotated key part for all heads
    head h: key [W_uk,h c | rot(k_r)], value W_uv,h c, score (q_h . key) * scale
    causal, the last `window` positions (0: all), softmax (with `sinks`: exp(sink_h) more in its denominator)
    out_gate: the heads' results side by side are multiplied element by element by sigmoid(W_g n)
    out = W_o (heads' results side by side)
The cache keeps c and rot(k_r) per token and nothing per head. Since q . (W_uk,h c) = (W_uk,h^T q) . c, the
step takes each head's unrotated query through W_uk,h^T and then runs the shared attention kernels as H
query heads over ONE key/value head whose key is [rot(k_r) | c] (r + rank wide, the rotated dims first)
and whose value is c; a head's result over the latents goes through W_uv,h (and the gate) before the output product.
The rotation is the position part's (half-split or interleaved pairs, optional YaRN scaling, whose factor on cos and
sin rides along); the scale is taken as given. kv_projection False: the part has no W_dkv and reads the latents of
another run's cache (the schedule's cache_from), with matrices of its own.

One product over n gives [q (| k latent) | gate] (with a query latent W_dq stays a product of its own); then the per-head
key products write the queries' latent dims, ops.latent_cache does the norm, the rotations and the cache write, and
everything behind (cache pages, window, sinks, the routes to the plain / MFMA kernels) is the attention part's.
names: the suffixes of its tensors (q, dq, dq_norm, uq, dkv, dkv_norm, uk, uv, sinks, gate, o)."""
from __future__ import annotations

import torch

from ..kernels import ops
from .attention import Attention
from .base import BuildEnv, LayerCache, PartSpec, StepContext, TensorSpec, param, register_part, tensor_name
from .linear import Linear

_NAMES = {"q": "q_proj.weight", "dq": "q_a_proj.weight", "dq_norm": "q_a_norm.weight", "uq": "q_b_proj.weight",
          "dkv": "kv_a_proj.weight", "dkv_norm": "kv_a_norm.weight", "uk": "k_b_proj.weight", "uv": "v_b_proj.weight",
          "sinks": "sinks", "gate": "gate.weight", "o": "o_proj.weight"}


@register_part("mixer", "latent_attention")
class LatentAttention(Attention):
    accepts_normed_rows = True

    def __init__(self, params: dict, prefix: str, env: BuildEnv):
        self.d = param(params, "head_dim", int)            # unrotated dims of a head's query and key
        self.r = param(params, "rotary_dim", int, 0)        # rotated dims
        self.e = param(params, "value_dim", int, self.d)
        self.rank = param(params, "kv_rank", int)
        self.q_rank = param(params, "q_rank", int, 0)
        self.norm_eps = param(params, "eps", float)
        self.gated = param(params, "out_gate", bool, False)
        heads = param(params, "num_heads", int)
        if min(self.d, self.e, self.rank, heads) <= 0 or self.q_rank < 0 or self.r < 0 or self.r % 2:
            raise ValueError("latent_attention: sizes must be positive and the rotated dims even")
        inner = {"hidden_size": param(params, "hidden_size", int), "num_heads": heads, "num_kv_heads": 1,
                 "head_dim": self.r + self.rank, "value_dim": self.rank, "window": param(params, "window", int, 0),
                 "scale": param(params, "scale", float), "sinks": param(params, "sinks", bool, False),
                 "kv_projection": param(params, "kv_projection", bool, True),
                 "position": param(params, "position", PartSpec, PartSpec("none"))}
        super().__init__(inner, prefix, env)
        rot = self.position.rotary()
        if self.position.custom or (rot[1] if rot else 0) != self.r:
            raise ValueError("latent_attention: the position part must be a rotation of exactly the rotated dims")
        names = param(params, "names", dict, {})
        self._lnames = {k: tensor_name(prefix, names, k, v) for k, v in _NAMES.items()}
        self.dq = self.uq = self.front = self.front_q = None
        self.dq_norm = self.dkv_norm = self.w_keys = self.w_values = None
        self.keys_mfma = self.values_mfma = False
        # columns of the front product: q or nothing, the latent and the rotated key part, the gate
        self.q_cols = 0 if self.q_rank else heads * (self.d + self.r)
        self.down_cols = self.rank + self.r if self.kv_projection else 0
        self.gate_cols = heads * self.e if self.gated else 0

    def tensor_specs(self):
        n, H, D = self._lnames, self.H, self.hidden
        specs = {n["uk"]: TensorSpec((H * self.d, self.rank), ("normal", 0.1)),
                 n["uv"]: TensorSpec((H * self.e, self.rank), ("normal", 0.1)),
                 n["o"]: TensorSpec((D, H * self.e))}
        if self.q_rank:
            specs.update({n["dq"]: TensorSpec((self.q_rank, D)), n["dq_norm"]: TensorSpec((self.q_rank,), ("gain", 1.0, 0.1)),
                          n["uq"]: TensorSpec((H * (self.d + self.r), self.q_rank), ("normal", 0.1))})
        else:
            specs[n["q"]] = TensorSpec((H * (self.d + self.r), D))
        if self.kv_projection:
            specs.update({n["dkv"]: TensorSpec((self.rank + self.r, D)),
                          n["dkv_norm"]: TensorSpec((self.rank,), ("gain", 1.0, 0.1))})
        if self.gated:
            specs[n["gate"]] = TensorSpec((H * self.e, D))
        if self.has_sinks:
            specs[n["sinks"]] = TensorSpec((H,), ("normal", 1.0))
        specs.update(self.position.tensor_specs())
        return specs

    def bind(self, tensors):
        n, H = self._lnames, self.H

        def front(*parts):
            """One matrix of the given rows, with rows of zeros so that the product's rows stay a multiple of 8 wide."""
            ws = [p for p in parts if p is not None]
            if not ws:
                return None
            spare = -sum(w.shape[0] for w in ws) % 8
            if spare:
                ws.append(torch.zeros((spare, self.hidden), dtype=ws[0].dtype, device=ws[0].device))
            return Linear(torch.cat(ws, 0).contiguous() if len(ws) > 1 else ws[0])

        gate = tensors.pop(n["gate"]) if self.gated else None
        q = None if self.q_rank else tensors.pop(n["q"])
        down = tensors.pop(n["dkv"]) if self.kv_projection else None
        self.front = front(q, down, gate)
        # a run that reads another run's cache leaves the latent's rows out
        self.front_q = front(q, gate) if self.kv_projection else self.front
        if self.q_rank:
            self.dq, self.uq, self.dq_norm = Linear(tensors[n["dq"]]), Linear(tensors[n["uq"]]), tensors[n["dq_norm"]]
        if self.kv_projection:
            self.dkv_norm = tensors[n["dkv_norm"]]
        # a head's matrices: W_uk,h^T takes d to rank, W_uv,h takes rank to e; on the matrix cores both lie [head][out][in],
        # for the plain products [head][in][out]
        uk, uv = tensors[n["uk"]].view(H, self.d, self.rank), tensors[n["uv"]].view(H, self.e, self.rank)
        mfma = self.fast and uk.dtype == uv.dtype == torch.bfloat16
        # (the rows q lies in are a multiple of 8 wide: the front product's by its spare rows)
        self.keys_mfma = mfma and ops.head_product_mfma_ok(self.d, self.uq.out_features if self.q_rank else 8, self.d + self.r)
        self.values_mfma = mfma and ops.head_product_mfma_ok(self.rank, H * self.pd, self.pd)
        self.w_keys = (uk.transpose(1, 2) if self.keys_mfma else uk).contiguous()
        self.w_values = (uv if self.values_mfma else uv.transpose(1, 2)).contiguous()
        self.o_proj = Linear(tensors[n["o"]])
        if self.has_sinks:
            self.sinks = tensors[n["sinks"]]
        self.position.bind(tensors)

    def _encoded_q(self, x, ctx: StepContext, cache: LayerCache):
        rows, H, d, r, rank, pd = ctx.rows, self.H, self.d, self.r, self.rank, self.pd
        writes = cache.writes
        proj = self.front if writes else self.front_q
        y = proj(x, rows, ctx) if proj is not None else None      # [rows, q | rank | r | gate]
        at = self.q_cols
        if self.q_rank:
            cq = self.dq(x, rows, ctx)
            ops.rmsnorm_rows(cq, cq, self.dq_norm, rows, self.q_rank, self.q_rank, self.q_rank, self.norm_eps)
            q = self.uq(cq, rows, ctx)                            # [rows, H (d | r)]
        else:
            q = y[:, :at]
        down = None
        if writes:
            down = y[:, at:at + self.down_cols]
            at += self.down_cols
        gate = y[:, at:at + self.gate_cols] if self.gated else None
        q_out = ctx.alloc((rows, H * pd))                         # [rows, H (r | rank | padding)]
        ops.head_product(q_out.unflatten(1, (H, pd))[:, :, r:r + rank], q.unflatten(1, (H, d + r))[:, :, :d], self.w_keys, rows,
                         transposed=self.keys_mfma)
        rot = self.position.rotary()
        ops.latent_cache(q_out, cache.kpool, cache.vpool, q, down, self.dkv_norm, self.norm_eps, ctx.positions, ctx.row_seq,
                         ctx.seq_slot, cache.page_table, rot[0] if rot else None, rows, H, d, r, rank, pd,
                         interleaved=self.position.interleaved, mscale=self.position.mscale)
        return q_out, gate

    def _project(self, out, rows: int, ctx: StepContext, gate=None):
        H = self.H
        values = ctx.alloc((rows, H * self.e))
        ops.head_product(values.unflatten(1, (H, self.e)), out.unflatten(1, (H, self.pd))[:, :, :self.rank],
                         self.w_values, rows, gate=gate, transposed=self.values_mfma)
        return self.o_proj(values, rows, ctx, sink=ctx.take_sink())
