"""A memory per head that fades by a constant factor a token (linear attention with a fixed decay): no keys and
values in the cache, but a state of fixed size per sequence.

With H heads, keys of dk and values of dv dims (all from n, the mixer's input), act either nothing or SiLU:
    q = act(W_q n),  k = act(W_k n),  v = act(W_v n),  g = W_g n
    q and k through the position encoding (a half-split rotation or none), then k times k_scale
    S_t = decay_h S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t                       (decay: one constant a head)
    out = W_o (norm(o) * gate(g))
norm is the division of every head by its own root mean square ("heads", no stored gain), or the RMS norm over all
heads at once with a stored gain ("row"); gate is the sigmoid or SiLU. S starts at zero and lives in 32-bit floats in
the sequence's row of the cache's state area, which the kernels address on the device through the step's slots: prompt
steps, one-token steps, mixed steps and replayed graphs run the same launches. Rotation, activation, powers of the
decay, products and sums behind the projections are all in 32 bits, also under bfloat16 activations.

names: the suffixes of its tensors (q, k, v, g, o, norm)."""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import BuildEnv, LayerCache, Mixer, PartSpec, StepContext, TensorSpec, build_part, param, register_part, tensor_name
from .linear import Linear

_NAMES = {"q": "q_proj.weight", "k": "k_proj.weight", "v": "v_proj.weight", "g": "gate.weight", "o": "out_proj.weight",
          "norm": "norm.weight"}


@register_part("mixer", "decay_memory")
class DecayMemory(Mixer):
    accepts_normed_rows = False

    def __init__(self, params: dict, prefix: str, env: BuildEnv):
        super().__init__(prefix, env)
        self.hidden = param(params, "hidden_size", int)
        self.H = param(params, "num_heads", int)
        self.dk = param(params, "head_dim", int)
        self.dv = param(params, "value_dim", int, self.dk)
        self.decay = [float(d) for d in param(params, "decay", list)]
        self.eps = param(params, "eps", float)
        self.k_scale = param(params, "k_scale", float, 1.0)
        act = param(params, "activation", str, "")
        self.silu = act == "silu"
        self.norm_kind = param(params, "out_norm", str, "heads")
        self.gate = param(params, "gate", str, "sigmoid")
        if min(self.H, self.dk, self.dv) <= 0 or self.dk > 512:
            raise ValueError(f"decay_memory: heads, head_dim and value_dim must be positive, head_dim at most 512")
        if len(self.decay) != self.H or not all(0.0 <= d <= 1.0 for d in self.decay):
            raise ValueError(f"decay_memory: decay must give {self.H} numbers in [0, 1], got {self.decay}")
        if act not in ("", "silu") or self.norm_kind not in ("heads", "row") or self.gate not in ("sigmoid", "silu"):
            raise ValueError(f"decay_memory: unknown activation '{act}', out_norm '{self.norm_kind}' or gate '{self.gate}'")
        self.position = build_part("position", param(params, "position", PartSpec, PartSpec("none")), prefix, env)
        if self.position.custom or self.position.interleaved or self.position.mscale != 1.0:
            raise ValueError("decay_memory: the position encoding must be a plain half-split rotation or none")
        names = param(params, "names", dict, {})
        self._names = {k: tensor_name(prefix, names, k, d) for k, d in _NAMES.items()}
        self.qkvg: Linear | None = None
        self.o_proj: Linear | None = None
        self.norm = self.powers = None

    def children(self):
        return [self.position]

    def _state_floats(self) -> int:
        # the rule of csrc/decay_memory.hip, kept here so that the cache can be sized where no kernel library is loaded
        return self.H * self.dk * ((self.dv + 3) // 4 * 4)

    def state_bytes(self) -> int:
        return 4 * self._state_floats()

    def tensor_specs(self):
        n, H, dk, dv, D = self._names, self.H, self.dk, self.dv, self.hidden
        specs = {n["q"]: TensorSpec((H * dk, D)), n["k"]: TensorSpec((H * dk, D)), n["v"]: TensorSpec((H * dv, D)),
                 n["g"]: TensorSpec((H * dv, D)), n["o"]: TensorSpec((D, H * dv))}
        if self.norm_kind == "row":
            specs[n["norm"]] = TensorSpec((H * dv,), ("gain", 1.0, 0.1))
        specs.update(self.position.tensor_specs())
        return specs

    def bind(self, tensors):
        n = self._names
        ws = [tensors.pop(n[x]) for x in ("q", "k", "v", "g")]
        if len({w.dtype for w in ws}) != 1:
            raise TypeError(f"{self.prefix}: the projections are stored in different dtypes")
        self.qkvg = Linear(torch.cat(ws, 0).contiguous())
        device = ws[0].device
        del ws
        self.o_proj = Linear(tensors[n["o"]])
        self.norm = tensors[n["norm"]] if self.norm_kind == "row" \
            else torch.ones(self.H * self.dv, dtype=torch.float32, device=device)
        exponents = torch.arange(ops.DECAY_POWERS, dtype=torch.float64)
        self.powers = (torch.tensor(self.decay, dtype=torch.float64)[:, None] ** exponents).to(torch.float32).to(device)
        self.position.bind(tensors)

    def forward(self, x, ctx: StepContext, cache: LayerCache):
        if cache.state is None:
            raise RuntimeError(f"{self.prefix}: a fading memory needs its row of the state area")
        rows, H, dk, dv = ctx.rows, self.H, self.dk, self.dv
        if ops.decay_state_floats(H, dk, dv) != self._state_floats():
            raise RuntimeError(f"{self.prefix}: the kernel's state layout differs from the cache's")
        proj = self.qkvg(x, rows, ctx)                                   # [rows, q | k | v | g]
        y = ctx.alloc((rows, H * dv), torch.float32)
        rot = self.position.rotary()
        inv_freq = rot[0] if rot is not None else None
        floats = ops.decay_workspace_floats(rows, ctx.num_seqs, ctx.max_q_len, H, dk, dv)
        ws = ctx.alloc((floats,), torch.float32) if floats else None
        ops.decay_scan(y, proj[:, :H * dk], proj[:, H * dk:2 * H * dk], proj[:, 2 * H * dk:2 * H * dk + H * dv], self.powers,
                       cache.state, 0, ctx.positions, ctx.cu_seqlens, ctx.seq_slot, rows, ctx.num_seqs, ctx.max_q_len, H, dk,
                       dv, act=self.silu, k_scale=self.k_scale, inv_freq=inv_freq, workspace=ws)
        out = ctx.alloc((rows, H * dv))
        ops.gated_group_norm(out, y, proj[:, 2 * H * dk + H * dv:], self.norm, rows, H if self.norm_kind == "heads" else 1,
                             self.eps, gate_after="silu" if self.gate == "silu" else True)
        return self.o_proj(out, rows, ctx, sink=ctx.take_sink())
