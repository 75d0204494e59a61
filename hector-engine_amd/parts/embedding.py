"""Token embedding and output head.

Embedding: h[t] = E[id_t], no scaling, written straight into the fp32 residual
stream (reference: src/graph_builder.cpp:998, kernels/linear.cu:36-69).
Head: logits = n W^T with W the head's own matrix, or the embedding matrix when
tied (src/graph_builder.cpp:1019-1036); only the wanted rows are computed and
the logits are fp32 in both precisions.

The embedding's `norm` (a norm that is a row scale and a gain, with its own prefix `norm_prefix`) is applied to the row
before it becomes the stream, in the same launch.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import BuildEnv, Part, PartSpec, StepContext, TensorSpec, build_part, param, register_part, tensor_name
from .linear import Linear


@register_part("embedding", "token_embedding")
class TokenEmbedding(Part):
    def __init__(self, params: dict, prefix: str, env: BuildEnv):
        super().__init__(prefix, env)
        self.vocab = param(params, "vocab_size", int)
        self.hidden = param(params, "hidden_size", int)
        self.scale = param(params, "scale", float, 1.0)      # h[t] = E[id_t] * scale
        self._name = tensor_name(prefix, param(params, "names", dict, {}), "weight", "weight")
        self.table: torch.Tensor | None = None
        spec = param(params, "norm", PartSpec, None)
        self.norm = None if spec is None else build_part("norm", spec, param(params, "norm_prefix", str), env)

    def children(self):
        return [] if self.norm is None else [self.norm]

    def tensor_specs(self):
        specs = {self._name: TensorSpec((self.vocab, self.hidden))}
        for c in self.children():
            specs.update(c.tensor_specs())
        return specs

    def bind(self, tensors):
        self.table = tensors[self._name]
        for c in self.children():
            c.bind(tensors)
            if c.carried() is None or len(c.carried()) != 2:
                raise ValueError("token_embedding: its norm must be a row scale and a gain")

    def forward(self, ids: torch.Tensor, rows: int, ctx: StepContext) -> torch.Tensor:
        out = ctx.alloc((rows, self.hidden), torch.float32)
        gain, eps = (None, 0.0) if self.norm is None else self.norm.carried()
        ops.embedding(out, self.table, ids, rows, self.scale, gain, eps)
        return out


@register_part("head", "linear_head")
class LinearHead(Part):
    accepts_normed_rows = True

    def __init__(self, params: dict, prefix: str, env: BuildEnv):
        super().__init__(prefix, env)
        self.vocab = param(params, "vocab_size", int)
        self.hidden = param(params, "hidden_size", int)
        self.tied_to = param(params, "tied_to", str, "")   # full name of the tensor it shares
        self._name = tensor_name(prefix, param(params, "names", dict, {}), "weight", "weight")
        self.linear: Linear | None = None

    def tensor_specs(self):
        if self.tied_to:
            return {}
        return {self._name: TensorSpec((self.vocab, self.hidden))}

    def bind(self, tensors):
        name = self.tied_to or self._name
        self.linear = Linear(tensors[name])

    def forward(self, x: torch.Tensor, rows: int, ctx: StepContext) -> torch.Tensor:
        return self.linear(x, rows, ctx, out_dtype=torch.float32)
