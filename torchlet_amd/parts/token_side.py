"""A per-layer token input: besides the token's embedding, every layer adds something that it makes of the stream and of the layer's own
slice ``e`` of the token's row in a second table::

    y = proj (act(gate x) * e);    x <- x + w * y / rms(y)

The table is the model's (one tensor for all layers); :meth:`TokenSide.attach` hands the layer its columns.  ``y`` is left pending on the stream
with its norm, so that the next kernel that reads the stream norms it and adds it in 32-bit.
"""
from __future__ import annotations

import torch

from ..config.base import ConfigError
from ..kernels import ops
from .base import KEEP_COMPUTE, KEEP_FLOAT32, Part, WeightSpec, project_out


class TokenSide(Part):
    graph_safe = True

    def __init__(self, spec, dtype, device):
        super().__init__(spec, dtype, device)
        if ops.ACTIVATIONS.get(spec.activation, 99) >= 16:
            raise ConfigError(f"a token input's activation is an elementwise one, not {spec.activation!r}")
        self.hidden, self.dim, self.eps = spec.hidden, spec.dim, float(spec.eps)
        self.w_gate = self.w_proj = self.norm = self.table = None

    def kernel_libraries(self):
        return ["experts"]

    def weight_specs(self):
        return {"gate": WeightSpec((self.dim, self.hidden)), "proj": WeightSpec((self.hidden, self.dim)),
                "norm": WeightSpec((self.hidden,), keep=KEEP_FLOAT32, init="one_plus_normal")}

    def load_weights(self, tensors):
        self.w_gate = self._place(tensors["gate"], KEEP_COMPUTE)
        self.w_proj = self._place(tensors["proj"], KEEP_COMPUTE)
        self.norm = self._place(tensors["norm"], KEEP_FLOAT32)

    def attach(self, table: torch.Tensor) -> None:
        """``table [vocab, dim]``: this layer's columns of the model's table (a view)."""
        if table.dim() != 2 or table.shape[1] != self.dim:
            raise ConfigError(f"a token input of {self.dim} numbers got a slice of shape {tuple(table.shape)}")
        self.table = table

    def forward(self, x: torch.Tensor, ctx) -> torch.Tensor:
        """``x [T, hidden]`` -> ``y``: ``[T, hidden]``, or float32 slabs of partial sums ``[P, T, hidden]``."""
        T = x.shape[0]
        z = torch.empty((T, self.dim), dtype=torch.float32, device=x.device)
        ops.linear(x, self.w_gate, None, z)
        g = torch.empty((T, self.dim), dtype=self.dtype, device=x.device)
        ops.token_gate(z, ctx.token_ids, self.table, g, self.spec.activation)
        return project_out(g, self.w_proj, self.dtype)
