"""A layer's own input per token: down( gelu(gate(h)) * table[token][part of the layer] ), gelu in its tanh form.

The table holds `dim` numbers per token and layer side by side ([vocab, layers * dim], one tensor for all layers); a
layer reads its `dim` columns from `offset` on.  Tensor names below the prefix: gate [dim, hidden], proj [hidden, dim];
the table's name is given whole.  The inner size is filled up to a multiple of 8 with zero rows and columns.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from ..kernels import ops
from .base import FeedForward, WeightSpec, add_to_residual, register_feed_forward


class TokenInput(FeedForward):
    graph_safe = True

    def __init__(self, prefix, dtype, device, *, hidden_size: int, vocab_size: int, dim: int, offset: int, table_width: int,
                 table_name: str, names: Dict[str, str] = None):
        super().__init__(prefix, dtype, device)
        self.hidden_size, self.vocab_size, self.dim = int(hidden_size), int(vocab_size), int(dim)
        self.offset, self.table_width, self.table_name = int(offset), int(table_width), table_name
        if self.dim <= 0 or self.offset < 0 or self.offset + self.dim > self.table_width:
            raise ValueError(f"{prefix}: columns {self.offset} .. {self.offset + self.dim - 1} of a table {self.table_width} wide")
        ops.check_linear_sizes(dtype, self.hidden_size, f"{prefix}: hidden_size")
        self.wide = -(-self.dim // 8) * 8
        n = {"gate": "gate", "proj": "proj"}
        n.update(names or {})
        self.names = {k: f"{prefix}.{v}" for k, v in n.items()}
        self.table = self.w_gate = self.w_proj = None

    def weights(self) -> List[WeightSpec]:
        return [WeightSpec(self.table_name, (self.vocab_size, self.table_width)),
                WeightSpec(self.names["gate"], (self.dim, self.hidden_size)),
                WeightSpec(self.names["proj"], (self.hidden_size, self.dim))]

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.table = tensors[self.table_name].contiguous()
        gate, proj = tensors[self.names["gate"]], tensors[self.names["proj"]]
        w_gate = torch.zeros((self.wide, self.hidden_size), dtype=self.dtype, device=gate.device)
        w_gate[:self.dim] = gate
        w_proj = torch.zeros((self.hidden_size, self.wide), dtype=self.dtype, device=gate.device)
        w_proj[:, :self.dim] = proj
        self.w_gate, self.w_proj = w_gate, w_proj

    def forward(self, h, ctx, residual):
        T, dev = h.shape[0], h.device
        z = ops.scratch("token_input_gated", (T, self.wide), self.dtype, dev)
        if T <= ops.TOKEN_GATE_ROWS:            # few rows (decoding): the product, the gelu and the table's row in one kernel
            ops.token_gate(h, self.w_gate, ctx.tokens, self.table, self.offset, self.dim, z)
        else:
            g = ops.linear(h, self.w_gate, ops.scratch("token_input_gate", (T, self.wide), torch.float32, dev))
            ops.gelu_table_rows(g, ctx.tokens, self.table, self.offset, self.dim, z)
        out = ops.linear(z, self.w_proj, ops.scratch("sublayer_out", (T, self.hidden_size), torch.float32, dev))
        return out if residual is None else add_to_residual(residual, out)


register_feed_forward("token_input", TokenInput)
