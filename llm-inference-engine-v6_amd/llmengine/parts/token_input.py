"""A layer's own input from the token's id: a table holds `dim` entries a layer for every token (one tensor, layer i's columns
from i dim on); a layer takes its entries e, gates them with the stream x, maps them to the stream's width and adds them:

    x <- x + N(P (gelu(G x) * e))

with the tanh form of GELU and N an RMS norm. Tensors of a layer: "gate" (G [dim, hidden]), "proj" (P [hidden, dim]), "norm".
"""
from __future__ import annotations

import torch

from .. import ops
from .base import Getter, Norm, ParamSpec, Part, Placement


class TokenTable(Part):
    """The table of every layer's entries, [vocab, layers * dim]."""
    graph_safe = True

    def __init__(self, vocab_size: int, layers: int, dim: int, tensor: str = "embed"):
        self.vocab_size, self.layers, self.dim, self.tensor = int(vocab_size), int(layers), int(dim), tensor
        self.weight: torch.Tensor | None = None

    def param_specs(self):
        return {self.tensor: ParamSpec((self.vocab_size, self.layers * self.dim))}

    def load_params(self, get: Getter, placement: Placement) -> None:
        self.weight = placement.place(get(self.tensor))


class TokenInput(Part):
    """Layer `index`'s step above. `norm` stands behind the map, as a block's norms stand behind its sublayers."""
    graph_safe = True

    def __init__(self, hidden_size: int, table: TokenTable, index: int, norm: Norm):
        if not 0 <= index < table.layers:
            raise ValueError(f"token input {index} of a table for {table.layers} layers")
        self.hidden_size, self.table, self.index, self.norm = int(hidden_size), table, int(index), norm

    def children(self):
        return {"norm": self.norm}

    def param_specs(self):
        H, d = self.hidden_size, self.table.dim
        return {"gate": ParamSpec((d, H)), "proj": ParamSpec((H, d))}

    def load_params(self, get: Getter, placement: Placement) -> None:
        self.w_gate = placement.place_matrix(get("gate"))
        self.w_proj = placement.place_matrix(get("proj"))

    def forward(self, x: torch.Tensor, step, out: torch.Tensor, accumulate: bool) -> None:
        """out [T, H] (32-bit) (+)= P (gelu(G x) * e), in front of the norm."""
        T, d = x.shape[0], self.table.dim
        g = step.buffer("token_input.gated", (T, d), step.act_dtype)
        if not ops.token_input.gemm_token_gate(x, self.w_gate, self.table.weight, self.index * d, step.tokens, g, choices=step.choices):
            z = step.buffer("token_input.gate", (T, d), torch.float32)
            ops.gemm(x, self.w_gate, z, choices=step.choices)
            ops.token_input.token_gate(z, self.table.weight, self.index * d, step.tokens, g)
        ops.gemm(g, self.w_proj, out, accumulate, fixed_order=step.fixed_order, choices=step.choices)
