"""Token embedding and output head.

Embedding: h = E[token] with no multiplier (src/kernels.cpp:59-66). Head:
logits = x . W^T in 32-bit (src/engine.cpp:242-249); a tied head is the embedding
table itself, one buffer under two names (src/weights.cpp:244-267, src/model.cpp:185-190).
"""
from __future__ import annotations

import torch

from .. import ops
from .base import Getter, Head, Norm, ParamSpec, Placement, TokenEmbedding
from .registry import register_part


class Embedding(TokenEmbedding):
    graph_safe = True

    def __init__(self, vocab_size: int, hidden_size: int, tensor: str = "weight", scale: float = 1.0, norm: Norm | None = None):
        self.vocab_size, self.hidden_size = int(vocab_size), int(hidden_size)
        self.tensor = tensor            # the local name of the table ("": the part's own name)
        self.norm = norm                # what the (scaled) rows pass before they become the stream ("norm")
        self.scale = float(scale)       # a multiplier on every row, applied in 32-bit
        self.weight: torch.Tensor | None = None

    def param_specs(self):
        return {self.tensor: ParamSpec((self.vocab_size, self.hidden_size), "linear")}

    def children(self):
        return {"norm": self.norm} if self.norm is not None else {}

    def load_params(self, get: Getter, placement: Placement) -> None:
        # (a tied head reads the table as a weight matrix: the gather takes either layout)
        self.weight = placement.place_matrix(get(self.tensor))

    def forward(self, tokens: torch.Tensor, out: torch.Tensor, step=None) -> None:
        rms = self.norm.fused_rms() if self.norm is not None else None
        if rms is not None and self.scale == 1.0 and self.hidden_size <= ops.token_input.EMBED_NORM_MAX_WIDTH:
            ops.token_input.embed_norm(self.weight, tokens, rms[0], rms[1], out)
            return
        rows = out if self.norm is None else step.buffer("embedding.rows", tuple(out.shape), torch.float32)
        ops.embed_gather(self.weight, tokens, rows)
        if self.scale != 1.0:
            ops.scale_(rows, self.scale)
        if self.norm is not None:
            self.norm.forward(rows, out)


class OutputHead(Head):
    graph_safe = True

    def __init__(self, vocab_size: int, hidden_size: int, tied_to: TokenEmbedding | None = None, tensor: str = "weight",
                 scale: float = 1.0, softcap: float = 0.0):
        self.vocab_size, self.hidden_size = int(vocab_size), int(hidden_size)
        self.scale = float(scale)       # a multiplier on the logits, applied in 32-bit
        self.softcap = float(softcap)   # > 0: the (scaled) logits become softcap * tanh(logits / softcap), in 32-bit
        self.tied_to = tied_to
        self.tensor = tensor
        self._weight: torch.Tensor | None = None

    def param_specs(self):
        if self.tied_to is not None:
            return {}
        return {self.tensor: ParamSpec((self.vocab_size, self.hidden_size), "linear")}

    def load_params(self, get: Getter, placement: Placement) -> None:
        if self.tied_to is None:
            self._weight = placement.place_matrix(get(self.tensor))

    @property
    def weight(self) -> torch.Tensor:
        return self.tied_to.weight if self.tied_to is not None else self._weight

    def fuses_norm(self, h: torch.Tensor, norm, n_rows: int, step) -> bool:
        rms = norm.fused_rms()
        return (rms is not None and step.act_dtype == torch.bfloat16
                and ops.gemv_norm_supported(h, rms[0], self.weight, n_rows, gated=False, choices=step.choices))

    def _finish(self, out: torch.Tensor) -> None:
        if self.scale != 1.0:
            ops.scale_(out, self.scale)
        if self.softcap > 0:
            ops.soft_cap_(out, self.softcap)

    def forward(self, x: torch.Tensor, out: torch.Tensor, step=None) -> None:
        ops.gemm(x, self.weight, out, choices=getattr(step, "choices", None))
        self._finish(out)

    def forward_normed_rows(self, h: torch.Tensor, rows: torch.Tensor, norm, out: torch.Tensor, step=None) -> None:
        """Logits of the chosen rows of the 32-bit stream, the final norm applied inside the product."""
        weight, eps = norm.fused_rms()
        ops.gemv_norm(h, weight, eps, self.weight, out, rows=rows)
        self._finish(out)


register_part("embedding", "table", Embedding)
register_part("head", "linear", OutputHead)
