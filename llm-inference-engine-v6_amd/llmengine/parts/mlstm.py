"""Matrix memory with exponential gates (the mLSTM of xLSTM): per head a memory S [dim, vdim], a sum of keys z [dim] and a
level m that keeps the exponentials in range, all starting at zero:

    m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  z <- e^(f + m - m') z + e^(i - m') k;  m <- m'
    o = S^T q / (max(|z . q|, e^(-m)) + 1e-6)

q (times dim^-1/2) and k (heads x dim) and v (heads x vdim) are projections of the input without biases. The gates'
logarithms are numbers a head, softly capped at c = `gate_cap`: i = c tanh((Wi x + bi) / c) and
f = logsigmoid(c tanh((Wf x + bf) / c)) ("i", "i.b", "f", "f.b"). Each head's o is divided by its root mean square over
vdim, the joined heads are multiplied by a weight of their whole size ("norm") and by sigmoid(Wg x), then the output matrix.

Kept per request, 32-bit: the memory with z as one column more (a value that is always 1), transposed, and the level, a
copy for every column. The gates, their exponentials, the recurrence, the division, the norm and the gate are 32-bit.
"""
from __future__ import annotations

import torch

from .. import ops
from .base import CacheSpec, Getter, ParamSpec, Placement
from .projected import ProjectedMixer
from .registry import register_part


class MatrixMemory(ProjectedMixer):
    def __init__(self, hidden_size: int, heads: int, dim: int, vdim: int, gate_cap: float, eps: float):
        if not gate_cap > 0:
            raise ValueError(f"matrix memory: gate_cap={gate_cap} must be > 0")
        self.hidden_size = int(hidden_size)
        self.heads, self.dim, self.vdim = int(heads), int(dim), int(vdim)
        self.gate_cap, self.eps = float(gate_cap), float(eps)
        self.out_width = self.heads * self.vdim
        at, starts = 0, {}
        for name, rows in self.input_names():
            starts[name] = at
            at += rows
        self.columns = ops.mlstm.MlstmColumns(**starts)

    def input_names(self):
        qk, hv = self.heads * self.dim, self.heads * self.vdim
        return [("q", qk), ("k", qk), ("v", hv), ("g", hv), ("i", self.heads), ("f", self.heads)]

    def output_name(self):
        return "o"

    def param_specs(self):
        out = {name: ParamSpec((rows, self.hidden_size)) for name, rows in self.input_names()}
        out.update({"i.b": ParamSpec((self.heads,)), "f.b": ParamSpec((self.heads,)), "norm": ParamSpec((self.out_width,), "norm"),
                    "o": ParamSpec((self.hidden_size, self.out_width))})
        return out

    def refusals(self):
        if self.dim > ops.mlstm.MAX_DIM:
            return [f"dim={self.dim}: the recurrence kernels take key sizes up to {ops.mlstm.MAX_DIM}"]
        return []

    def cache_spec(self) -> CacheSpec:
        f32 = torch.float32
        return CacheSpec(state={"memory": ((self.heads, self.vdim + 1, self.dim), f32), "level": ((self.heads, self.vdim + 1), f32)})

    def load_core(self, get: Getter, placement: Placement) -> None:
        f32 = torch.float32
        self.gate_bias = placement.place(torch.cat([get("i.b").to(f32), get("f.b").to(f32)]), f32)
        self.norm_w = placement.place(get("norm"), f32)

    def core(self, p, step, cache, o, scale=1.0):
        ops.mlstm.mlstm(p, self.columns, self.gate_bias, self.gate_cap, cache.state["memory"], cache.state["level"], self.norm_w, step, o,
                        self.heads, self.dim, self.vdim, self.eps, scale)


register_part("mixer", "matrix_memory", MatrixMemory)
