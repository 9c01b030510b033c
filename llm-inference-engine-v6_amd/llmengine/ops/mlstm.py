"""Python faces of the kernels of the matrix memory with exponential gates (csrc/mlstm.hip). As everywhere in ops:
operands are checked on the host, then the kernels are launched on the current stream."""
from __future__ import annotations

import ctypes
from dataclasses import dataclass

import torch

from .lib import KernelError, check, code, declare, entry, ptr, require, stream
from .recurrent import _cols

_vp, _i, _f = ctypes.c_void_p, ctypes.c_int, ctypes.c_float
_FLOATS = (torch.float32, torch.bfloat16)
MAX_VDIM_SINGLE = 8192          # value entries of a head that the kernel for steps of single rows holds
MAX_DIM = 256                   # key channels of a head that the kernels hold
CHUNK_FROM = 48                 # rows a request brings from which a bfloat16 model's chunked kernels take it (smaller: the walk)
CHUNK_BYTES = 4 << 30           # the most scratch memory the chunked form may take
NEVER = 1 << 30
SINGLE_ROWS = True              # steps of one row a request have a kernel of their own (False: the walk; tests, measurements)

declare("llme_mlstm_walk", [_vp, _i, _i, _i, _i, _i, _i, _vp, _f, _f, _i, _i, _i, _vp, _vp, _vp, _vp, _vp, _i, _i, _vp])
declare("llme_mlstm_finish", [_vp, _vp, _vp, _i, _vp, _i, _i, _i, _i, _i, _f, _f, _vp, _vp, _i, _vp])
declare("llme_mlstm_single", [_vp, _i, _i, _i, _i, _i, _i, _i, _vp, _f, _f, _i, _i, _i, _vp, _vp, _vp, _i, _vp, _f, _f, _vp, _i, _i, _vp])
declare("llme_mlstm_chunk", [])
declare("llme_mlstm_chunked", [_vp, _i, _i, _i, _i, _i, _i, _i, _vp, _f, _f, _i, _i, _i, _vp, _vp, _vp, _vp, _i, _i, _i, _vp, _vp, _vp,
                               _vp, _vp, _vp, _vp, _f, _f, _vp, _i, _vp])


@dataclass(frozen=True)
class MlstmColumns:
    """Where the parts of the input product's rows begin: q, k [heads x dim], v, g [heads x vdim], i, f [heads]."""
    q: int
    k: int
    v: int
    g: int
    i: int
    f: int


def chunked_fits(p: torch.Tensor, cols: MlstmColumns, out: torch.Tensor, dim: int, vdim: int) -> bool:
    """Whether the chunked kernels take these operands: a bfloat16 result, key sizes a multiple of 8 and value sizes of 16,
    both up to 256, rows and columns aligned."""
    return (out.dtype == torch.bfloat16 and dim % 8 == 0 and vdim % 16 == 0 and max(dim, vdim) <= 256 and p.stride(0) % 4 == 0
            and p.data_ptr() % 16 == 0 and out.stride(0) % 4 == 0 and out.data_ptr() % 8 == 0
            and all(c % 4 == 0 for c in (cols.q, cols.k, cols.v, cols.g)))


def mlstm(p: torch.Tensor, cols: MlstmColumns, gate_bias: torch.Tensor, cap: float, memory: torch.Tensor, level: torch.Tensor,
          norm_w: torch.Tensor, step, out: torch.Tensor, heads: int, dim: int, vdim: int, eps: float, scale: float = 1.0,
          chunk_from: int | None = None) -> None:
    """The matrix memory over each request's rows, from and into its slot of memory [slots, heads, vdim + 1, dim] and level
    [slots, heads, vdim + 1]; out [T, heads vdim] = scale * (o / rms(o)) * norm_w * sigmoid(g), o the reads with queries times
    dim^-1/2. p [T, ..]: the input product's 32-bit rows (a view), gate_bias [2 heads] 32-bit, cap: the gates' soft cap.
    chunk_from: a request that brings that many rows or more goes through the chunked kernels where they take the operands
    (None: CHUNK_FROM)."""
    T = p.shape[0]
    ld = _cols(p, "p", torch.float32, T)
    need = max(cols.q + heads * dim, cols.k + heads * dim, cols.v + heads * vdim, cols.g + heads * vdim, cols.i + heads, cols.f + heads)
    if p.shape[1] < need or min(cols.q, cols.k, cols.v, cols.g, cols.i, cols.f) < 0:
        raise KernelError(f"mlstm: rows of {p.shape[1]} columns hold no {need}")
    if dim > MAX_DIM:
        raise KernelError(f"mlstm: key size {dim} is beyond the kernels' limit of {MAX_DIM}")
    if not cap > 0:
        raise KernelError(f"mlstm: cap={cap} must be > 0")
    require(gate_bias, "gate_bias", torch.float32, (2 * heads,))
    require(memory, "memory", torch.float32, (None, heads, vdim + 1, dim))
    require(level, "level", torch.float32, (memory.shape[0], heads, vdim + 1))
    require(norm_w, "norm_w", torch.float32, (heads * vdim,))
    ld_out = _cols(out, "out", _FLOATS, T, heads * vdim)
    if T != step.num_tokens:
        raise KernelError("mlstm: one row per token of the step")
    q_scale = float(dim) ** -0.5
    if T == step.num_seqs and vdim <= MAX_VDIM_SINGLE and SINGLE_ROWS:
        check(entry("llme_mlstm_single")(ptr(p), ld, cols.q, cols.k, cols.v, cols.g, cols.i, cols.f, ptr(gate_bias), float(cap), q_scale,
                                         heads, dim, vdim, ptr(memory), ptr(level), ptr(step.slots), T, ptr(norm_w), float(eps),
                                         float(scale), ptr(out), code(out.dtype), ld_out, stream()), "mlstm_single")
        return
    limit = CHUNK_FROM if chunk_from is None else int(chunk_from)
    longest = max(step.new_lens)
    if longest >= limit and chunked_fits(p, cols, out, dim, vdim):
        chunk = entry("llme_mlstm_chunk")()
        places = T // chunk + step.num_seqs
        if 2 * places * heads * (vdim + 1) * dim * 4 > CHUNK_BYTES:
            limit = NEVER
    else:
        limit = NEVER
    if limit < NEVER:
        f32, b16 = torch.float32, torch.bfloat16
        add = step.buffer("mlstm.add", (places, heads, vdim + 1, dim), f32)
        ends = step.buffer("mlstm.ends", (places, heads, 2), f32)
        s_hi = step.buffer("mlstm.start_hi", (places, heads, vdim, dim), b16)
        s_lo = step.buffer("mlstm.start_lo", (places, heads, vdim, dim), b16)
        z = step.buffer("mlstm.start_z", (places, heads, dim), f32)
        m = step.buffer("mlstm.start_m", (places, heads), f32)
        check(entry("llme_mlstm_chunked")(ptr(p), ld, cols.q, cols.k, cols.v, cols.g, cols.i, cols.f, ptr(gate_bias), float(cap), q_scale,
                                          heads, dim, vdim, ptr(memory), ptr(level), ptr(step.q_start), ptr(step.slots), step.num_seqs,
                                          (longest + chunk - 1) // chunk, limit, ptr(add), ptr(ends), ptr(s_hi), ptr(s_lo), ptr(z), ptr(m),
                                          ptr(norm_w), float(eps), float(scale), ptr(out), ld_out, stream()), "mlstm_chunked")
    if min(step.new_lens) < limit:
        o = step.buffer("mlstm.read", (T, heads, vdim + 2), torch.float32)
        check(entry("llme_mlstm_walk")(ptr(p), ld, cols.q, cols.k, cols.v, cols.i, cols.f, ptr(gate_bias), float(cap), q_scale, heads, dim,
                                       vdim, ptr(memory), ptr(level), ptr(step.q_start), ptr(step.slots), ptr(o), step.num_seqs, limit,
                                       stream()), "mlstm_walk")
        check(entry("llme_mlstm_finish")(ptr(o), ptr(norm_w), ptr(p) + 4 * cols.g, ld, ptr(out), code(out.dtype), ld_out, T, heads, vdim,
                                         float(eps), float(scale), ptr(step.seq_idx), ptr(step.q_start), limit, stream()), "mlstm_finish")
