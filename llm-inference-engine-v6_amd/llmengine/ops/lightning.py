"""Python faces of the kernels of linear attention with a fixed decay a head (csrc/lightning.hip). As everywhere in ops:
operands are checked on the host, then the kernels are launched on the current stream."""
from __future__ import annotations

import ctypes

import torch

from .lib import KernelError, check, code, declare, entry, ptr, require, stream
from .recurrent import _cols

_vp, _i, _f = ctypes.c_void_p, ctypes.c_int, ctypes.c_float
_FLOATS = (torch.float32, torch.bfloat16)
MAX_DIM = 256                   # key channels of a head that the kernels hold
CHUNK_FROM = 48                 # rows a request brings from which a bfloat16 model's chunked kernels take it (smaller: the walk)
CHUNK_BYTES = 4 << 30           # the most scratch memory the chunked form may take
NEVER = 1 << 30
SINGLE_ROWS = True              # steps of one row a request have a kernel of their own (False: the walk; tests, measurements)

declare("llme_lightning_walk", [_vp, _i, _i, _i, _i, _vp, _i, _i, _i, _vp, _vp, _vp, _vp, _i, _i, _vp])
declare("llme_lightning_single", [_vp, _i, _i, _i, _i, _vp, _i, _i, _i, _vp, _vp, _vp, _i, _vp])
declare("llme_lightning_chunk", [])
declare("llme_lightning_chunked", [_vp, _i, _i, _i, _i, _vp, _i, _i, _i, _vp, _vp, _vp, _i, _i, _i, _vp, _vp, _vp, _vp, _vp])
declare("llme_joined_norm_gate", [_vp, _vp, _vp, _i, _vp, _i, _i, _i, _i, _f, _f, _vp])


def chunked_fits(p: torch.Tensor, q_col: int, k_col: int, v_col: int, dim: int, vdim: int) -> bool:
    """Whether the chunked kernels take these operands: key sizes a multiple of 8 and value sizes of 16, both up to 256, rows
    and columns aligned."""
    return (dim % 8 == 0 and vdim % 16 == 0 and max(dim, vdim) <= 256 and p.stride(0) % 4 == 0 and p.data_ptr() % 16 == 0
            and all(c % 4 == 0 for c in (q_col, k_col, v_col)))


def lightning(p: torch.Tensor, q_col: int, k_col: int, v_col: int, decay: torch.Tensor, memory: torch.Tensor, step, o: torch.Tensor,
              heads: int, dim: int, vdim: int, chunk_from: int | None = None) -> None:
    """S <- a S + silu(k) silu(v)^T; o = S^T silu(q) over each request's rows, from and into its slot of memory
    [slots, heads, vdim, dim]; o [T, heads vdim] 32-bit. p [T, ..]: the input product's 32-bit rows (a view) with q, k
    (heads x dim) and v (heads x vdim) at their columns; decay [2 heads] (32-bit): a and ln a of every head. chunk_from: a
    request that brings that many rows or more goes through the chunked kernels, whose products round q, k and v to
    bfloat16, where they take the operands (NEVER: none; None: CHUNK_FROM in a bfloat16 model, none in a 32-bit one)."""
    T = p.shape[0]
    ld = _cols(p, "p", torch.float32, T)
    need = max(q_col + heads * dim, k_col + heads * dim, v_col + heads * vdim)
    if p.shape[1] < need or min(q_col, k_col, v_col) < 0:
        raise KernelError(f"lightning: rows of {p.shape[1]} columns hold no {need}")
    if dim > MAX_DIM:
        raise KernelError(f"lightning: key size {dim} is beyond the kernels' limit of {MAX_DIM}")
    require(decay, "decay", torch.float32, (2 * heads,))
    require(memory, "memory", torch.float32, (None, heads, vdim, dim))
    require(o, "o", torch.float32, (T, heads * vdim))
    if T != step.num_tokens:
        raise KernelError("lightning: one row per token of the step")
    if T == step.num_seqs and SINGLE_ROWS:
        check(entry("llme_lightning_single")(ptr(p), ld, q_col, k_col, v_col, ptr(decay), heads, dim, vdim, ptr(memory), ptr(step.slots),
                                             ptr(o), T, stream()), "lightning_single")
        return
    if chunk_from is None:
        chunk_from = CHUNK_FROM if step.act_dtype == torch.bfloat16 else NEVER
    limit, longest = int(chunk_from), max(step.new_lens)
    if longest >= limit and chunked_fits(p, q_col, k_col, v_col, dim, vdim):
        chunk = entry("llme_lightning_chunk")()
        places = T // chunk + step.num_seqs
        if 2 * places * heads * vdim * dim * 4 > CHUNK_BYTES:
            limit = NEVER
    else:
        limit = NEVER
    if limit < NEVER:
        shape = (places, heads, vdim, dim)
        add = step.buffer("lightning.add", shape, torch.float32)
        s_hi = step.buffer("lightning.start_hi", shape, torch.bfloat16)
        s_lo = step.buffer("lightning.start_lo", shape, torch.bfloat16)
        check(entry("llme_lightning_chunked")(ptr(p), ld, q_col, k_col, v_col, ptr(decay), heads, dim, vdim, ptr(memory), ptr(step.q_start),
                                              ptr(step.slots), step.num_seqs, (longest + chunk - 1) // chunk, limit, ptr(add), ptr(s_hi),
                                              ptr(s_lo), ptr(o), stream()), "lightning_chunked")
    if min(step.new_lens) < limit:
        check(entry("llme_lightning_walk")(ptr(p), ld, q_col, k_col, v_col, ptr(decay), heads, dim, vdim, ptr(memory), ptr(step.q_start),
                                           ptr(step.slots), ptr(o), step.num_seqs, limit, stream()), "lightning_walk")


def joined_norm_gate(o: torch.Tensor, weight: torch.Tensor, gate: torch.Tensor, out: torch.Tensor, eps: float, scale: float = 1.0) -> None:
    """out [T, width] = scale * o / sqrt(mean(o^2) + eps) * weight * sigmoid(gate), the mean over a whole row of o [T, width]
    (32-bit); gate and out may be column ranges of wider buffers."""
    require(o, "o", torch.float32, (None, None))
    T, width = o.shape
    require(weight, "weight", torch.float32, (width,))
    ld_g = _cols(gate, "gate", torch.float32, T, width)
    ld_out = _cols(out, "out", _FLOATS, T, width)
    check(entry("llme_joined_norm_gate")(ptr(o), ptr(weight), ptr(gate), ld_g, ptr(out), code(out.dtype), ld_out, T, width, float(eps),
                                         float(scale), stream()), "joined_norm_gate")
