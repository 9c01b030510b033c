"""Python faces of the kernels for what a token's id brings to the stream (csrc/token_input.hip): a normed embedding, and the
gate of a layer's own per-token table. As everywhere in ops: operands are checked on the host, then the kernel is launched on
the current stream."""
from __future__ import annotations

import ctypes

import torch

from .kernels import _require_weight, is_blocked
from .lib import KernelError, check, code, declare, entry, ptr, require, stream
from .recurrent import _cols

_vp, _i, _f = ctypes.c_void_p, ctypes.c_int, ctypes.c_float
_FLOATS = (torch.float32, torch.bfloat16)
EMBED_NORM_MAX_WIDTH = 15000

declare("llme_embed_norm", [_vp, _i, _vp, _vp, _i, _vp, _i, _i, _f, _i, _vp])
declare("llme_token_gate", [_vp, _i, _vp, _i, _i, _i, _vp, _vp, _i, _i, _i, _vp])


def embed_norm(table: torch.Tensor, tokens: torch.Tensor, weight: torch.Tensor, eps: float, out: torch.Tensor) -> None:
    """out[t] = weight * e / sqrt(mean(e^2) + eps), e = table[tokens[t]] (the table row-major or blocked), 32-bit."""
    _, H = _require_weight(table, "table", _FLOATS)
    T = tokens.shape[0]
    require(tokens, "tokens", torch.int32, (T,))
    require(weight, "weight", _FLOATS, (H,))
    require(out, "out", torch.float32, (T, H))
    check(entry("llme_embed_norm")(ptr(table), code(table.dtype), ptr(tokens), ptr(weight), code(weight.dtype), ptr(out), T, H, float(eps),
                                   1 if is_blocked(table) else 0, stream()), "embed_norm")


def token_gate(z: torch.Tensor, table: torch.Tensor, col: int, tokens: torch.Tensor, out: torch.Tensor) -> None:
    """out[t, j] = gelu_tanh(z[t, j]) * table[tokens[t], col + j] for out [T, n] (32-bit or bfloat16), z [T, n] a column range
    of a 32-bit buffer."""
    require(out, "out", _FLOATS, (None, None))
    T, n = out.shape
    ld = _cols(z, "z", torch.float32, T, n)
    require(table, "table", _FLOATS, (None, None))
    require(tokens, "tokens", torch.int32, (T,))
    if not 0 <= col <= table.shape[1] - n:
        raise KernelError(f"token_gate: columns {col} .. {col + n} of a table of {table.shape[1]}")
    check(entry("llme_token_gate")(ptr(z), ld, ptr(table), code(table.dtype), table.shape[1], int(col), ptr(tokens), ptr(out),
                                   code(out.dtype), T, n, stream()), "token_gate")


def gemm_token_gate(x: torch.Tensor, w: torch.Tensor, table: torch.Tensor, col: int, tokens: torch.Tensor, out: torch.Tensor,
                    choices=None) -> bool:
    """token_gate of z = x w^T in one launch, for few rows of a bfloat16 model (returns False, with nothing done, for any other
    step): x [T, K], w [n, K] (row-major or blocked), out [T, n]."""
    from .choices import DEFAULT
    from .mfma import FEW_ROWS, gemm_bf16_supported
    T, n = out.shape
    if not ((choices or DEFAULT).fast_gemm and T <= FEW_ROWS and out.dtype == torch.bfloat16 and table.dtype == torch.bfloat16
            and x.dtype == torch.bfloat16 and gemm_bf16_supported(x, w, out, False)):
        return False
    require(x, "x", torch.bfloat16, (T, None))
    K = x.shape[1]
    n_rows, _ = _require_weight(w, "w", torch.bfloat16, K)
    require(table, "table", torch.bfloat16, (None, None))
    require(tokens, "tokens", torch.int32, (T,))
    if n_rows != n or not 0 <= col <= table.shape[1] - n:
        raise KernelError(f"gemm_token_gate: {n_rows} rows, columns {col} .. {col + n} of a table of {table.shape[1]}")
    check(entry("llme_gemm_few_token_gate")(ptr(x), ptr(w), ptr(out), T, n, K, 1 if is_blocked(w) else 0, ptr(table), table.shape[1], int(col),
                                            ptr(tokens), stream()), "gemm_token_gate")
    return True
