"""A plain, slow implementation of the Lukupel design: whole sequences, float64, no cache, no batches, one function
per mechanism. It shares nothing with the engine and is what the engine's results are held against. Weights come as
a dict name -> torch tensor (any float type), the configuration as the dict that config.json holds.

Notation: T tokens, D the residual width, n query heads, g key/value heads, d query/key entries and dv value entries
per head, r rotated entries; i is the position of a query and j that of a key.

The layer: x <- x + c N1(mixer(x)); x <- x + c N2(ff(x)) with a constant c, the sublayers reading x itself and the
norms standing behind them. A layer may borrow all tensors of another one; what it remembers is its own.
"""
from __future__ import annotations

import contextlib
import math

import torch

F64 = torch.float64


# What a model of narrower storage keeps between its kernels (inputs of matrix products, the attention's and the memory's
# queries, keys and values) passes through here; the identity unless `bfloat16_storage` is in force.
_kept = lambda x: x


@contextlib.contextmanager
def bfloat16_storage():
    """Inside, those values are rounded to bfloat16: what rounding alone makes of a model's logits."""
    global _kept
    _kept = lambda x: x.to(torch.bfloat16).to(F64)
    try:
        yield
    finally:
        _kept = lambda x: x


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over the root of (the mean of its squares + eps), along the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms_unit(x, eps) * w.to(F64)


def linear(x, w, b=None):
    y = _kept(x) @ w.to(F64).T
    return y if b is None else y + b.to(F64)


# ---- positions ---------------------------------------------------------------------------------------
def pair_frequencies(rot: dict) -> torch.Tensor:
    """The angular step of pair c = (c, c + dims / 2): base^(-2c / dims), every one divided by the scaling factor."""
    r = int(rot["dims"])
    c = torch.arange(r // 2, dtype=F64)
    f = float(rot["base"]) ** (-2.0 * c / r)
    return f / float((rot.get("scaling") or {}).get("factor", 1.0))


def rotate_halves(x: torch.Tensor, positions: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """x [T, heads, >= dims]: entries c and c + dims / 2 of the first `dims` turn together by position * f_c; the
    entries behind them pass."""
    if not rot or not int(rot["dims"]):
        return x.clone()
    r = int(rot["dims"])
    ang = positions.to(F64)[:, None] * pair_frequencies(rot)[None, :]          # [T, r / 2]
    cs, sn = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    a, b = x[..., :r // 2], x[..., r // 2:r]
    return torch.cat([a * cs - b * sn, b * cs + a * sn, x[..., r:]], dim=-1)


def visible(T: int, chunk: int = 0) -> torch.Tensor:
    """[T, T] True where query i may read key j: j <= i and, with chunks, both in the same stretch of `chunk`
    positions counted from the sequence's start."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    if chunk:
        ok = ok & (i // chunk == j // chunk)
    return ok


# ---- softmax attention over a chunk --------------------------------------------------------------------
def attend(q, k, v, scale, mask):
    """q [T, n, d], k [T, g, d], v [T, g, dv] -> [T, n, dv]; head h reads key/value head h // (n // g)."""
    T, n, _ = q.shape
    g = k.shape[1]
    q, k, v = _kept(q), _kept(k), _kept(v)
    out = torch.zeros(T, n, v.shape[2], dtype=F64)
    for h in range(n):
        kv = h // (n // g)
        s = ((q[:, h] @ k[:, kv].T) * scale).masked_fill(~mask, -math.inf)
        out[:, h] = torch.softmax(s, dim=-1) @ v[:, kv]
    return out


def queries_keys(x, w, m, eps, positions):
    """Queries [T, n, d] and keys [T, g, d]: turned first, then every head over its root mean square."""
    T = x.shape[0]
    q = linear(x, w["q"]).view(T, m["heads"], m["dim"])
    k = linear(x, w["k"]).view(T, m["kv_heads"], m["dim"])
    return (rms_unit(rotate_halves(q, positions, m.get("rot")), eps), rms_unit(rotate_halves(k, positions, m.get("rot")), eps))


def chunked_attention(x, w, m, eps):
    T = x.shape[0]
    q, k = queries_keys(x, w, m, eps, torch.arange(T))
    v = linear(x, w["v"]).view(T, m["kv_heads"], m["vdim"])
    o = attend(q, k, v, m["scale"], visible(T, (m.get("mask") or {}).get("size", 0)))
    return linear(o.reshape(T, -1), w["o"])


# ---- matrix memory with exponential gates --------------------------------------------------------------
def soft_bounded(z, cap):
    return cap * torch.tanh(z / cap)


def log_gates(x, w, cap):
    """(i, f), each [T, n]: the logarithms of the input gate and of the forget gate."""
    i = soft_bounded(linear(x, w["i"], w["i.b"]), cap)
    f = -torch.log1p(torch.exp(-soft_bounded(linear(x, w["f"], w["f.b"]), cap)))
    return i, f


def matrix_memory(q, k, v, i, f, state=None):
    """q, k [T, n, d], v [T, n, dv], i, f [T, n]. Per head, with a running maximum m that starts at zero:
    m' = max(f + m, i), S' = e^(f + m - m') S + e^(i - m') k v^T, z' = e^(f + m - m') z + e^(i - m') k,
    o = S'^T q / (max(|z' . q|, e^(-m')) + 1e-6). Returns (o [T, n, dv], (S, z, m))."""
    T, n, d = q.shape
    dv = v.shape[2]
    q, k, v = _kept(q), _kept(k), _kept(v)
    if state is None:
        state = (torch.zeros(n, d, dv, dtype=F64), torch.zeros(n, d, dtype=F64), torch.zeros(n, dtype=F64))
    S, z, m = state
    out = torch.zeros(T, n, dv, dtype=F64)
    for t in range(T):
        top = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - top), torch.exp(i[t] - top)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = keep[:, None] * z + add[:, None] * k[t]
        m = top
        read = (S * q[t][:, :, None]).sum(1)
        weight = (z * q[t]).sum(-1).abs()
        out[t] = read / (torch.maximum(weight, torch.exp(-m)) + 1e-6)[:, None]
    return out, (S, z, m)


def mlstm(x, w, m, eps):
    T = x.shape[0]
    n, d, dv = m["heads"], m["dim"], m["vdim"]
    q = linear(x, w["q"]).view(T, n, d) * d ** -0.5
    k = linear(x, w["k"]).view(T, n, d)
    v = linear(x, w["v"]).view(T, n, dv)
    i, f = log_gates(x, w, float(m["gate_cap"]))
    o, _ = matrix_memory(q, k, v, i, f)
    o = rms_unit(o, eps).reshape(T, n * dv) * w["norm"].to(F64) * torch.sigmoid(linear(x, w["g"]))
    return linear(o, w["o"])


# ---- feed-forward -------------------------------------------------------------------------------------
def feed_forward(x, w):
    return linear(torch.clamp(linear(x, w["up"]), min=0.0) ** 2, w["down"])


def sub(weights: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


# ---- the model ----------------------------------------------------------------------------------------
def tensors_of(cfg: dict, i: int) -> int:
    """The layer whose tensors layer i runs on."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg: dict, weights: dict, tokens, return_layers: bool = False):
    """Logits [T, vocab] of one whole sequence (and the residual after every layer)."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = cfg["norm"]["eps"]
    c = float(cfg.get("residual_mult", 1.0))
    table = weights["embed"].to(F64)
    x = table[tokens] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    seen = []
    for i, layer in enumerate(cfg["layers"]):
        w = sub(weights, f"l{tensors_of(cfg, i)}.")
        mix = {"attention": chunked_attention, "mlstm": mlstm}[layer["type"]]
        x = x + c * norm(mix(x, sub(w, "mix."), layer["mixer"], eps), w["norm1"], eps)
        if layer.get("mlp"):
            x = x + c * norm(feed_forward(x, sub(w, "mlp.")), w["norm2"], eps)
        seen.append(x.clone())
    logits = linear(norm(x, weights["final.norm"], eps), table)
    cap = cfg.get("logit_softcap")
    if cap:
        logits = soft_bounded(logits, float(cap))
    return (logits, torch.stack(seen)) if return_layers else logits
