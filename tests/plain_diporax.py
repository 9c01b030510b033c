"""A plain, slow implementation of the Diporax design: whole sequences, float64, no cache, no batches, one function per
mechanism. It shares nothing with the engine and is what the engine's results are held against. Weights come as a dict
name -> torch tensor (any float type), the configuration as the dict that config.json holds.

Notation: T tokens, D the residual width, n query heads, g key/value heads, d query/key entries and dv value entries per
head, r rotated entries; i is the position of a query and j that of a key.

The layer: x <- x + a N1(mixer(x)); x <- x + b N2(ff(x)) with vectors a and b, the sublayers reading x itself and the norms
standing behind them; then x <- x + N3(P (gelu(G x) * e)), e the token's row of a table of the layer's own.
"""
from __future__ import annotations

import contextlib
import math

import torch

F64 = torch.float64


# What a model of narrower storage keeps between its kernels (inputs of matrix products, the attentions' and the memory's
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


def rms_norm(x: torch.Tensor, w, eps: float) -> torch.Tensor:
    """x over the root of (the mean of its squares + eps), along the last axis, times w."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(F64)


def linear(x, w, b=None):
    y = _kept(x) @ w.to(F64).T
    return y if b is None else y + b.to(F64)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- positions ---------------------------------------------------------------------------------------
def turns(rot: dict) -> tuple[torch.Tensor, float]:
    """(the angular step of each of dims / 2 pairs, the factor on cos and sin). Without scaling base^(-2c / dims) and 1.
    With scaling, a pair's step is divided by `factor` where the pair makes few turns over `original` positions, kept where
    it makes many, and a mixture along a ramp of pairs between the two."""
    r, base = int(rot["dims"]), float(rot["base"])
    steps = [base ** (-2.0 * c / r) for c in range(r // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(steps, dtype=F64), 1.0
    where = lambda t: r * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo = max(math.floor(where(sc["fast"])), 0)
    hi = min(math.ceil(where(sc["slow"])), r - 1)
    out = []
    for c, f in enumerate(steps):
        slowed = min(max((c - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * slowed + f * (1.0 - slowed))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(sc["factor"]) + 1.0


def _angles(positions, rot):
    f, mag = turns(rot)
    ang = positions.to(F64)[:, None] * f[None, :]
    return torch.cos(ang)[:, None, :] * mag, torch.sin(ang)[:, None, :] * mag         # [T, 1, r / 2]


def rotate_halves(x: torch.Tensor, positions: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """x [T, heads, >= dims]: entries c and c + dims / 2 of the first `dims` turn together; the entries behind them pass."""
    if not rot or not int(rot["dims"]):
        return x.clone()
    r = int(rot["dims"])
    cs, sn = _angles(positions, rot)
    a, b = x[..., :r // 2], x[..., r // 2:r]
    return torch.cat([a * cs - b * sn, b * cs + a * sn, x[..., r:]], dim=-1)


def rotate_neighbours(x: torch.Tensor, positions: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """The same with entries 2c and 2c + 1 as a pair."""
    if not rot or not int(rot["dims"]):
        return x.clone()
    r = int(rot["dims"])
    cs, sn = _angles(positions, rot)
    y = x.clone()
    y[..., 0:r:2] = x[..., 0:r:2] * cs - x[..., 1:r:2] * sn
    y[..., 1:r:2] = x[..., 1:r:2] * cs + x[..., 0:r:2] * sn
    return y


# ---- softmax attention ---------------------------------------------------------------------------------
def attend(q, k, v, scale, softcap=0.0, sink=None):
    """q [T, n, d], k [T, g, d], v [T, g, dv] -> [T, n, dv], every earlier token and the token itself visible; head h reads
    key/value head h // (n // g). sink [n]: a number whose exponential joins the sum of the weights."""
    T, n, _ = q.shape
    g = k.shape[1]
    q, k, v = _kept(q), _kept(k), _kept(v)
    hidden = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = torch.zeros(T, n, v.shape[2], dtype=F64)
    for h in range(n):
        kv = h // (n // g)
        s = (q[:, h] @ k[:, kv].T) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        s = s.masked_fill(hidden, -math.inf)
        if sink is not None:
            s = torch.cat([s, sink[h].to(F64).expand(T, 1)], dim=1)
        out[:, h] = torch.softmax(s, dim=-1)[:, :T] @ v[:, kv]
    return out


def head_gate(o, x, w):
    """o [T, n, dv] times one sigmoid a head."""
    return o * torch.sigmoid(linear(x, w))[:, :, None]


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros in front of the sequence."""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j].to(F64) * u[:T - back]
    return y


def mix_values(v, first, lam):
    lam = lam.to(F64).reshape(())
    return (1.0 - lam) * v + lam * first


def attention(x, w, m, eps, values):
    """values: the values of the first layer that mixes ({} until that layer has run; it puts its own there)."""
    T = x.shape[0]
    n, g, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    proj = {}
    for c in ("q", "k", "v"):
        u = linear(x, w[c], w[c + ".b"])
        proj[c] = causal_conv(u, w[c + ".conv"]) if m.get("conv") else u
    pos = torch.arange(T)
    q = rotate_halves(rms_norm(proj["q"].view(T, n, d), w["q.norm"], eps), pos, m.get("rot"))
    k = rotate_halves(rms_norm(proj["k"].view(T, g, d), w["k.norm"], eps), pos, m.get("rot"))
    v = proj["v"].view(T, g, dv)
    if m.get("v_mix"):
        if "first" in values:
            v = mix_values(v, values["first"].reshape(v.shape), w["vmix"])        # (entry by entry, however they are cut into heads)
        else:
            values["first"] = v
    o = attend(q, k, v, m["scale"], float(m.get("softcap") or 0.0))
    return linear(head_gate(o, x, w["g"]).reshape(T, -1), w["o"])


def latent_attention(x, w, m, eps):
    T = x.shape[0]
    n, d, dv, R, r = m["heads"], m["dim"], m["vdim"], m["kv_rank"], m["rot_dim"]
    pos = torch.arange(T)
    q = linear(rms_norm(linear(x, w["dq"]), w["dq.norm"], eps), w["uq"]).view(T, n, d + r)
    down = linear(x, w["dkv"])
    c = _kept(rms_norm(down[:, :R], w["dkv.norm"], eps))
    shared = rotate_neighbours(down[:, R:].view(T, 1, r), pos, m.get("rot"))
    q = torch.cat([q[..., :d], rotate_neighbours(q[..., d:], pos, m.get("rot"))], dim=-1)
    k = torch.cat([linear(c, w["uk"]).view(T, n, d), shared.expand(T, n, r)], dim=-1)
    v = linear(c, w["uv"]).view(T, n, dv)
    o = attend(q, k, v, m["scale"], sink=w["sink"])
    return linear(head_gate(o, x, w["g"]).reshape(T, -1), w["o"])


# ---- linear attention with a fixed decay a head ---------------------------------------------------------
def decayed_memory(q, k, v, decay, state=None):
    """q, k [T, n, d], v [T, n, dv], decay [n]. Per head S <- decay S + k v^T; o = S^T q. Returns (o, S)."""
    T, n, d = q.shape
    dv = v.shape[2]
    q, k, v = _kept(q), _kept(k), _kept(v)
    S = torch.zeros(n, d, dv, dtype=F64) if state is None else state
    out = torch.zeros(T, n, dv, dtype=F64)
    a = torch.as_tensor(decay, dtype=F64)[:, None, None]
    for t in range(T):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def lightning(x, w, m, eps):
    T = x.shape[0]
    n, d, dv = m["heads"], m["dim"], m["vdim"]
    q, k = (silu(linear(x, w[c])).view(T, n, d) for c in ("q", "k"))
    v = silu(linear(x, w["v"])).view(T, n, dv)
    o, _ = decayed_memory(q, k, v, m["decay"])
    o = rms_norm(o.reshape(T, n * dv), w["norm"], eps) * torch.sigmoid(linear(x, w["g"]))
    return linear(o, w["o"])


# ---- feed-forward --------------------------------------------------------------------------------------
def expert(x, w, name):
    return linear(silu(linear(x, w[name + ".gate"])) * linear(x, w[name + ".up"]), w[name + ".down"])


def experts(x, w, mlp):
    T = x.shape[0]
    top = mlp["router"]["top"]
    z = linear(x, w["router"])
    out = torch.zeros_like(x)
    for t in range(T):
        chosen = torch.argsort(z[t], descending=True, stable=True)[:top]
        weights = torch.softmax(z[t, chosen], dim=-1)
        for e, c in zip(chosen.tolist(), weights):
            out[t] += c * expert(x[t:t + 1], w, f"e{e}")[0]
    if mlp.get("shared"):
        out = out + expert(x, w, "shared") * torch.sigmoid(linear(x, w["shared.sg"]))
    return out


# ---- the token's own input to a layer ------------------------------------------------------------------
def token_input(x, w, e, eps):
    return rms_norm(linear(gelu(linear(x, w["side.gate"])) * e, w["side.proj"]), w["side.norm"], eps)


def sub(weights: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


# ---- the model ----------------------------------------------------------------------------------------
def forward(cfg: dict, weights: dict, tokens, return_layers: bool = False):
    """Logits [T, vocab] of one whole sequence (and the residual after every layer)."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = cfg["norm"]["eps"]
    x = rms_norm(weights["embed"].to(F64)[tokens], weights["embed.norm"], eps)
    dim = int(cfg["token_side"]["dim"]) if cfg.get("token_side") else 0
    seen, values = [], {}
    for i, layer in enumerate(cfg["layers"]):
        w = sub(weights, f"l{i}.")
        m, mw = layer["mixer"], sub(w, "mix.")
        if layer["type"] == "attention":
            y = attention(x, mw, m, eps, values)
        else:
            y = {"latent_attention": latent_attention, "lightning": lightning}[layer["type"]](x, mw, m, eps)
        x = x + rms_norm(y, w["norm1"], eps) * w["ls1"].to(F64)
        if layer.get("mlp"):
            x = x + rms_norm(experts(x, sub(w, "mlp."), layer["mlp"]), w["norm2"], eps) * w["ls2"].to(F64)
        if dim:
            e = weights["side.embed"].to(F64)[tokens][:, i * dim:(i + 1) * dim]
            x = x + token_input(x, w, e, eps)
        seen.append(x.clone())
    logits = linear(rms_norm(x, weights["final.norm"], eps), weights["head"])
    return (logits, torch.stack(seen)) if return_layers else logits
