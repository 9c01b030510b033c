"""Small Diporax configurations for the tests, and weights for them that the tests draw themselves (matrices of order one over
the root of their inputs, norm weights and layer scales around one, sinks and biases of order one). `sharp` multiplies an
attention's scale so that its softmax stands on a few keys: a key that is lost, or one too many, then moves the whole row."""
from __future__ import annotations

import json
import os

import torch


def moe(experts=5, top=2, ff=20, shared=14):
    out = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def _rot(dims, base, factor, original):
    out = {"base": base, "dims": dims}
    if factor:
        out["scaling"] = {"factor": factor, "original": original, "fast": 8.0, "slow": 0.5}
    return out


def latent(heads=3, dim=10, rot_dim=6, vdim=7, kv_rank=12, q_rank=18, scale=0.3, base=40.0, factor=3.0, original=60, sharp=1.0, mlp=None):
    """The mixer 'latent_attention'."""
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale * sharp}
    if rot_dim:
        m["rot"] = _rot(rot_dim, base, factor, original)
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def lightning(heads=3, dim=10, vdim=6, decay=(0.5, 0.93, 0.997), mlp=None):
    """The mixer 'lightning'."""
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)[:heads]}, "mlp": mlp}


def full(heads=6, kv_heads=2, dim=12, vdim=10, scale=0.3, softcap=8.0, conv=3, dims=8, base=70.0, factor=2.5, original=90, v_mix=True, sharp=1.0,
         mlp=None):
    """The mixer 'attention'."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale * sharp}
    if softcap:
        m["softcap"] = softcap
    if conv:
        m["conv"] = conv
    if dims:
        m["rot"] = _rot(dims, base, factor, original)
    if v_mix:
        m["v_mix"] = True
    return {"type": "attention", "mixer": m, "mlp": mlp}


def config(layers, width=28, vocab=61, eps=1e-5, side=6):
    out = {"architecture": "Diporax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": list(layers)}
    if side:
        out["token_side"] = {"dim": side}
    return out


# every mixer with and without a feed-forward, sizes that are no powers of two and that differ where the usual ones are equal
# or 1, three layers whose values mix (two head counts that give the same values) around one whose values do not
MIXED = config([
    full(mlp=moe()), lightning(mlp=moe(experts=4, top=4, shared=0)), latent(mlp=None), full(heads=5, kv_heads=5, dim=8, vdim=4, conv=4, v_mix=False, softcap=0),
    full(heads=4, kv_heads=4, dim=6, vdim=5, dims=6, conv=2, factor=0, mlp=moe(experts=7, top=1, ff=9, shared=30)), lightning(heads=2, dim=7, vdim=9),
    latent(heads=5, dim=6, rot_dim=8, vdim=11, kv_rank=20, q_rank=9, factor=0, mlp=moe()), full(conv=1, mlp=moe(experts=3, top=2))])

# sizes that the matrix kernels take (multiples of 16 and 32), as a model served in bfloat16 has them
ALIGNED = config([
    lightning(heads=4, dim=32, vdim=48, decay=(0.4, 0.9, 0.99, 0.999), mlp=moe(experts=6, top=2, ff=48, shared=64)),
    full(heads=8, kv_heads=2, dim=32, vdim=48, dims=16, conv=4, scale=0.2, softcap=20.0, base=10000.0, mlp=moe(experts=8, top=3, ff=32, shared=32)),
    latent(heads=4, dim=32, rot_dim=16, vdim=16, kv_rank=64, q_rank=48, scale=0.2, base=10000.0, mlp=moe(experts=4, top=1, ff=64, shared=16)),
    full(heads=6, kv_heads=6, dim=64, vdim=16, dims=64, conv=2, scale=0.15, softcap=15.0, base=3000.0)], width=64, vocab=128, side=16)

# the same without experts, so that no close call between two of them moves a row
NO_EXPERTS = config([dict(l, mlp=None) for l in ALIGNED["layers"]], width=64, vocab=128, side=24)


def random_config(seed: int) -> dict:
    """A configuration drawn at random: two to six layers of all kinds in any order, head counts, sizes and constants of many
    kinds (sizes the matrix kernels take and sizes they refuse), with and without experts, shared experts, mixed values."""
    import random
    rng = random.Random(seed)
    values = rng.choice([32, 48, 60, 96, 144])              # entries of the values that mix
    layers = []
    for _ in range(rng.randint(2, 6)):
        mlp = None
        if rng.random() < 0.6:
            experts = rng.choice([2, 3, 6, 9])
            mlp = moe(experts=experts, top=rng.randint(1, min(4, experts)), ff=rng.choice([16, 24, 40, 96]), shared=rng.choice([0, 16, 36, 64]))
        kind = rng.choice(["latent", "lightning", "full"])
        rot = dict(base=rng.choice([2000.0, 50000.0, 2e6]), factor=rng.choice([0, 2.0, 9.0]), original=rng.choice([64, 300, 2000]))
        if kind == "latent":
            layers.append(latent(heads=rng.choice([1, 2, 3, 5, 8]), dim=rng.choice([8, 16, 20, 40]), rot_dim=rng.choice([2, 8, 16, 24, 32]),
                                 vdim=rng.choice([8, 12, 16, 40]), kv_rank=rng.choice([16, 40, 64, 80, 144]), q_rank=rng.choice([16, 40, 56]),
                                 scale=rng.choice([0.1, 0.25, 0.5]), mlp=mlp, **rot))
        elif kind == "lightning":
            n = rng.choice([1, 2, 3, 5])
            layers.append(lightning(heads=n, dim=rng.choice([8, 16, 20, 40, 64, 136]), vdim=rng.choice([8, 16, 32, 40, 112, 144]),
                                    decay=[rng.choice([0.0, 0.3, 0.8, 0.97, 0.9995, 1.0]) if rng.random() < 0.5 else 0.98 for _ in range(n)], mlp=mlp))
        else:
            kv = rng.choice([k for k in (1, 2, 3, 4) if values % k == 0])
            dim = rng.choice([16, 24, 32, 48, 80, 128])
            mix = rng.random() < 0.7
            layers.append(full(heads=kv * rng.choice([1, 2, 3, 8]), kv_heads=kv, dim=dim, vdim=values // kv if mix else rng.choice([16, 20, 32, 96]),
                               scale=rng.choice([0.05, 0.2]), softcap=rng.choice([0, 5.0, 30.0]), conv=rng.choice([1, 2, 3, 4, 7]),
                               dims=rng.choice([0, 8, dim // 2 // 2 * 2, dim]), v_mix=mix, mlp=mlp, **rot))
    return config(layers, width=rng.choice([64, 96, 136, 160, 192]), vocab=rng.choice([100, 257, 384]), eps=rng.choice([1e-6, 1e-5]),
                  side=rng.choice([0, 7, 16, 40]))


def make_weights(cfg: dict, seed: int, dtype=torch.bfloat16) -> dict:
    """name -> tensor for every tensor of the configuration's model (names and shapes as the engine's model tree lists
    them; the values are the tests' own)."""
    from llmengine.config.registry import architecture_name, parse_config, resolve
    model = resolve(architecture_name(cfg)).build_model(parse_config(cfg))
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, spec in model.named_specs().items():
        shape = tuple(spec.shape)
        t = torch.randn(shape, generator=g)
        if name.endswith("vmix"):
            t = 0.5 + 0.1 * t
        elif name.endswith(".sink"):
            t = 1.5 * t
        elif name.endswith(".b"):
            t = 0.5 * t
        elif name.endswith((".ls1", ".ls2")):
            t = 0.8 + 0.3 * t
        elif name.endswith(".conv"):
            t = 0.6 * t
        elif len(shape) == 1:
            t = 1.0 + 0.2 * t                               # norm weights
        elif name in ("embed", "side.embed"):
            t = 0.7 * t
        else:
            t = 1.3 * t / shape[-1] ** 0.5
        out[name] = t.to(dtype)
    return out


def write_model(tmp_path, cfg: dict, seed: int, dtype=torch.bfloat16, weights: dict | None = None) -> tuple[str, dict]:
    from llmengine.weights import write_state_dict
    weights = weights if weights is not None else make_weights(cfg, seed, dtype)
    os.makedirs(str(tmp_path), exist_ok=True)
    with open(os.path.join(str(tmp_path), "config.json"), "w") as f:
        json.dump(cfg, f)
    write_state_dict(os.path.join(str(tmp_path), "model.safetensors"), weights)
    return str(tmp_path), weights
