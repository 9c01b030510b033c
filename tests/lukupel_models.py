"""Small Lukupel configurations for the tests, and weights for them that the tests draw themselves (matrices of order
one over the root of their inputs, norm weights around one, gate biases that let some heads remember and others forget).
`sharp` multiplies an attention's scale so that its softmax stands on a few keys: a key that is lost, or one too many, then
moves the whole row."""
from __future__ import annotations

import json
import os

import torch


def chunked(heads=6, kv_heads=2, dim=12, vdim=10, scale=0.9, base=50.0, dims=8, factor=2.0, chunk=9, ff=24, sharp=1.0, weights_of=None):
    """The mixer 'attention': rotated and then normed queries and keys, a chunk of the sequence visible."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale * sharp}
    if dims:
        m["rot"] = {"base": base, "dims": dims}
        if factor:
            m["rot"]["scaling"] = {"factor": factor}
    if chunk:
        m["mask"] = {"size": chunk}
    return _layer("attention", m, ff, weights_of)


def mlstm(heads=3, dim=10, vdim=6, gate_cap=5.0, ff=None, weights_of=None):
    """The mixer 'mlstm': a matrix memory with exponential gates."""
    return _layer("mlstm", {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}, ff, weights_of)


def _layer(kind, mixer, ff, weights_of):
    out = {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


def borrow(layers, j):
    """A layer that runs on the tensors of layers[j]."""
    return dict(json.loads(json.dumps(layers[j])), weights_of=j)


def config(layers, width=28, vocab=61, eps=1e-5, residual_mult=0.7, logit_softcap=9.0, embedding_scale=2.0):
    return {"architecture": "Lukupel", "vocab": vocab, "width": width, "embedding": {"scale": embedding_scale},
            "norm": {"eps": eps}, "residual_mult": residual_mult, "logit_softcap": logit_softcap, "layers": list(layers)}


def _mixed():
    layers = [chunked(chunk=11, ff=24), mlstm(ff=None), chunked(heads=3, kv_heads=3, dim=8, vdim=14, dims=8, factor=0, chunk=6, ff=None),
              mlstm(heads=2, dim=7, vdim=9, gate_cap=3.0, ff=20), chunked(heads=4, kv_heads=1, dim=10, vdim=5, dims=4, base=900.0, chunk=0, ff=18)]
    return layers + [borrow(layers, 1), borrow(layers, 0), borrow(layers, 3), mlstm(heads=1, dim=18, vdim=3), borrow(layers, 4)]


# both mixers with and without a feed-forward, sizes that are no powers of two, layers on the tensors of others (also two
# of one kind apart), a layer with tensors of its own behind them
MIXED = config(_mixed())


def _aligned():
    layers = [mlstm(heads=4, dim=32, vdim=48, gate_cap=8.0, ff=96),
              chunked(heads=8, kv_heads=2, dim=32, vdim=16, scale=0.8, base=10000.0, dims=16, factor=4.0, chunk=40, ff=128),
              mlstm(heads=2, dim=56, vdim=80, gate_cap=6.0),
              chunked(heads=6, kv_heads=1, dim=64, vdim=32, scale=0.6, base=3000.0, dims=64, factor=1.5, chunk=24, ff=64)]
    return layers + [borrow(layers, 0), borrow(layers, 3)]


# sizes that the matrix kernels take (multiples of 16 and 32), as a model served in bfloat16 has them
ALIGNED = config(_aligned(), width=64, vocab=128)


def random_config(seed: int) -> dict:
    """A configuration drawn at random: two to six layers of both kinds in any order, head counts, sizes, chunks and
    constants of many kinds (sizes the matrix kernels take and sizes they refuse), layers on the tensors of others."""
    import random
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(2, 6)):
        owners = [i for i, l in enumerate(layers) if "weights_of" not in l]
        if owners and rng.random() < 0.25:
            layers.append(borrow(layers, rng.choice(owners)))
        elif rng.random() < 0.5:
            kv, dim = rng.choice([1, 2, 3, 4]), rng.choice([16, 24, 32, 40, 48, 80, 96, 128])
            layers.append(chunked(heads=kv * rng.choice([1, 2, 3, 4, 8]), kv_heads=kv, dim=dim, vdim=rng.choice([16, 20, 32, 48, 72, 96, 128]),
                                  scale=rng.choice([0.3, 0.7, 1.2]), base=rng.choice([5000.0, 80000.0, 2e6]),
                                  dims=rng.choice([dim, dim // 4 * 2, 8, 0]), factor=rng.choice([0, 1.5, 3.0, 20.0]),
                                  chunk=rng.choice([0, 1, 7, 16, 33, 80, 100, 128, 150, 240]), ff=rng.choice([None, 40, 72, 100, 144])))
        else:
            layers.append(mlstm(heads=rng.choice([1, 2, 3, 5, 8]), dim=rng.choice([8, 16, 24, 40, 72, 100, 128, 200]),
                                vdim=rng.choice([8, 16, 32, 40, 64, 112, 128, 176]), gate_cap=rng.choice([1.0, 4.0, 10.0, 30.0]),
                                ff=rng.choice([None, None, 48, 100])))
    return config(layers, width=rng.choice([64, 96, 136, 160, 192, 320]), vocab=rng.choice([100, 257, 384]), eps=rng.choice([1e-6, 1e-5]),
                  residual_mult=rng.choice([0.3, 0.8, 1.0]), logit_softcap=rng.choice([5.0, 20.0, 40.0]), embedding_scale=rng.choice([1.0, 3.0, 8.0]))


def make_weights(cfg: dict, seed: int, dtype=torch.bfloat16, remember: float = 2.0) -> dict:
    """name -> tensor for every tensor of the configuration's model (names and shapes as the engine's model tree lists
    them; the values are the tests' own). remember: the mean of the forget gates' biases."""
    from llmengine.config.registry import architecture_name, parse_config, resolve
    model = resolve(architecture_name(cfg)).build_model(parse_config(cfg))
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, spec in model.named_specs().items():
        shape = tuple(spec.shape)
        if name.endswith("mix.f.b"):
            t = torch.randn(shape, generator=g) * 1.5 + remember
        elif name.endswith("mix.i.b"):
            t = torch.randn(shape, generator=g) * 1.5
        elif len(shape) == 1:
            t = torch.randn(shape, generator=g) * 0.2 + 1.0    # norm weights
        elif name == "embed":
            t = torch.randn(shape, generator=g) * 0.5
        else:
            t = torch.randn(shape, generator=g) * 1.3 / shape[-1] ** 0.5
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
