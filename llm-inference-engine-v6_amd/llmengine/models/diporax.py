"""Diporax as a list of layers: a normed embedding; layers whose sublayers read the stream itself and are normed behind, what
they add times a vector (x <- x + a norm1(mixer(x)); x <- x + b norm2(ff(x))), and a third sublayer that brings the layer's own
entries of a per-token table; latent attention with a sink in the softmax and a gate a head; linear attention with a fixed decay
a head (lightning attention); softmax attention over all earlier tokens with biases, short convolutions, normed and rotated
queries and keys, capped scores, values that mix with those of the first such layer and a gate a head; a mixture of experts
weighed by the softmax over the chosen ones, beside a shared expert with a gate of its own. Tensor names: "embed", "embed.norm",
"side.embed", "l<i>.norm1", "l<i>.ls1", "l<i>.mix.*", "l<i>.norm2", "l<i>.ls2", "l<i>.mlp.*", "l<i>.side.*", "final.norm", "head".
"""
from __future__ import annotations

from ..config.diporax import DiporaxConfig, DiporaxLayer
from ..config.registry import register_architecture
from ..parts import TokenInput, TokenTable, make_part
from .model import DecoderModel

_MLP_NAMES = {"gate": "gate", "up": "up", "down": "down"}


def diporax_mixer(cfg: DiporaxConfig, layer: DiporaxLayer, v_mix: str):
    """v_mix: the layer's part in the mixing of values, "first" or "mix" ("": none)."""
    m = layer.mixer
    sizes = dict(hidden_size=cfg.width, heads=m["heads"], dim=m["dim"], vdim=m["vdim"], eps=cfg.norm_eps)
    if layer.type == "latent_attention":
        return make_part("mixer", "latent_attention", **sizes, rot_dim=m["rot_dim"], kv_rank=m["kv_rank"], q_rank=m["q_rank"],
                         scale=m["scale"], rot=m["rot"], sink=True, gate="heads")
    if layer.type == "lightning":
        return make_part("mixer", "lightning_attention", **sizes, decay=m["decay"])
    rot = m["rot"] or {"dims": 0, "base": 1.0, "scaling": None}
    return make_part("mixer", "window_attention", **sizes, kv_heads=m["kv_heads"], scale=m["scale"], rot_dims=rot["dims"],
                     rot_base=rot["base"], rot_scaling=rot["scaling"], softcap=m["softcap"], qk_norm=True, gate="heads", bias=True,
                     conv_taps=m["conv"], v_mix=v_mix)


def diporax_feed_forward(cfg: DiporaxConfig, layer: DiporaxLayer):
    mlp = layer.mlp
    if mlp is None:
        return None
    shared = None
    if mlp["shared_ff"] is not None:
        shared = make_part("feed_forward", "gated_mlp", hidden_size=cfg.width, intermediate_size=mlp["shared_ff"], activation="silu",
                           names=_MLP_NAMES)
    return make_part("feed_forward", "mixture_of_experts", hidden_size=cfg.width, intermediate_size=mlp["ff"], experts=mlp["experts"],
                     top=mlp["top"], renormalize=True, activation="silu", shared=shared, shared_gate=shared is not None)


def build_diporax(cfg: DiporaxConfig) -> DecoderModel:
    norm = lambda: make_part("norm", "rmsnorm", size=cfg.width, eps=cfg.norm_eps, tensor="")
    table = TokenTable(cfg.vocab_size, len(cfg.layers), cfg.token_dim) if cfg.token_dim else None
    layers, mixing = [], 0
    for i, layer in enumerate(cfg.layers):
        v_mix = ""
        if layer.mixer.get("v_mix"):
            v_mix = "mix" if mixing else "first"
            mixing += 1
        ff = diporax_feed_forward(cfg, layer)
        side = TokenInput(cfg.width, table, i, norm()) if table is not None else None
        layers.append(make_part("block", "output_norm", mixer=diporax_mixer(cfg, layer, v_mix), feed_forward=ff, mixer_norm=norm(),
                                ffn_norm=norm() if ff is not None else None, layer_scale=True, token_input=side))
    embedding = make_part("embedding", "table", vocab_size=cfg.vocab_size, hidden_size=cfg.width, tensor="", norm=norm())
    head = make_part("head", "linear", vocab_size=cfg.vocab_size, hidden_size=cfg.width, tensor="")
    return DecoderModel(cfg, embedding, layers, norm(), head, shared={"side": table} if table is not None else None,
                        names={"embedding": "embed", "layers": "l{}", "final_norm": "final.norm", "head": "head"})


register_architecture("Diporax", DiporaxConfig.from_dict, build_diporax)
