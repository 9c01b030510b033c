"""Lukupel as a list of layers and a schedule: an embedding with a multiplier; layers whose sublayers read the stream itself
and are normed behind, what they add times a constant (x <- x + c norm1(mixer(x)); x <- x + c norm2(ff(x))); a softmax
attention within chunks of the sequence, whose queries and keys are rotated and then divided by their root mean square; a
matrix memory with exponential gates (mLSTM), its state kept per request; a feed-forward down(max(up(x), 0)^2) or none;
softly capped logits from the embedding table itself. A layer that runs on an earlier layer's tensors is that layer a second
time in the schedule, with a cache or state of its own. Tensor names: "embed", "l<i>.norm1", "l<i>.mix.*", "l<i>.norm2",
"l<i>.mlp.*", "final.norm".
"""
from __future__ import annotations

from ..config.lukupel import LukupelConfig, LukupelLayer
from ..config.registry import register_architecture
from ..parts import make_part
from .model import DecoderModel, LayerCall


def lukupel_mixer(cfg: LukupelConfig, layer: LukupelLayer):
    m = layer.mixer
    if layer.type == "attention":
        return make_part("mixer", "window_attention", hidden_size=cfg.width, heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
                         vdim=m["vdim"], scale=m["scale"], rot_dims=m["rot_dims"], rot_base=m["rot_base"],
                         rot_scaling={"factor": m["rot_factor"]} if m["rot_factor"] != 1.0 else None, chunk=m["chunk"],
                         qk_norm="unit", eps=cfg.norm_eps)
    return make_part("mixer", "matrix_memory", hidden_size=cfg.width, heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                     gate_cap=m["gate_cap"], eps=cfg.norm_eps)


def build_lukupel(cfg: LukupelConfig) -> DecoderModel:
    norm = lambda: make_part("norm", "rmsnorm", size=cfg.width, eps=cfg.norm_eps, tensor="")
    layers, numbers, place = [], [], {}
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is not None:
            continue
        place[i] = len(layers)
        numbers.append(i)
        ff = None
        if layer.ff is not None:
            ff = make_part("feed_forward", "squared_relu_mlp", hidden_size=cfg.width, intermediate_size=layer.ff,
                           names={"up": "up", "down": "down"})
        layers.append(make_part("block", "output_norm", mixer=lukupel_mixer(cfg, layer), feed_forward=ff, mixer_norm=norm(),
                                ffn_norm=norm() if ff is not None else None, residual_scale=cfg.residual_mult))
    schedule = [LayerCall(place[i if layer.weights_of is None else layer.weights_of], cache=i) for i, layer in enumerate(cfg.layers)]
    embedding = make_part("embedding", "table", vocab_size=cfg.vocab_size, hidden_size=cfg.width, tensor="",
                          scale=cfg.embedding_scale)
    head = make_part("head", "linear", vocab_size=cfg.vocab_size, hidden_size=cfg.width, tied_to=embedding, tensor="",
                     softcap=cfg.logit_softcap)
    return DecoderModel(cfg, embedding, layers, norm(), head, schedule=schedule, layer_numbers=numbers,
                        names={"embedding": "embed", "layers": "l{}", "final_norm": "final.norm", "head": "head"})


register_architecture("Lukupel", LukupelConfig.from_dict, build_lukupel)
