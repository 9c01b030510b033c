"""LukupelConfig: the typed view of a Lukupel config.json.

The file names the vocabulary ("vocab"), the residual width ("width"), a multiplier on the embedding ("embedding":
{"scale"}), the norms' epsilon ("norm": {"eps"}), a multiplier on what a sublayer adds to the residual ("residual_mult"), a
soft cap on the logits ("logit_softcap") and a list "layers", one entry per layer: "type" (which mixer), "mixer" (its sizes
and constants), "mlp" (the feed-forward: "kind" "dense" with "ff"; null for a layer without one) and optionally
"weights_of" (the layer whose tensors this one runs on; the rest of the entry equals that layer's).

Mixer of type "attention": "heads", "kv_heads", "dim", "vdim", "scale", "rot" {"base", "dims", "scaling" {"factor"}}, "mask"
{"size"} (the length of a chunk). Mixer of type "mlstm": "heads", "dim", "vdim", "gate_cap". Nothing else is read. The design
has no longest position and no end-of-sequence token.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Mapping

from .base import ConfigError, KeyReader

MIXER_TYPES = ("attention", "mlstm")


@dataclass(frozen=True)
class LukupelLayer:
    type: str
    mixer: Mapping[str, Any]            # the mixer's sizes and constants, checked, as plain values
    ff: int | None                      # the feed-forward's size, None for a layer without one
    weights_of: int | None = None       # the layer whose tensors this one runs on (never itself a borrower), None: its own


def _attention(m: KeyReader) -> dict:
    out = {"heads": m.integer("heads", minimum=1), "kv_heads": m.integer("kv_heads", minimum=1), "dim": m.integer("dim", minimum=1),
           "vdim": m.integer("vdim", minimum=1), "scale": m.number("scale"), "rot_dims": 0, "rot_base": 10000.0, "rot_factor": 1.0,
           "chunk": 0}
    if out["heads"] % out["kv_heads"]:
        raise ConfigError(f"{m.where}: heads={out['heads']} is no multiple of kv_heads={out['kv_heads']}")
    rot = m.mapping("rot")
    if rot is not None:
        out["rot_dims"], out["rot_base"] = rot.integer("dims", minimum=0), rot.number("base")
        if out["rot_dims"] % 2 or out["rot_dims"] > out["dim"]:
            raise ConfigError(f"{rot.where}: dims={out['rot_dims']} must be even and at most dim={out['dim']}")
        if out["rot_base"] <= 0:
            raise ConfigError(f"{rot.where}: base must be > 0")
        sc = rot.mapping("scaling")
        if sc is not None:
            out["rot_factor"] = sc.number("factor")
            if out["rot_factor"] <= 0:
                raise ConfigError(f"{sc.where}: factor must be > 0")
    mask = m.mapping("mask")
    if mask is not None:
        out["chunk"] = mask.integer("size", minimum=1)
    return out


def _mlstm(m: KeyReader) -> dict:
    out = {"heads": m.integer("heads", minimum=1), "dim": m.integer("dim", minimum=1), "vdim": m.integer("vdim", minimum=1),
           "gate_cap": m.number("gate_cap")}
    if out["gate_cap"] <= 0:
        raise ConfigError(f"{m.where}: gate_cap must be > 0")
    return out


def _ff(r: KeyReader) -> int | None:
    mlp = r.mapping("mlp")
    if mlp is None:
        return None
    kind = mlp.string("kind")
    if kind != "dense":
        raise ConfigError(f"{mlp.where}: kind {kind!r} is not 'dense'")
    return mlp.integer("ff", minimum=1)


@dataclass(frozen=True)
class LukupelConfig:
    architecture: str
    vocab_size: int
    width: int
    embedding_scale: float
    norm_eps: float
    residual_mult: float
    logit_softcap: float                # 0: none
    layers: tuple[LukupelLayer, ...]
    eos_token_ids: tuple[int, ...] = field(default_factory=tuple)

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def max_pos(self) -> int:
        """Positions are not limited by the design (angles are computed from the position)."""
        return 1 << 30

    @classmethod
    def from_dict(cls, cfg: Mapping[str, Any], generation_cfg: Mapping[str, Any] | None = None,
                  architecture: str = "Lukupel") -> "LukupelConfig":
        r = KeyReader(cfg)
        norm = r.mapping("norm")
        if norm is None:
            raise ConfigError("config.json: required key 'norm' is missing")
        raw = cfg.get("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError("config.json: key 'layers' must be a non-empty list")
        parsed: list[tuple] = []
        for i, entry in enumerate(raw):
            lr = KeyReader(entry, f"config.json:layers[{i}]")
            kind = lr.string("type")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{lr.where}: mixer type {kind!r} is none of {list(MIXER_TYPES)}")
            m = lr.mapping("mixer")
            if m is None:
                raise ConfigError(f"{lr.where}: required key 'mixer' is missing")
            lender = lr.integer("weights_of", minimum=0) if lr.has("weights_of") else None
            parsed.append((lr.where, kind, _attention(m) if kind == "attention" else _mlstm(m), _ff(lr), lender))
        layers: list[LukupelLayer] = []
        for i, (where, kind, mixer, ff, lender) in enumerate(parsed):
            passed = {i}
            while lender is not None:
                if lender >= len(parsed) or lender in passed:
                    raise ConfigError(f"{where}: weights_of={lender} names no layer with tensors of its own")
                passed.add(lender)
                if parsed[lender][4] is None:
                    break
                lender = parsed[lender][4]
            if lender is not None and (kind, mixer, ff) != parsed[lender][1:4]:
                raise ConfigError(f"{where}: differs from layer {lender}, on whose tensors it runs (weights_of)")
            layers.append(LukupelLayer(kind, mixer, ff, lender))
        emb = r.mapping("embedding")
        cap = r.number("logit_softcap", 0.0)
        if cap < 0:
            raise ConfigError("config.json: key 'logit_softcap' must be > 0")
        return cls(architecture=architecture, vocab_size=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                   embedding_scale=emb.number("scale", 1.0) if emb is not None else 1.0, norm_eps=norm.number("eps"),
                   residual_mult=r.number("residual_mult", 1.0), logit_softcap=cap, layers=tuple(layers))
