"""DiporaxConfig: the typed view of a Diporax config.json.

The file names the vocabulary ("vocab"), the residual width ("width"), the norms' epsilon ("norm": {"eps"}), the entries a
layer takes from the per-token table ("token_side": {"dim"}) and a list "layers", one entry per layer: "type" (which mixer),
"mixer" (its sizes and constants) and "mlp" (the feed-forward: "kind" "moe" with "router" {"experts", "top"}, "expert" {"ff"}
and optionally "shared" {"ff"}; null for a layer without one).

Mixer of type "latent_attention": "heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "scale", "rot". Mixer of type
"lightning": "heads", "dim", "vdim", "decay" (a number a head). Mixer of type "attention": "heads", "kv_heads", "dim", "vdim",
"scale", "softcap", "conv" (taps), "rot", "v_mix". "rot" is {"base", "dims", "scaling" {"factor", "original", "fast", "slow"}}.
Nothing else is read. The design has no longest position and no end-of-sequence token.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Mapping

from .base import ConfigError, KeyReader

MIXER_TYPES = ("latent_attention", "lightning", "attention")


@dataclass(frozen=True)
class DiporaxLayer:
    type: str
    mixer: Mapping[str, Any]            # the mixer's sizes and constants, checked, as plain values
    mlp: Mapping[str, Any] | None       # {"experts", "top", "ff", "shared_ff"}; None for a layer without a feed-forward


def _rotation(m: KeyReader, entries: int) -> dict | None:
    """`entries`: how many of a head's entries may turn."""
    rot = m.mapping("rot")
    if rot is None:
        return None
    out = {"dims": rot.integer("dims", minimum=0), "base": rot.number("base"), "scaling": None}
    if out["dims"] % 2 or out["dims"] > entries:
        raise ConfigError(f"{rot.where}: dims={out['dims']} must be even and at most {entries}")
    if out["base"] <= 0:
        raise ConfigError(f"{rot.where}: base must be > 0")
    sc = rot.mapping("scaling")
    if sc is not None:
        out["scaling"] = {k: sc.number(k) for k in ("factor", "original", "fast", "slow")}
        if min(out["scaling"].values()) <= 0:
            raise ConfigError(f"{sc.where}: factor, original, fast and slow must be > 0")
        if out["base"] == 1:
            raise ConfigError(f"{rot.where}: base must not be 1 with scaling")
    return out


def _sizes(m: KeyReader, *names: str) -> dict:
    return {k: m.integer(k, minimum=1) for k in names}


def _latent(m: KeyReader) -> dict:
    out = _sizes(m, "heads", "dim", "vdim", "kv_rank", "q_rank")
    out["scale"], out["rot_dim"] = m.number("scale"), m.integer("rot_dim", 0, minimum=0)
    if out["rot_dim"] % 2:
        raise ConfigError(f"{m.where}: rot_dim={out['rot_dim']} must be even")
    out["rot"] = _rotation(m, out["rot_dim"]) if out["rot_dim"] else None
    if out["rot_dim"] and out["rot"] is None:
        raise ConfigError(f"{m.where}: rot_dim={out['rot_dim']} needs 'rot'")
    return out


def _lightning(m: KeyReader) -> dict:
    out = _sizes(m, "heads", "dim", "vdim")
    decay = m.data.get("decay")
    if not isinstance(decay, list) or len(decay) != out["heads"] or any(isinstance(a, bool) or not isinstance(a, (int, float)) for a in decay):
        raise ConfigError(f"{m.where}: key 'decay' must be a list of {out['heads']} numbers, one a head")
    out["decay"] = tuple(float(a) for a in decay)
    if not all(0.0 <= a <= 1.0 for a in out["decay"]):
        raise ConfigError(f"{m.where}: key 'decay' must hold numbers between 0 and 1")
    return out


def _attention(m: KeyReader) -> dict:
    out = _sizes(m, "heads", "kv_heads", "dim", "vdim")
    if out["heads"] % out["kv_heads"]:
        raise ConfigError(f"{m.where}: heads={out['heads']} is no multiple of kv_heads={out['kv_heads']}")
    out.update(scale=m.number("scale"), softcap=m.number("softcap", 0.0), conv=m.integer("conv", 0, minimum=0),
               v_mix=m.boolean("v_mix", False), rot=_rotation(m, out["dim"]))
    if out["softcap"] < 0:
        raise ConfigError(f"{m.where}: softcap must be > 0")
    return out


_MIXERS = {"latent_attention": _latent, "lightning": _lightning, "attention": _attention}


def _mlp(r: KeyReader) -> dict | None:
    mlp = r.mapping("mlp")
    if mlp is None:
        return None
    kind = mlp.string("kind")
    if kind != "moe":
        raise ConfigError(f"{mlp.where}: kind {kind!r} is not 'moe'")
    router, expert, shared = mlp.mapping("router"), mlp.mapping("expert"), mlp.mapping("shared")
    if router is None or expert is None:
        raise ConfigError(f"{mlp.where}: a mixture of experts needs 'router' and 'expert'")
    out = {"experts": router.integer("experts", minimum=1), "top": router.integer("top", minimum=1),
           "ff": expert.integer("ff", minimum=1), "shared_ff": shared.integer("ff", minimum=1) if shared is not None else None}
    if out["top"] > out["experts"]:
        raise ConfigError(f"{router.where}: top={out['top']} is more than experts={out['experts']}")
    return out


@dataclass(frozen=True)
class DiporaxConfig:
    architecture: str
    vocab_size: int
    width: int
    norm_eps: float
    token_dim: int                      # entries a layer takes from the per-token table; 0: the model has none
    layers: tuple[DiporaxLayer, ...]
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
                  architecture: str = "Diporax") -> "DiporaxConfig":
        r = KeyReader(cfg)
        norm = r.mapping("norm")
        if norm is None:
            raise ConfigError("config.json: required key 'norm' is missing")
        raw = cfg.get("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError("config.json: key 'layers' must be a non-empty list")
        layers: list[DiporaxLayer] = []
        first = None                    # the first layer whose values the other mixing layers take
        for i, entry in enumerate(raw):
            lr = KeyReader(entry, f"config.json:layers[{i}]")
            kind = lr.string("type")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{lr.where}: mixer type {kind!r} is none of {list(MIXER_TYPES)}")
            m = lr.mapping("mixer")
            if m is None:
                raise ConfigError(f"{lr.where}: required key 'mixer' is missing")
            mixer = _MIXERS[kind](m)
            if mixer.get("v_mix"):
                if first is None:
                    first = mixer
                elif mixer["kv_heads"] * mixer["vdim"] != first["kv_heads"] * first["vdim"]:
                    raise ConfigError(f"{m.where}: kv_heads and vdim must give as many values as the first layer with 'v_mix' has")
            layers.append(DiporaxLayer(kind, mixer, _mlp(lr)))
        side = r.mapping("token_side")
        return cls(architecture=architecture, vocab_size=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                   norm_eps=norm.number("eps"), token_dim=side.integer("dim", minimum=1) if side is not None else 0,
                   layers=tuple(layers))
