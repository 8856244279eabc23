"""Typed configuration of Tesopel, read from its config.json.

The file is nested: `architecture`, `vocab`, `width`, `norm.eps`, `logit_scale` and `layers`, a list whose entries
carry `type` (which mixer: `latent_attention`, `mlstm` or `retention`), the mixer's sizes and constants under
`mixer`, and the feed-forward under `mlp` (`kind` = `dense` with `ff` and `limit`), or null for a layer without one.
A latent attention has `heads`, `dim`, `vdim`, `kv_rank`, `scale`, `mask.size` (the window) and, if it expands an
earlier layer's compressed vectors instead of its own, `kv_from`, that layer's number; the two recurrent mixers are
Lefisun's, key for key.  Every layer carries its own sizes, so two layers of one model may differ in all of them
(a layer and the one it names under `kv_from` agree in `kv_rank`), and the order of the mixers is the file's.  A key
the design needs and the file lacks is an error; a key this code does not read is named in a warning
(`UnknownConfigKey`).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

from wllm_amd.architectures.duvozen_config import _any_number
from wllm_amd.architectures.lefisun_config import LefisunMemory, LefisunRetention
from wllm_amd.architectures.tasosun_config import _number, _positive_int, _section
from wllm_amd.config.registry import ConfigError

MIXER_TYPES = ("latent_attention", "mlstm", "retention")


@dataclass(frozen=True)
class TesopelLatentAttention:
    heads: int
    dim: int                        # query/key size of a head
    vdim: int
    kv_rank: int
    scale: float
    window: Optional[int]           # mask.size: how many keys a query sees, itself among them; None: every earlier one
    kv_from: Optional[int] = None   # the layer whose compressed vectors this one expands; None: its own

    @classmethod
    def from_dict(cls, where: str, raw) -> "TesopelLatentAttention":
        raw = _section(where, raw, ("heads", "dim", "vdim", "kv_rank", "scale"), ("mask", "kv_from"))
        sizes = [_positive_int(f"{where}.{k}", raw[k]) for k in ("heads", "dim", "vdim", "kv_rank")]
        window = None
        if raw.get("mask") is not None:
            window = _positive_int(f"{where}.mask.size", _section(f"{where}.mask", raw["mask"], ("size",))["size"])
        source = raw.get("kv_from")
        if source is not None and (isinstance(source, bool) or not isinstance(source, int) or source < 0):
            raise ConfigError(f"{where}.kv_from must be a layer's number, got {source!r}")
        return cls(*sizes, _number(f"{where}.scale", raw["scale"]), window, source)

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "kv_rank": self.kv_rank, "scale": self.scale}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class TesopelFeedForward:
    ff: int
    limit: float                    # what the gate is held under, and the up projection between -limit and limit

    @classmethod
    def from_dict(cls, where: str, raw) -> "TesopelFeedForward":
        raw = _section(where, raw, ("kind", "ff", "limit"))
        if raw["kind"] != "dense":
            raise ConfigError(f"{where}.kind {raw['kind']!r}: this design's feed-forwards are: dense")
        return cls(_positive_int(f"{where}.ff", raw["ff"]), _number(f"{where}.limit", raw["limit"]))

    def to_dict(self) -> dict:
        return {"kind": "dense", "ff": self.ff, "limit": self.limit}


_MIXERS = {"latent_attention": TesopelLatentAttention, "mlstm": LefisunMemory, "retention": LefisunRetention}


@dataclass(frozen=True)
class TesopelLayer:
    type: str
    mixer: object
    mlp: Optional[TesopelFeedForward]


def _check_source(layers: list, i: int) -> None:
    """A layer that expands another's compressed vectors names an earlier latent attention with vectors of its own,
    of the same size."""
    m, where = layers[i].mixer, f"layers[{i}].mixer"
    j = m.kv_from
    if j >= i or layers[j].type != "latent_attention" or layers[j].mixer.kv_from is not None:
        raise ConfigError(f"{where}.kv_from ({j}) must name an earlier latent_attention layer with vectors of its own")
    if layers[j].mixer.kv_rank != m.kv_rank:
        raise ConfigError(f"{where}.kv_rank ({m.kv_rank}) differs from that of the layer kv_from names ({layers[j].mixer.kv_rank})")


@dataclass(frozen=True)
class TesopelConfig:
    vocab: int
    width: int
    norm_eps: float
    logit_scale: float
    layers: tuple
    raw: Optional[dict] = None

    @classmethod
    def from_dict(cls, raw: dict) -> "TesopelConfig":
        raw = _section("config.json", raw, ("vocab", "width", "norm", "layers"), ("architecture", "architectures", "logit_scale"))
        if not isinstance(raw["layers"], list) or not raw["layers"]:
            raise ConfigError("config.json: layers must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(raw["layers"]):
            where = f"layers[{i}]"
            entry = _section(where, entry, ("type", "mixer"), ("mlp",))
            if entry["type"] not in _MIXERS:
                raise ConfigError(f"{where}.type {entry['type']!r}: this design's mixers are: {', '.join(MIXER_TYPES)}")
            mixer = _MIXERS[entry["type"]].from_dict(f"{where}.mixer", entry["mixer"])
            mlp = TesopelFeedForward.from_dict(f"{where}.mlp", entry["mlp"]) if entry.get("mlp") is not None else None
            layers.append(TesopelLayer(entry["type"], mixer, mlp))
            if getattr(mixer, "kv_from", None) is not None:
                _check_source(layers, i)
        return cls(vocab=_positive_int("vocab", raw["vocab"]), width=_positive_int("width", raw["width"]),
                   norm_eps=_number("norm.eps", _section("norm", raw["norm"], ("eps",))["eps"], positive=False),
                   logit_scale=_any_number("logit_scale", raw["logit_scale"]) if raw.get("logit_scale") is not None else 1.0,
                   layers=tuple(layers), raw=raw)

    def to_dict(self) -> dict:
        """The config.json of this configuration."""
        if self.raw is not None:
            return dict(self.raw)
        return {"architecture": "Tesopel", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "logit_scale": self.logit_scale,
                "layers": [{"type": layer.type, "mixer": layer.mixer.to_dict(),
                            "mlp": None if layer.mlp is None else layer.mlp.to_dict()} for layer in self.layers]}
