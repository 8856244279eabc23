"""Typed configuration of Modasun, read from its config.json.

The file is nested: `architecture`, `vocab`, `width`, `embedding.scale`, `norm.eps`, `postln_alpha` and `layers`, a list
whose entries carry `type` (which mixer: `attention` or `channel_delta`), the mixer's sizes and constants under `mixer`,
and the feed-forward under `mlp` (`kind` = `dense` with `ff`, or `moe` with `expert.ff`, `router` and optionally
`shared.ff`), or null for a layer without one.  An attention has `heads`, `kv_heads`, `dim`, `vdim`, `scale` and
optionally `q_temp` (`coef`, `every`); a channel_delta has `heads`, `kv_heads`, `dim`, `vdim` and `conv` (the taps of its
convolutions; the sizes of its inner projections are the tensors').  An entry with `weights_of` runs another layer's
weights once more; what else it holds must be that layer's.  Every layer carries its own sizes, and the order of the
mixers is the file's.  A key the design needs and the file lacks is an error; a key this code does not read is named
in a warning (`UnknownConfigKey`).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

from wllm_amd.architectures.duvozen_config import _any_number
from wllm_amd.architectures.tasosun_config import _number, _positive_int, _section
from wllm_amd.config.registry import ConfigError

MIXER_TYPES = ("attention", "channel_delta")


def _heads(where: str, raw) -> tuple:
    heads, kv_heads = _positive_int(f"{where}.heads", raw["heads"]), _positive_int(f"{where}.kv_heads", raw["kv_heads"])
    if heads % kv_heads:
        raise ConfigError(f"{where}: heads ({heads}) must be a multiple of kv_heads ({kv_heads})")
    return heads, kv_heads, _positive_int(f"{where}.dim", raw["dim"]), _positive_int(f"{where}.vdim", raw["vdim"])


@dataclass(frozen=True)
class ModasunAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_temp: Optional[tuple] = None      # (coef, every); None: no temperature

    @classmethod
    def from_dict(cls, where: str, raw) -> "ModasunAttention":
        raw = _section(where, raw, ("heads", "kv_heads", "dim", "vdim", "scale"), ("q_temp",))
        temp = None
        if raw.get("q_temp") is not None:
            t = _section(f"{where}.q_temp", raw["q_temp"], ("coef", "every"))
            temp = (_any_number(f"{where}.q_temp.coef", t["coef"]), _positive_int(f"{where}.q_temp.every", t["every"]))
        return cls(*_heads(where, raw), _number(f"{where}.scale", raw["scale"]), temp)

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.q_temp is not None:
            out["q_temp"] = {"coef": self.q_temp[0], "every": self.q_temp[1]}
        return out


@dataclass(frozen=True)
class ModasunDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int

    @classmethod
    def from_dict(cls, where: str, raw) -> "ModasunDelta":
        raw = _section(where, raw, ("heads", "kv_heads", "dim", "vdim", "conv"))
        return cls(*_heads(where, raw), _positive_int(f"{where}.conv", raw["conv"]))

    def to_dict(self) -> dict:
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.taps}


@dataclass(frozen=True)
class ModasunDense:
    ff: int
    kind = "dense"

    @classmethod
    def from_dict(cls, where: str, raw) -> "ModasunDense":
        raw = _section(where, raw, ("kind", "ff"))
        return cls(_positive_int(f"{where}.ff", raw["ff"]))

    def to_dict(self) -> dict:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class ModasunExperts:
    ff: int
    experts: int
    top: int
    groups: int = 1
    keep: int = 1
    shared_ff: Optional[int] = None
    kind = "moe"

    @classmethod
    def from_dict(cls, where: str, raw) -> "ModasunExperts":
        raw = _section(where, raw, ("kind", "expert", "router"), ("shared",))
        ff = _positive_int(f"{where}.expert.ff", _section(f"{where}.expert", raw["expert"], ("ff",))["ff"])
        r = f"{where}.router"
        router = _section(r, raw["router"], ("experts", "top"), ("groups",))
        experts, top = _positive_int(f"{r}.experts", router["experts"]), _positive_int(f"{r}.top", router["top"])
        groups = keep = 1
        if router.get("groups") is not None:
            g = _section(f"{r}.groups", router["groups"], ("count", "keep"))
            groups, keep = _positive_int(f"{r}.groups.count", g["count"]), _positive_int(f"{r}.groups.keep", g["keep"])
        if experts % groups or keep > groups:
            raise ConfigError(f"{r}: groups.count ({groups}) must divide experts ({experts}) and groups.keep ({keep}) be at most "
                              f"groups.count")
        if top > keep * (experts // groups):
            raise ConfigError(f"{r}.top ({top}) is more than the experts of the kept groups ({keep * (experts // groups)})")
        shared = None
        if raw.get("shared") is not None:
            shared = _positive_int(f"{where}.shared.ff", _section(f"{where}.shared", raw["shared"], ("ff",))["ff"])
        return cls(ff, experts, top, groups, keep, shared)

    def to_dict(self) -> dict:
        out = {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.groups != 1:
            out["router"]["groups"] = {"count": self.groups, "keep": self.keep}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


_MIXERS = {"attention": ModasunAttention, "channel_delta": ModasunDelta}
_MLPS = {"dense": ModasunDense, "moe": ModasunExperts}


def _mlp(where: str, raw):
    if raw is None:
        return None
    if not isinstance(raw, dict) or raw.get("kind") not in _MLPS:
        raise ConfigError(f"{where}.kind: this design's feed-forwards are: {', '.join(_MLPS)}; got {raw!r}")
    return _MLPS[raw["kind"]].from_dict(where, raw)


@dataclass(frozen=True)
class ModasunLayer:
    type: str
    mixer: object
    mlp: object                         # None: a layer without a feed-forward
    weights_of: Optional[int] = None    # the layer whose tensors this one uses (one that has its own)


@dataclass(frozen=True)
class ModasunConfig:
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    alpha: float                        # postln_alpha: the stream's weight in the sums that the norms take
    layers: tuple
    raw: Optional[dict] = None

    @classmethod
    def from_dict(cls, raw: dict) -> "ModasunConfig":
        raw = _section("config.json", raw, ("vocab", "width", "norm", "layers", "embedding", "postln_alpha"),
                       ("architecture", "architectures"))
        if not isinstance(raw["layers"], list) or not raw["layers"]:
            raise ConfigError("config.json: layers must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(raw["layers"]):
            where = f"layers[{i}]"
            entry = _section(where, entry, ("type", "mixer"), ("mlp", "weights_of"))
            if entry["type"] not in _MIXERS:
                raise ConfigError(f"{where}.type {entry['type']!r}: this design's mixers are: {', '.join(MIXER_TYPES)}")
            mixer = _MIXERS[entry["type"]].from_dict(f"{where}.mixer", entry["mixer"])
            layer = ModasunLayer(entry["type"], mixer, _mlp(f"{where}.mlp", entry.get("mlp")))
            source = entry.get("weights_of")
            if source is not None:
                if isinstance(source, bool) or not isinstance(source, int) or not 0 <= source < i:
                    raise ConfigError(f"{where}.weights_of must be the number of an earlier layer, got {source!r}")
                if layers[source].weights_of is not None:       # a layer that itself uses another's
                    source = layers[source].weights_of
                theirs = layers[source]
                if (layer.type, layer.mixer, layer.mlp) != (theirs.type, theirs.mixer, theirs.mlp):
                    raise ConfigError(f"{where}.weights_of: the entry differs from layer {source}, whose weights it uses")
                layer = ModasunLayer(layer.type, layer.mixer, layer.mlp, source)
            layers.append(layer)
        return cls(vocab=_positive_int("vocab", raw["vocab"]), width=_positive_int("width", raw["width"]),
                   embedding_scale=_any_number("embedding.scale", _section("embedding", raw["embedding"], ("scale",))["scale"]),
                   norm_eps=_number("norm.eps", _section("norm", raw["norm"], ("eps",))["eps"], positive=False),
                   alpha=_any_number("postln_alpha", raw["postln_alpha"]), layers=tuple(layers), raw=raw)

    def to_dict(self) -> dict:
        """The config.json of this configuration."""
        if self.raw is not None:
            return dict(self.raw)
        layers = []
        for layer in self.layers:
            entry = {"type": layer.type, "mixer": layer.mixer.to_dict(), "mlp": None if layer.mlp is None else layer.mlp.to_dict()}
            if layer.weights_of is not None:
                entry["weights_of"] = layer.weights_of
            layers.append(entry)
        return {"architecture": "Modasun", "vocab": self.vocab, "width": self.width, "embedding": {"scale": self.embedding_scale},
                "norm": {"eps": self.norm_eps}, "postln_alpha": self.alpha, "layers": layers}
