"""Typed configuration of the Befirax decoder, read from config.json's own keys.

config.json gives `vocab`, `width`, `norm.eps`, `streams` (the copies of the residual stream) and `layers`, a list whose
entries name the layer's mixer by `type`: "attention" (differential attention behind a short convolution), "latent_attention"
(one latent per token, a sliding window, a gate per head) or "mamba2" (the state-space mixer); the mixer's sizes and
constants in `mixer`; the feed-forward in `mlp`: null or {"kind": "moe", "expert": {"ff"}, "router": {"experts",
"identity", "top"}}.  An attention layer with `kv_from` reads that layer's keys and values.  Layers differ from each
other; nothing about them stands in code.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple, Union

from .kotipel import StateSpaceMixerConfig, _need
from .llama import ConfigError


@dataclass(frozen=True)
class PlainRotConfig:
    base: float
    dims: int

    @staticmethod
    def from_dict(r: Dict[str, Any], where: str) -> "PlainRotConfig":
        _need(r, ("base", "dims"), where)
        c = PlainRotConfig(float(r["base"]), int(r["dims"]))
        if c.dims <= 0 or c.dims % 2 or not c.base > 0:
            raise ConfigError(f"{where}: dims must be positive and even, base positive")
        return c

    def to_dict(self) -> Dict[str, Any]:
        return {"base": self.base, "dims": self.dims}


@dataclass(frozen=True)
class DifferentialAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float
    conv: int
    rot: Optional[PlainRotConfig] = None
    kv_from: Optional[int] = None

    @staticmethod
    def from_dict(m: Dict[str, Any], where: str) -> "DifferentialAttentionConfig":
        _need(m, ("heads", "kv_heads", "dim", "vdim", "scale", "diff"), where)
        rot = PlainRotConfig.from_dict(m["rot"], where + ".rot") if m.get("rot") else None
        src = m.get("kv_from")
        c = DifferentialAttentionConfig(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]),
                                        float(m["diff"]), int(m.get("conv") or 0), rot, None if src is None else int(src))
        if min(c.heads, c.kv_heads, c.dim, c.vdim) <= 0 or c.heads % c.kv_heads or c.conv < 0:
            raise ConfigError(f"{where}: sizes must be positive and heads a multiple of kv_heads")
        if rot is not None and rot.dims > c.dim:
            raise ConfigError(f"{where}.rot.dims={rot.dims} does not fit maps of {c.dim}")
        return c

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"conv": self.conv, "diff": self.diff, "dim": self.dim, "heads": self.heads}
        if self.kv_from is not None:
            d["kv_from"] = self.kv_from
        d["kv_heads"] = self.kv_heads
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        d.update(scale=self.scale, vdim=self.vdim)
        return d


@dataclass(frozen=True)
class WindowedLatentConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: PlainRotConfig
    window: Optional[int] = None

    @staticmethod
    def from_dict(m: Dict[str, Any], where: str) -> "WindowedLatentConfig":
        _need(m, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot"), where)
        rot = PlainRotConfig.from_dict(m["rot"], where + ".rot")
        mask = m.get("mask")
        if mask:
            _need(mask, ("size",), where + ".mask")
        c = WindowedLatentConfig(int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]),
                                 float(m["scale"]), rot, int(mask["size"]) if mask else None)
        if min(c.heads, c.dim, c.rot_dim, c.vdim, c.kv_rank) <= 0:
            raise ConfigError(f"{where}: sizes must be positive")
        if rot.dims != c.rot_dim:
            raise ConfigError(f"{where}: the rotation takes the whole rotated part: rot.dims={rot.dims}, rot_dim={c.rot_dim}")
        if c.window is not None and c.window <= 0:
            raise ConfigError(f"{where}.mask.size must be positive")
        return c

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank}
        if self.window is not None:
            d["mask"] = {"size": self.window}
        d.update(rot=self.rot.to_dict(), rot_dim=self.rot_dim, scale=self.scale, vdim=self.vdim)
        return d


@dataclass(frozen=True)
class IdentityMoeConfig:
    experts: int
    identity: int
    top: int
    ff: int

    @staticmethod
    def from_dict(mlp: Optional[Dict[str, Any]], where: str) -> Optional["IdentityMoeConfig"]:
        if mlp is None:
            return None
        kind = mlp.get("kind") if isinstance(mlp, dict) else None
        if kind != "moe":
            raise ConfigError(f"{where}.kind={kind!r} is not supported (known: 'moe')")
        _need(mlp, ("expert", "router"), where)
        _need(mlp["expert"], ("ff",), where + ".expert")
        _need(mlp["router"], ("experts", "top"), where + ".router")
        r = mlp["router"]
        c = IdentityMoeConfig(int(r["experts"]), int(r.get("identity") or 0), int(r["top"]), int(mlp["expert"]["ff"]))
        if c.ff <= 0 or c.experts <= 0 or c.identity < 0 or not 0 < c.top <= c.experts + c.identity:
            raise ConfigError(f"{where}: widths must be positive and top within the number of experts")
        return c

    def to_dict(self) -> Dict[str, Any]:
        return {"expert": {"ff": self.ff}, "kind": "moe",
                "router": {"experts": self.experts, "identity": self.identity, "top": self.top}}


Mixer = Union[DifferentialAttentionConfig, WindowedLatentConfig, StateSpaceMixerConfig]
_TYPES = {DifferentialAttentionConfig: "attention", WindowedLatentConfig: "latent_attention", StateSpaceMixerConfig: "mamba2"}


@dataclass(frozen=True)
class BefiraxLayerConfig:
    mixer: Mixer
    mlp: Optional[IdentityMoeConfig]

    @property
    def type(self) -> str:
        return _TYPES[type(self.mixer)]

    def to_dict(self) -> Dict[str, Any]:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


@dataclass(frozen=True)
class BefiraxConfig:
    vocab: int
    width: int
    eps: float
    streams: int
    layers: Tuple[BefiraxLayerConfig, ...]

    architecture = "Befirax"

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @staticmethod
    def from_hf_dict(d: Dict[str, Any]) -> "BefiraxConfig":
        _need(d, ("vocab", "width", "norm", "streams", "layers"), "config.json")
        _need(d["norm"], ("eps",), "config.json norm")
        readers = {"attention": DifferentialAttentionConfig.from_dict, "latent_attention": WindowedLatentConfig.from_dict,
                   "mamba2": StateSpaceMixerConfig.from_dict}
        layers: List[BefiraxLayerConfig] = []
        for i, layer in enumerate(d["layers"]):
            where = f"layers[{i}]"
            _need(layer, ("type", "mixer"), where)
            if layer["type"] not in readers:
                raise ConfigError(f"{where}.type={layer['type']!r} is not supported (known: {sorted(readers)})")
            layers.append(BefiraxLayerConfig(readers[layer["type"]](layer["mixer"], where + ".mixer"),
                                             IdentityMoeConfig.from_dict(layer.get("mlp"), where + ".mlp")))
        cfg = BefiraxConfig(int(d["vocab"]), int(d["width"]), float(d["norm"]["eps"]), int(d["streams"]), tuple(layers))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0 or self.eps <= 0 or self.streams <= 0 or not self.layers:
            raise ConfigError("vocab, width, norm.eps and streams must be positive, and there must be layers")
        for i, layer in enumerate(self.layers):
            j = getattr(layer.mixer, "kv_from", None)
            if j is None:
                continue
            where = f"layers[{i}].mixer.kv_from={j}"
            src = self.layers[j].mixer if 0 <= j < i else None
            if not isinstance(src, DifferentialAttentionConfig) or src.kv_from is not None:
                raise ConfigError(f"{where}: an earlier attention layer with keys and values of its own is needed")
            m = layer.mixer
            if (m.heads, m.kv_heads, m.dim, m.vdim, m.rot) != (src.heads, src.kv_heads, src.dim, src.vdim, src.rot):
                raise ConfigError(f"{where}: head counts, head sizes and rotation must be that layer's")

    def to_hf_dict(self) -> Dict[str, Any]:
        return {"architecture": self.architecture, "layers": [l.to_dict() for l in self.layers], "norm": {"eps": self.eps},
                "streams": self.streams, "vocab": self.vocab, "width": self.width}
