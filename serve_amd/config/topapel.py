"""Typed configuration of the Topapel decoder, read from config.json's own keys.

config.json gives `vocab`, `width`, `norm.eps`, `embedding.scale`, `logit_scale`, `logit_softcap` and `layers`, a list whose
entries name the layer's mixer by `type`: "attention" (grouped-query attention with biases whose values are its keys,
seen in chunks of `mask.size` positions), "lightning" (a linear attention with one constant `decay` per head) or "mingru" (an
element-wise gated recurrence of `width` channels); the mixer's sizes and constants stand in `mixer`, the feed-forward in
`mlp`: null or {"kind": "dense", "ff"}.  Layers differ from each other; nothing about them stands in code.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple, Union

from .kotipel import _need
from .llama import ConfigError


@dataclass(frozen=True)
class LinearRotConfig:
    """A rotation whose frequencies are divided by `factor` (None: as they are)."""
    base: float
    dims: int
    factor: Optional[float] = None

    @staticmethod
    def from_dict(r: Dict[str, Any], where: str) -> "LinearRotConfig":
        _need(r, ("base", "dims"), where)
        s = r.get("scaling")
        if s:
            _need(s, ("factor",), where + ".scaling")
        c = LinearRotConfig(float(r["base"]), int(r["dims"]), float(s["factor"]) if s else None)
        if c.dims <= 0 or c.dims % 2 or not c.base > 0:
            raise ConfigError(f"{where}: dims must be positive and even, base positive")
        if c.factor is not None and not c.factor > 0:
            raise ConfigError(f"{where}.scaling.factor must be positive")
        return c

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.factor is not None:
            d["scaling"] = {"factor": self.factor}
        return d


@dataclass(frozen=True)
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    chunk: Optional[int] = None
    rot: Optional[LinearRotConfig] = None

    @staticmethod
    def from_dict(m: Dict[str, Any], where: str) -> "ChunkAttentionConfig":
        _need(m, ("heads", "kv_heads", "dim", "scale"), where)
        rot = LinearRotConfig.from_dict(m["rot"], where + ".rot") if m.get("rot") else None
        mask = m.get("mask")
        if mask:
            _need(mask, ("size",), where + ".mask")
        c = ChunkAttentionConfig(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), float(m["scale"]),
                                 int(mask["size"]) if mask else None, rot)
        if min(c.heads, c.kv_heads, c.dim) <= 0 or c.heads % c.kv_heads:
            raise ConfigError(f"{where}: sizes must be positive and heads a multiple of kv_heads")
        if int(m.get("vdim", c.dim)) != c.dim:
            raise ConfigError(f"{where}.vdim={m['vdim']}: the values are the keys and have their size {c.dim}")
        if rot is not None and rot.dims > c.dim:
            raise ConfigError(f"{where}.rot.dims={rot.dims} does not fit heads of {c.dim}")
        if c.chunk is not None and c.chunk <= 0:
            raise ConfigError(f"{where}.mask.size must be positive")
        return c

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads}
        if self.chunk is not None:
            d["mask"] = {"size": self.chunk}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        d.update(scale=self.scale, vdim=self.dim)
        return d


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    @staticmethod
    def from_dict(m: Dict[str, Any], where: str) -> "LightningConfig":
        _need(m, ("heads", "dim", "vdim", "decay"), where)
        c = LightningConfig(int(m["heads"]), int(m["dim"]), int(m["vdim"]), tuple(float(a) for a in m["decay"]))
        if min(c.heads, c.dim, c.vdim) <= 0:
            raise ConfigError(f"{where}: sizes must be positive")
        if len(c.decay) != c.heads or not all(0.0 < a <= 1.0 for a in c.decay):
            raise ConfigError(f"{where}.decay must hold one number in (0, 1] for each of the {c.heads} heads")
        return c

    def to_dict(self) -> Dict[str, Any]:
        return {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}


@dataclass(frozen=True)
class MinGruConfig:
    width: int

    @staticmethod
    def from_dict(m: Dict[str, Any], where: str) -> "MinGruConfig":
        _need(m, ("width",), where)
        c = MinGruConfig(int(m["width"]))
        if c.width <= 0:
            raise ConfigError(f"{where}.width must be positive")
        return c

    def to_dict(self) -> Dict[str, Any]:
        return {"width": self.width}


MIXERS = {"attention": ChunkAttentionConfig, "lightning": LightningConfig, "mingru": MinGruConfig}


@dataclass(frozen=True)
class TopapelLayerConfig:
    mixer: Union[ChunkAttentionConfig, LightningConfig, MinGruConfig]
    ff: Optional[int] = None            # the width of the feed-forward; None: the layer has none

    @property
    def type(self) -> str:
        return next(n for n, cls in MIXERS.items() if isinstance(self.mixer, cls))

    def to_dict(self) -> Dict[str, Any]:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.ff is None else {"ff": self.ff, "kind": "dense"},
                "type": self.type}


@dataclass(frozen=True)
class TopapelConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    logit_scale: float
    logit_softcap: float
    layers: Tuple[TopapelLayerConfig, ...]

    architecture = "Topapel"

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @staticmethod
    def from_hf_dict(d: Dict[str, Any]) -> "TopapelConfig":
        _need(d, ("vocab", "width", "norm", "embedding", "logit_scale", "logit_softcap", "layers"), "config.json")
        _need(d["norm"], ("eps",), "config.json norm")
        _need(d["embedding"], ("scale",), "config.json embedding")
        layers: List[TopapelLayerConfig] = []
        for i, layer in enumerate(d["layers"]):
            where = f"layers[{i}]"
            _need(layer, ("type", "mixer"), where)
            if layer["type"] not in MIXERS:
                raise ConfigError(f"{where}.type={layer['type']!r} is not supported (known: {sorted(MIXERS)})")
            mixer = MIXERS[layer["type"]].from_dict(layer["mixer"], where + ".mixer")
            mlp, ff = layer.get("mlp"), None
            if mlp is not None:
                _need(mlp, ("kind", "ff"), where + ".mlp")
                if mlp["kind"] != "dense":
                    raise ConfigError(f"{where}.mlp.kind={mlp['kind']!r} is not supported (known: 'dense')")
                ff = int(mlp["ff"])
                if ff <= 0:
                    raise ConfigError(f"{where}.mlp.ff must be positive")
            layers.append(TopapelLayerConfig(mixer, ff))
        cfg = TopapelConfig(int(d["vocab"]), int(d["width"]), float(d["norm"]["eps"]), float(d["embedding"]["scale"]),
                            float(d["logit_scale"]), float(d["logit_softcap"]), tuple(layers))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0 or not self.eps > 0 or not self.layers:
            raise ConfigError("vocab, width and norm.eps must be positive, and there must be layers")
        if not self.logit_softcap > 0:
            raise ConfigError("logit_softcap must be positive")

    def to_hf_dict(self) -> Dict[str, Any]:
        return {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
                "layers": [l.to_dict() for l in self.layers], "logit_scale": self.logit_scale,
                "logit_softcap": self.logit_softcap, "norm": {"eps": self.eps}, "vocab": self.vocab, "width": self.width}
