"""Typed configuration of the Kaditar decoder.

A Kaditar ``config.json`` is nested: ``vocab``, ``width``, ``streams`` (copies of the residual stream that the layers
read from and write to through learned weights), ``norm.eps``, optionally ``logit_softcap``, optionally ``loop``
(``start``, ``stop``, ``times``: the layers from ``start`` up to ``stop``, not included, are gone through ``times`` times),
and a list ``layers`` whose entries each name a mixer ``type`` with that mixer's sizes under ``mixer`` and a feed-forward
under ``mlp`` (or null):

* ``attention``: ``heads``, ``kv_heads``, ``dim`` (one map's query and key), ``vdim``, ``scale``, ``diff``; optionally
  ``mask.size`` (a sliding window) and ``rot`` with ``dims`` and ``base``;
* ``mlp``: ``{"kind": "dense", "ff"}`` or ``{"kind": "moe", "expert": {ff}, "router": {experts, top}, "shared": {ff} |
  null}``.

Every size and every constant that may differ from model to model is read from the file. Problems are collected into
one ``ConfigError`` with paths like ``layers[2].mixer.rot.dims``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any

from ..limits import MAX_EXPERTS, MAX_HEAD_DIM, MAX_STREAMS
from .base import ConfigError, KeyReader, LoopConfig

MIXER_TYPES = ("attention",)


@dataclass(frozen=True)
class KaditarLayer:
    type: str
    mixer: dict[str, Any]
    mlp: dict[str, Any] | None


@dataclass(frozen=True)
class KaditarConfig:
    vocab: int
    width: int
    streams: int
    norm_eps: float
    logit_softcap: float | None
    layers: tuple[KaditarLayer, ...]
    loop: LoopConfig | None
    raw: tuple[tuple[str, Any], ...] = ()

    architecture = "Kaditar"

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "KaditarConfig":
        r = KeyReader(raw)
        vocab, width = r.integer("vocab"), r.integer("width")
        streams = r.integer("streams", default=1)
        r.check(streams <= MAX_STREAMS, f"streams: at most {MAX_STREAMS}, got {streams}")
        softcap = r.number("logit_softcap") if raw.get("logit_softcap") is not None else None
        norm = _sub(r, "norm")
        eps = norm.number("eps")
        r.problems += [f"norm.{p}" for p in norm.problems]
        layers_raw = raw.get("layers")
        layers: list[KaditarLayer] = []
        if not isinstance(layers_raw, list) or not layers_raw:
            r.problems.append("layers: expected a non-empty list")
            layers_raw = []
        for i, entry in enumerate(layers_raw):
            where = f"layers[{i}]"
            if not isinstance(entry, dict) or entry.get("type") not in MIXER_TYPES or not isinstance(entry.get("mixer"), dict):
                r.problems.append(f"{where}: expected an object with type (one of {list(MIXER_TYPES)}) and mixer")
                continue
            m = KeyReader(entry["mixer"])
            mixer = _read_attention(m)
            r.problems += [f"{where}.mixer.{p}" for p in m.problems]
            mlp = entry.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict):
                    r.problems.append(f"{where}.mlp: expected an object or null")
                    mlp = None
                else:
                    f = KeyReader(mlp)
                    mlp = _read_mlp(f)
                    r.problems += [f"{where}.mlp.{p}" for p in f.problems]
            layers.append(KaditarLayer(entry["type"], mixer, mlp))
        loop = LoopConfig.read(r, len(layers_raw))
        r.finish("unsupported or malformed Kaditar config.json")
        return cls(vocab, width, streams, eps, softcap, tuple(layers), loop, tuple(raw.items()))

    def to_dict(self) -> dict[str, Any]:
        if self.raw:
            return dict(self.raw)
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "streams": self.streams,
                "norm": {"eps": self.norm_eps}, "logit_softcap": self.logit_softcap,
                "loop": self.loop.to_dict() if self.loop else None,
                "layers": [{"type": l.type, "mixer": l.mixer, "mlp": l.mlp} for l in self.layers]}


def _sub(r: KeyReader, key: str, optional: bool = False) -> KeyReader | None:
    value = r.raw.get(key)
    if value is None and optional:
        return None
    if not isinstance(value, dict):
        r.problems.append(f"{key}: expected an object")
        value = {}
    return KeyReader(value)


def _read_attention(m: KeyReader) -> dict[str, Any]:
    out: dict[str, Any] = {k: m.integer(k) for k in ("heads", "kv_heads", "dim", "vdim")}
    out["scale"], out["diff"] = m.number("scale"), m.number("diff", positive=False)
    if out["heads"] and out["kv_heads"]:
        m.check(out["heads"] % out["kv_heads"] == 0, f"heads ({out['heads']}) is not a multiple of kv_heads ({out['kv_heads']})")
    m.check(max(out["dim"], out["vdim"]) <= MAX_HEAD_DIM, f"dim, vdim: the attention kernels take at most {MAX_HEAD_DIM}")
    out["mask"] = out["rot"] = None
    mask = _sub(m, "mask", optional=True)
    if mask is not None:
        out["mask"] = {"size": mask.integer("size")}
        m.problems += [f"mask.{p}" for p in mask.problems]
    rot = _sub(m, "rot", optional=True)
    if rot is not None:
        dims, base = rot.integer("dims", minimum=0), rot.number("base")
        rot.check(dims % 2 == 0 and dims <= out["dim"], f"dims: must be even and at most dim ({out['dim']}), got {dims}")
        m.problems += [f"rot.{p}" for p in rot.problems]
        if dims:
            out["rot"] = {"dims": dims, "base": base}
    return out


def _read_mlp(f: KeyReader) -> dict[str, Any] | None:
    kind = f.raw.get("kind")
    if kind == "dense":
        return {"kind": "dense", "ff": f.integer("ff")}
    if kind != "moe":
        f.problems.append(f"kind: expected 'dense' or 'moe', got {kind!r}")
        return None
    out: dict[str, Any] = {"kind": "moe"}
    expert = _sub(f, "expert")
    out["expert"] = {"ff": expert.integer("ff")}
    f.problems += [f"expert.{p}" for p in expert.problems]
    router = _sub(f, "router")
    out["router"] = {"experts": router.integer("experts"), "top": router.integer("top")}
    router.check(out["router"]["top"] <= out["router"]["experts"], "top: more than there are experts")
    router.check(out["router"]["experts"] <= MAX_EXPERTS, f"experts: the router takes at most {MAX_EXPERTS}")
    f.problems += [f"router.{p}" for p in router.problems]
    out["shared"] = None
    shared = _sub(f, "shared", optional=True)
    if shared is not None:
        out["shared"] = {"ff": shared.integer("ff")}
        f.problems += [f"shared.{p}" for p in shared.problems]
    return out


__all__ = ["KaditarConfig", "KaditarLayer", "ConfigError"]
