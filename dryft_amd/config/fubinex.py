"""Typed configuration of the Fubinex decoder.

A Fubinex ``config.json`` is nested: ``vocab``, ``width``, ``embedding.scale``, ``norm.eps``, ``norm.groups``, and a list
``layers`` whose entries each name a mixer ``type`` with that mixer's sizes under ``mixer`` and a feed-forward under
``mlp`` (or null):

* ``parallel``: ``left`` (attention over chunks: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``; optionally
  ``mask.size`` and ``rot`` with ``dims`` and ``base``), ``right`` (gated linear attention: ``heads``, ``dim``, ``vdim``,
  ``tau``; the rank of the decay's inner projection is the checkpoint tensor's, and ``decay_rank`` says it where there
  is no checkpoint), ``left_scale``, ``right_scale``;
* ``retention``: ``heads``, ``dim``, ``vdim``, ``decay`` (one number per head); optionally ``rot``;
* ``latent_attention``: ``heads``, ``dim``, ``rot_dim``, ``vdim``, ``q_rank``, ``kv_rank``, ``scale``; optionally ``rot``
  with ``scaling`` (``factor``, ``original``, ``fast``, ``slow``), and ``kv_from``: the number of an earlier layer of
  this kind whose cached latent the layer reads instead of one of its own;
* ``mlp``: ``{"kind": "dense", "ff"}``.

Every size and every constant that may differ from model to model is read from the file. Problems are collected into
one ``ConfigError`` with paths like ``layers[2].mixer.rot.scaling.factor``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any

from ..limits import MAX_HEAD_DIM, MAX_LATENT_WIDTH, MAX_LINEAR_STATE, MAX_NORM_GROUPS
from .base import KeyReader

MIXER_TYPES = ("parallel", "retention", "latent_attention")


@dataclass(frozen=True)
class FubinexLayer:
    type: str
    mixer: dict[str, Any]
    mlp: dict[str, Any] | None


@dataclass(frozen=True)
class FubinexConfig:
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    norm_groups: int
    layers: tuple[FubinexLayer, ...]
    raw: tuple[tuple[str, Any], ...] = ()

    architecture = "Fubinex"

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "FubinexConfig":
        r = KeyReader(raw)
        vocab, width = r.integer("vocab"), r.integer("width")
        embedding = _sub(r, "embedding")
        scale = embedding.number("scale", 1.0, positive=False)
        _close(r, embedding, "embedding")
        norm = _sub(r, "norm")
        eps, groups = norm.number("eps"), norm.integer("groups", 1)
        norm.check(groups <= MAX_NORM_GROUPS, f"groups: the norm kernels take at most {MAX_NORM_GROUPS}")
        norm.check(not (groups and width) or width % groups == 0, f"groups: {width} values do not split into {groups} equal parts")
        _close(r, norm, "norm")
        layers_raw = raw.get("layers")
        layers: list[FubinexLayer] = []
        if not isinstance(layers_raw, list) or not layers_raw:
            r.problems.append("layers: expected a non-empty list")
            layers_raw = []
        for i, entry in enumerate(layers_raw):
            where = f"layers[{i}]"
            if not isinstance(entry, dict) or entry.get("type") not in MIXER_TYPES or not isinstance(entry.get("mixer"), dict):
                r.problems.append(f"{where}: expected an object with type (one of {list(MIXER_TYPES)}) and mixer")
                layers.append(FubinexLayer("", {}, None))
                continue
            m = KeyReader(entry["mixer"])
            mixer = _READERS[entry["type"]](m)
            _close(r, m, f"{where}.mixer")
            mlp = None
            if entry.get("mlp") is not None:
                f = _sub(KeyReader(entry), "mlp")
                kind = f.raw.get("kind")
                f.check(kind == "dense", f"kind: expected 'dense', got {kind!r}")
                mlp = {"kind": "dense", "ff": f.integer("ff")}
                _close(r, f, f"{where}.mlp")
            layers.append(FubinexLayer(entry["type"], mixer, mlp))
        for i, layer in enumerate(layers):
            j = layer.mixer.get("kv_from")
            if j is None:
                continue
            lender = layers[j] if 0 <= j < i else None
            if lender is None or lender.type != "latent_attention" or lender.mixer.get("kv_from") is not None:
                r.problems.append(f"layers[{i}].mixer.kv_from: layer {j} is no earlier latent_attention layer with a latent of its own")
                continue
            for key in ("kv_rank", "rot_dim", "rot"):
                r.check(lender.mixer[key] == layer.mixer[key],
                        f"layers[{i}].mixer.{key}: differs from that of layer {j}, whose latent this layer reads")
        r.finish("unsupported or malformed Fubinex config.json")
        return cls(vocab, width, scale, eps, groups, tuple(layers), tuple(raw.items()))

    def to_dict(self) -> dict[str, Any]:
        if self.raw:
            return dict(self.raw)
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                "embedding": {"scale": self.embedding_scale}, "norm": {"eps": self.norm_eps, "groups": self.norm_groups},
                "layers": [{"type": l.type, "mixer": l.mixer, "mlp": l.mlp} for l in self.layers]}


def _sub(r: KeyReader, key: str, optional: bool = False) -> KeyReader | None:
    value = r.raw.get(key)
    if value is None and optional:
        return None
    if not isinstance(value, dict):
        r.problems.append(f"{key}: expected an object")
        value = {}
    return KeyReader(value)


def _close(r: KeyReader, inner: KeyReader, where: str) -> None:
    r.problems += [f"{where}.{p}" for p in inner.problems]


def _rotation(m: KeyReader, width: int, what: str, scalable: bool = False) -> dict[str, Any] | None:
    """``{dims, base, scaling}``, or None for a mixer that does not rotate."""
    rot = _sub(m, "rot", optional=True)
    if rot is None:
        return None
    dims, base = rot.integer("dims", minimum=0), rot.number("base")
    rot.check(dims % 2 == 0 and dims <= width, f"dims: must be even and at most {what} ({width}), got {dims}")
    scaling = None
    sc = _sub(rot, "scaling", optional=True)
    if sc is not None:
        rot.check(scalable, "scaling: this mixer's rotation has none")
        scaling = {k: sc.number(k) for k in ("factor", "original", "fast", "slow")}
        _close(rot, sc, "scaling")
    _close(m, rot, "rot")
    return {"dims": dims, "base": base, "scaling": scaling} if dims else None


def _read_left(m: KeyReader) -> dict[str, Any]:
    out: dict[str, Any] = {k: m.integer(k) for k in ("heads", "kv_heads", "dim", "vdim")}
    out["scale"] = m.number("scale", positive=False)
    if out["heads"] and out["kv_heads"]:
        m.check(out["heads"] % out["kv_heads"] == 0, f"heads ({out['heads']}) is not a multiple of kv_heads ({out['kv_heads']})")
    m.check(max(out["dim"], out["vdim"]) <= MAX_HEAD_DIM, f"dim, vdim: the attention kernels take at most {MAX_HEAD_DIM}")
    out["mask"] = None
    mask = _sub(m, "mask", optional=True)
    if mask is not None:
        out["mask"] = {"size": mask.integer("size")}
        _close(m, mask, "mask")
    out["rot"] = _rotation(m, out["dim"], "dim")
    return out


def _linear_sizes(m: KeyReader) -> dict[str, Any]:
    out: dict[str, Any] = {k: m.integer(k) for k in ("heads", "dim", "vdim")}
    m.check(max(out["dim"], out["vdim"]) <= MAX_LINEAR_STATE, f"dim, vdim: the kernels take at most {MAX_LINEAR_STATE}")
    return out


def _read_right(m: KeyReader) -> dict[str, Any]:
    out = _linear_sizes(m)
    out["tau"] = m.number("tau")
    out["decay_rank"] = m.integer("decay_rank") if m.raw.get("decay_rank") is not None else None
    return out


def _read_parallel(m: KeyReader) -> dict[str, Any]:
    out: dict[str, Any] = {}
    for side, read in (("left", _read_left), ("right", _read_right)):
        inner = _sub(m, side)
        out[side] = read(inner)
        _close(m, inner, side)
    out["left_scale"], out["right_scale"] = m.number("left_scale", positive=False), m.number("right_scale", positive=False)
    return out


def _read_retention(m: KeyReader) -> dict[str, Any]:
    out = _linear_sizes(m)
    decay = m.raw.get("decay")
    numbers = isinstance(decay, list) and all(isinstance(d, (int, float)) and not isinstance(d, bool) for d in decay)
    if not numbers or len(decay) != out["heads"] or not all(0.0 < d <= 1.0 for d in decay):
        m.problems.append(f"decay: expected {out['heads']} numbers in (0, 1], one per head, got {decay!r}")
        decay = []
    out["decay"] = [float(d) for d in decay]
    out["rot"] = _rotation(m, out["dim"], "dim")
    return out


def _read_latent(m: KeyReader) -> dict[str, Any]:
    out: dict[str, Any] = {k: m.integer(k) for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")}
    out["scale"] = m.number("scale", positive=False)
    m.check(max(out["dim"] + out["rot_dim"], out["vdim"]) <= MAX_HEAD_DIM,
            f"dim + rot_dim, vdim: the attention kernels take at most {MAX_HEAD_DIM}")
    m.check(out["kv_rank"] + out["rot_dim"] <= MAX_LATENT_WIDTH,
            f"kv_rank + rot_dim: the attention kernels take at most {MAX_LATENT_WIDTH}")
    out["rot"] = _rotation(m, out["rot_dim"], "rot_dim", scalable=True)
    out["kv_from"] = m.integer("kv_from", minimum=0) if m.raw.get("kv_from") is not None else None
    return out


_READERS = {"parallel": _read_parallel, "retention": _read_retention, "latent_attention": _read_latent}
__all__ = ["FubinexConfig", "FubinexLayer"]
