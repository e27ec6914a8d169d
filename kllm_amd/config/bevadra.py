"""Typed configuration of the Bevadra decoder.

config.json names the architecture in ``architecture`` and gives ``vocab``, ``width``, ``norm``
(``eps``), ``logit_softcap`` and ``layers``: per layer its ``type``, the sizes of its mixer
(``mixer``) and its feed-forward (``mlp``: null for none, or ``kind`` "dense" with ``ff``).

Mixers by ``type``:

``attention``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, optional ``mask`` {``size``}
(without it every earlier position is read) and optional ``kv_from``: the index of an earlier
attention layer whose keys and values this layer reads in place of its own (its KV heads and
sizes of keys and values are that layer's; its mask, scale and everything else are its own).

``latent_attention``: ``heads``, ``dim``, ``rot_dim``, ``vdim``, ``q_rank``, ``kv_rank``, ``scale``,
``rot`` {``dims``, ``base``} and optional ``mask`` {``size``}.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

from .base import ConfigError, KeyReader, ModelConfig

MIXER_TYPES = ("attention", "latent_attention")


def _number(reader: KeyReader, key: str) -> float:
    v = reader.get(key)
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"{reader.where}: '{key}' must be a number, got {v!r}")
    return float(v)


@dataclass(frozen=True)
class GatedAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0                    # 0: every earlier position is read
    kv_from: Optional[int] = None      # reads the keys and values of that layer

    def to_dict(self):
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window:
            out["mask"] = {"size": self.window}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class LatentMixer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float
    window: int = 0

    def to_dict(self):
        out = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "q_rank": self.q_rank,
               "kv_rank": self.kv_rank, "scale": self.scale, "rot": {"dims": self.rot_dim, "base": self.rot_base}}
        if self.window:
            out["mask"] = {"size": self.window}
        return out


@dataclass(frozen=True)
class BevadraLayer:
    type: str
    mixer: object                      # GatedAttention or LatentMixer
    ff: Optional[int] = None           # None: no feed-forward

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(),
                "mlp": {"kind": "dense", "ff": self.ff} if self.ff is not None else None}


def _window(m: KeyReader, at) -> int:
    return KeyReader(m.get("mask"), at + ".mask").positive_int("size") if m.has("mask") else 0


def _mixer(kind, raw, at, index):
    m = KeyReader(raw, at)
    heads, dim = m.positive_int("heads"), m.positive_int("dim")
    if kind == "attention":
        kv = m.positive_int("kv_heads", heads)
        if heads % kv:
            raise ConfigError(f"{at}: {heads} heads are not a multiple of {kv} kv_heads")
        source = None
        if m.has("kv_from"):
            source = m.get("kv_from")
            if isinstance(source, bool) or not isinstance(source, int) or not 0 <= source < index:
                raise ConfigError(f"{at}: 'kv_from' must name an earlier layer, got {source!r}")
        return GatedAttention(heads, kv, dim, m.positive_int("vdim", dim), _number(m, "scale"), _window(m, at), source)
    rot_dim = m.positive_int("rot_dim")
    rot = KeyReader(m.get("rot"), at + ".rot")
    if rot_dim % 2 or rot.positive_int("dims", rot_dim) != rot_dim:
        raise ConfigError(f"{at}: rot.dims {rot.get('dims', rot_dim)} must be rot_dim {rot_dim}, an even number")
    return LatentMixer(heads, dim, rot_dim, m.positive_int("vdim"), m.positive_int("q_rank"), m.positive_int("kv_rank"),
                       _number(m, "scale"), rot.positive_float("base"), _window(m, at))


@dataclass(frozen=True)
class BevadraConfig(ModelConfig):
    vocab: int = 0
    width: int = 0
    layers: Tuple[BevadraLayer, ...] = ()
    norm_eps: float = 1e-5
    logit_softcap: float = 0.0

    @classmethod
    def from_dict(cls, raw: dict, where: str = "config.json") -> "BevadraConfig":
        r = KeyReader(raw, where)
        vocab, width = r.positive_int("vocab"), r.positive_int("width")
        eps = KeyReader(r.get("norm"), where + ":norm").positive_float("eps")
        cap = r.positive_float("logit_softcap")
        entries = r.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError(f"{where}: 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(entries):
            at = f"{where}:layers[{i}]"
            e = KeyReader(entry, at)
            kind = e.get("type")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{at}: type {kind!r} is not one of {MIXER_TYPES}")
            mixer = _mixer(kind, e.get("mixer"), at + ".mixer", i)
            ff = None
            if e.has("mlp"):
                mlp = KeyReader(entry["mlp"], at + ".mlp")
                if mlp.get("kind", "dense") != "dense":
                    raise ConfigError(f"{at}.mlp: kind {mlp.get('kind')!r} is not 'dense'")
                ff = mlp.positive_int("ff")
            layers.append(BevadraLayer(kind, mixer, ff))
        for i, layer in enumerate(layers):
            source = getattr(layer.mixer, "kv_from", None)
            if source is None:
                continue
            at, other = f"{where}:layers[{i}].mixer", layers[source]
            if other.type != "attention" or other.mixer.kv_from is not None:
                raise ConfigError(f"{at}: 'kv_from' names layer {source}, which has no keys and values of its own")
            if (other.mixer.kv_heads, other.mixer.dim, other.mixer.vdim) != (layer.mixer.kv_heads, layer.mixer.dim,
                                                                             layer.mixer.vdim):
                raise ConfigError(f"{at}: a layer that reads layer {source}'s keys and values has its kv_heads, dim and vdim")
        return cls(architecture="Bevadra", vocab=vocab, width=width, layers=tuple(layers), norm_eps=eps, logit_softcap=cap)

    def to_dict(self) -> dict:
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                "norm": {"eps": self.norm_eps}, "logit_softcap": self.logit_softcap,
                "layers": [layer.to_dict() for layer in self.layers]}
