"""The Durelix architecture's configuration, typed, from its own ``config.json`` keys.

A Durelix file gives the width (``width``), the vocabulary (``vocab``), the norms' epsilon (``norm.eps``), the bigram
embedding (``embedding.bigram``: the number of buckets and the two multipliers of its hash) and its layers one by one
(``layers``: each with ``type`` = which mixer, the mixer's sizes and constants under ``mixer`` and its feed-forward under ``mlp``
or null). Every size and constant is read from there; a key this parser does not know raises, because a rule dropped
without a word would load and then compute something else.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .llama import UnsupportedModelError
from .radivik import _only

ARCHITECTURE = "Durelix"
# No position limit is part of the design; the engine's own ``max_seq_len`` bounds the tables.
MAX_POSITION = 1 << 20


@dataclass(frozen=True)
class Rotary:
    dims: int                # the first that many dimensions of a head rotate
    base: float

    @classmethod
    def from_json(cls, r: Mapping[str, Any] | None, dim: int, where: str) -> "Rotary | None":
        if r is None:
            return None
        _only(r, ("dims", "base"), where)
        dims = int(r["dims"])
        if dims < 0 or dims % 2 or dims > dim:
            raise UnsupportedModelError(f"{where}: {dims} rotating dimensions in a head of {dim} (an even number)")
        return cls(dims, float(r["base"]))

    def to_json(self) -> dict[str, Any]:
        return {"base": self.base, "dims": self.dims}


@dataclass(frozen=True)
class WindowAttention:
    """Grouped-query softmax attention in a sliding window, with short convolutions on q, k and v, a norm per head, a sink
    per head and a gate on the output."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int                # taps
    scale: float
    window: int
    rot: Rotary | None

    @classmethod
    def from_json(cls, m: Mapping[str, Any], where: str) -> "WindowAttention":
        _only(m, ("conv", "dim", "heads", "kv_heads", "mask", "rot", "scale", "vdim"), where)
        _only(m["mask"], ("size",), where + ".mask")
        heads, dim, conv, window = int(m["heads"]), int(m["dim"]), int(m["conv"]), int(m["mask"]["size"])
        kv_heads, vdim = int(m.get("kv_heads", heads)), int(m.get("vdim", dim))
        if heads < 1 or kv_heads < 1 or heads % kv_heads:
            raise UnsupportedModelError(f"{where}: {heads} heads cannot share {kv_heads} key heads")
        if min(dim, vdim, window) < 1 or not 1 <= conv <= 16:
            raise UnsupportedModelError(f"{where}: dim {dim}, vdim {vdim}, window {window}, {conv} taps (1 to 16 are implemented)")
        return cls(heads, kv_heads, dim, vdim, conv, float(m["scale"]), window, Rotary.from_json(m.get("rot"), dim, where + ".rot"))

    def to_json(self) -> dict[str, Any]:
        out: dict[str, Any] = {"conv": self.conv, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                               "mask": {"size": self.window}, "scale": self.scale, "vdim": self.vdim}
        if self.rot is not None:
            out["rot"] = self.rot.to_json()
        return out


@dataclass(frozen=True)
class Retention:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]
    rot: Rotary | None

    @classmethod
    def from_json(cls, m: Mapping[str, Any], where: str) -> "Retention":
        _only(m, ("decay", "dim", "heads", "rot", "vdim"), where)
        heads, dim = int(m["heads"]), int(m["dim"])
        vdim, decay = int(m.get("vdim", dim)), tuple(float(d) for d in m["decay"])
        if heads < 1 or dim < 1 or vdim < 1 or len(decay) != heads:
            raise UnsupportedModelError(f"{where}: {heads} heads of {dim} and {vdim}, {len(decay)} decays")
        return cls(heads, dim, vdim, decay, Rotary.from_json(m.get("rot"), dim, where + ".rot"))

    def to_json(self) -> dict[str, Any]:
        out: dict[str, Any] = {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}
        if self.rot is not None:
            out["rot"] = self.rot.to_json()
        return out


@dataclass(frozen=True)
class SideBySide:
    """Two mixers on the same input."""

    left: WindowAttention
    right: Retention

    @classmethod
    def from_json(cls, m: Mapping[str, Any], where: str) -> "SideBySide":
        _only(m, ("left", "right"), where)
        return cls(WindowAttention.from_json(m["left"], where + ".left"), Retention.from_json(m["right"], where + ".right"))

    def to_json(self) -> dict[str, Any]:
        return {"left": self.left.to_json(), "right": self.right.to_json()}


@dataclass(frozen=True)
class DenseFeedForward:
    ff: int

    def to_json(self) -> dict[str, Any]:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class Experts:
    experts: int
    top: int
    ff: int                              # inner size of one expert
    identity: int                        # identity experts behind the others
    groups: int | None                   # equal groups of neighbours, identity experts among them; None: all can be chosen
    keep: int | None                     # how many groups can be chosen from

    @classmethod
    def from_json(cls, f: Mapping[str, Any], where: str) -> "Experts":
        _only(f, ("kind", "expert", "router"), where)
        _only(f["expert"], ("ff",), where + ".expert")
        r = f["router"]
        _only(r, ("experts", "groups", "identity", "top"), where + ".router")
        experts, top, identity = int(r["experts"]), int(r["top"]), int(r.get("identity", 0))
        count = keep = None
        total = experts + identity
        if experts < 1 or identity < 0:
            raise UnsupportedModelError(f"{where}: {experts} experts and {identity} identity experts")
        if r.get("groups") is not None:
            _only(r["groups"], ("count", "keep"), where + ".router.groups")
            count, keep = int(r["groups"]["count"]), int(r["groups"]["keep"])
            if not 1 <= count <= 256 or total % count or not 1 <= keep <= count:
                raise UnsupportedModelError(f"{where}: {total} experts in {count} groups of which {keep} are kept")
        if not 1 <= top <= (total if count is None else keep * (total // count)):
            raise UnsupportedModelError(f"{where}: top {top} of {total} experts, groups {r.get('groups')}")
        return cls(experts, top, int(f["expert"]["ff"]), identity, count, keep)

    def to_json(self) -> dict[str, Any]:
        router: dict[str, Any] = {"experts": self.experts, "identity": self.identity, "top": self.top}
        if self.groups is not None:
            router["groups"] = {"count": self.groups, "keep": self.keep}
        return {"kind": "moe", "expert": {"ff": self.ff}, "router": router}


def _feed_forward(f: Mapping[str, Any] | None, where: str) -> "DenseFeedForward | Experts | None":
    if f is None:
        return None
    if f.get("kind") == "dense":
        _only(f, ("kind", "ff"), where)
        return DenseFeedForward(int(f["ff"]))
    if f.get("kind") == "moe":
        return Experts.from_json(f, where)
    raise UnsupportedModelError(f"{where}: feed-forward kind {f.get('kind')!r}; implemented: 'dense', 'moe'")


MIXERS = {"parallel": SideBySide}


@dataclass(frozen=True)
class DurelixLayer:
    type: str
    mixer: SideBySide
    mlp: DenseFeedForward | Experts | None


@dataclass(frozen=True)
class Bigram:
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass(frozen=True)
class DurelixConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    bigram: Bigram
    layers: tuple[DurelixLayer, ...]
    stop_token_ids: frozenset[int] = frozenset()

    @classmethod
    def from_dicts(cls, raw: Mapping[str, Any], gen: Mapping[str, Any] | None = None) -> "DurelixConfig":
        _only(raw, ("architecture", "architectures", "embedding", "layers", "norm", "vocab", "width"), "config.json")
        _only(raw["norm"], ("eps",), "norm")
        _only(raw["embedding"], ("bigram",), "embedding")
        b = raw["embedding"]["bigram"]
        _only(b, ("buckets", "mul_cur", "mul_prev"), "embedding.bigram")
        if int(b["buckets"]) < 1 or int(b["mul_cur"]) < 0 or int(b["mul_prev"]) < 0:
            raise UnsupportedModelError(f"embedding.bigram: {dict(b)}")
        layers = []
        for i, entry in enumerate(raw["layers"]):
            where = f"layers[{i}]"
            _only(entry, ("type", "mixer", "mlp"), where)
            kind = entry.get("type")
            if kind not in MIXERS:
                raise UnsupportedModelError(f"{where}: mixer type {kind!r}; implemented: {sorted(MIXERS)}")
            layers.append(DurelixLayer(kind, MIXERS[kind].from_json(entry["mixer"], where + ".mixer"),
                                       _feed_forward(entry.get("mlp"), where + ".mlp")))
        return cls(int(raw["vocab"]), int(raw["width"]), float(raw["norm"]["eps"]),
                   Bigram(int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"])), tuple(layers))

    def to_config_json(self) -> dict[str, Any]:
        return {
            "architecture": ARCHITECTURE,
            "embedding": {"bigram": {"buckets": self.bigram.buckets, "mul_cur": self.bigram.mul_cur, "mul_prev": self.bigram.mul_prev}},
            "layers": [{"type": l.type, "mixer": l.mixer.to_json(), "mlp": None if l.mlp is None else l.mlp.to_json()}
                       for l in self.layers],
            "norm": {"eps": self.norm_eps}, "vocab": self.vocab_size, "width": self.hidden_size,
        }
