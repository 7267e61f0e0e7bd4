"""The Zurolorn architecture's configuration, typed, from its own ``config.json`` keys.

A Zurolorn file gives the width (``width``), the vocabulary (``vocab``), the norms' epsilon
(``norm.eps``), the factors on the token table's rows (``embedding.scale``) and on the logits
(``logit_scale``), its layers one by one (``layers``: each with ``type`` = which mixer, the mixer's
sizes and constants under ``mixer`` and its mixture of experts under ``mlp`` or null) and, under
``loop``, a run of layers that is passed through several times with the same weights. Every size and
constant is read from there; a key this parser does not know raises, because a rule dropped without
a word would load and then compute something else.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .gokolix import Loop
from .llama import UnsupportedModelError
from .radivik import _only

ARCHITECTURE = "Zurolorn"
# No position limit is part of the design; the engine's own ``max_seq_len`` bounds the tables.
MAX_POSITION = 1 << 20


@dataclass(frozen=True)
class LatentAttention:
    """Attention whose keys and values are made from one compressed vector per token; with ``q_rank`` the
    queries come from a compressed vector of their own."""

    heads: int
    dim: int                 # un-rotated query/key dimensions per head
    rot_dim: int             # rotated ones
    vdim: int
    kv_rank: int
    q_rank: int | None
    scale: float
    rot_base: float

    @classmethod
    def from_json(cls, m: Mapping[str, Any], where: str, with_q_rank: bool) -> "LatentAttention":
        _only(m, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot") + (("q_rank",) if with_q_rank else ()), where)
        rot_dim = int(m.get("rot_dim", 0))
        rot = m.get("rot") or {"base": 10000.0, "dims": rot_dim}      # a mixer without a rotated part need not describe a rotation
        _only(rot, ("base", "dims"), where + ".rot")
        if int(rot.get("dims", rot_dim)) != rot_dim or rot_dim % 2 or rot_dim < 0:
            raise UnsupportedModelError(f"{where}: the rotated part is rot_dim = {rot_dim} wide and even; rot.dims says {rot.get('dims')}")
        heads, dim, vdim, rank = int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["kv_rank"])
        q_rank = int(m["q_rank"]) if with_q_rank else None
        if min(heads, vdim, rank, 1 if q_rank is None else q_rank) < 1 or dim < 0 or dim + rot_dim < 1:
            raise UnsupportedModelError(f"{where}: heads {heads}, dim {dim}, vdim {vdim}, kv_rank {rank}, q_rank {q_rank}")
        return cls(heads, dim, rot_dim, vdim, rank, q_rank, float(m["scale"]), float(rot["base"]))

    def to_json(self) -> dict[str, Any]:
        out: dict[str, Any] = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim,
                               "kv_rank": self.kv_rank, "scale": self.scale, "rot": {"base": self.rot_base, "dims": self.rot_dim}}
        if self.q_rank is not None:
            out["q_rank"] = self.q_rank
        return out


MIXERS = {"latent_attention": False, "latent_attention_2": True}      # type -> whether its queries have a latent


@dataclass(frozen=True)
class Experts:
    experts: int
    top: int
    ff: int                              # inner size of one expert
    scale: float                         # factor on the chosen scores
    groups: int | None                   # equal groups of neighbouring experts; None: all can be chosen
    keep: int | None                     # how many groups can be chosen from

    @classmethod
    def from_json(cls, f: Mapping[str, Any], where: str) -> "Experts":
        if f.get("kind") != "moe":
            raise UnsupportedModelError(f"{where}: feed-forward kind {f.get('kind')!r}; only 'moe' is implemented")
        _only(f, ("kind", "expert", "router"), where)
        _only(f["expert"], ("ff",), where + ".expert")
        r = f["router"]
        _only(r, ("experts", "top", "scale", "groups"), where + ".router")
        experts, top = int(r["experts"]), int(r["top"])
        count = keep = None
        if r.get("groups") is not None:
            _only(r["groups"], ("count", "keep"), where + ".router.groups")
            count, keep = int(r["groups"]["count"]), int(r["groups"]["keep"])
            if not 1 <= count <= 256 or experts % count or not 1 <= keep <= count:
                raise UnsupportedModelError(f"{where}: {experts} experts in {count} groups of which {keep} are kept")
        if not 1 <= top <= (experts if count is None else keep * (experts // count)):
            raise UnsupportedModelError(f"{where}: top {top} of {experts} experts, groups {r.get('groups')}")
        return cls(experts, top, int(f["expert"]["ff"]), float(r.get("scale", 1.0)), count, keep)

    def to_json(self) -> dict[str, Any]:
        router: dict[str, Any] = {"experts": self.experts, "top": self.top, "scale": self.scale}
        if self.groups is not None:
            router["groups"] = {"count": self.groups, "keep": self.keep}
        return {"kind": "moe", "expert": {"ff": self.ff}, "router": router}


@dataclass(frozen=True)
class ZurolornLayer:
    type: str
    mixer: LatentAttention
    mlp: Experts | None


@dataclass(frozen=True)
class ZurolornConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    embedding_scale: float
    logit_scale: float
    layers: tuple[ZurolornLayer, ...]
    loop: Loop | None
    stop_token_ids: frozenset[int] = frozenset()

    @classmethod
    def from_dicts(cls, raw: Mapping[str, Any], gen: Mapping[str, Any] | None = None) -> "ZurolornConfig":
        _only(raw, ("architecture", "architectures", "embedding", "layers", "logit_scale", "loop", "norm", "vocab", "width"), "config.json")
        _only(raw["norm"], ("eps",), "norm")
        emb = raw.get("embedding") or {}
        _only(emb, ("scale",), "embedding")
        layers = []
        for i, entry in enumerate(raw["layers"]):
            where = f"layers[{i}]"
            _only(entry, ("type", "mixer", "mlp"), where)
            kind = entry.get("type")
            if kind not in MIXERS:
                raise UnsupportedModelError(f"{where}: mixer type {kind!r}; implemented: {sorted(MIXERS)}")
            mixer = LatentAttention.from_json(entry["mixer"], where + ".mixer", MIXERS[kind])
            mlp = None if entry.get("mlp") is None else Experts.from_json(entry["mlp"], where + ".mlp")
            layers.append(ZurolornLayer(kind, mixer, mlp))
        loop = None
        if raw.get("loop") is not None:
            lp = raw["loop"]
            _only(lp, ("start", "stop", "times"), "loop")
            loop = Loop(int(lp["start"]), int(lp["stop"]), int(lp["times"]))
            if not 0 <= loop.start < loop.stop <= len(layers) or loop.times < 1:
                raise UnsupportedModelError(f"loop {lp} does not fit {len(layers)} layers")
        return cls(int(raw["vocab"]), int(raw["width"]), float(raw["norm"]["eps"]), float(emb.get("scale", 1.0)),
                   float(raw.get("logit_scale", 1.0)), tuple(layers), loop)

    def to_config_json(self) -> dict[str, Any]:
        out: dict[str, Any] = {
            "architecture": ARCHITECTURE, "embedding": {"scale": self.embedding_scale}, "logit_scale": self.logit_scale,
            "layers": [{"type": l.type, "mixer": l.mixer.to_json(), "mlp": None if l.mlp is None else l.mlp.to_json()}
                       for l in self.layers],
            "norm": {"eps": self.norm_eps}, "vocab": self.vocab_size, "width": self.hidden_size,
        }
        if self.loop is not None:
            out["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        return out
