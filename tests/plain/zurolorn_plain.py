"""A plain, slow Zurolorn in numpy (float64), whole sequences at a time, one function per
mechanism. It shares no code with the package: it is what the engine is compared with.

Zurolorn is a pre-norm decoder, x <- x + s1 * mixer(n1(x)), x <- x + s2 * experts(n2(x)), where s1
and s2 are learned vectors (one number per coordinate). A layer's mixer is latent attention in one
of two forms: queries straight from the input, a rotation that pairs (i, i + r/2) and a sigmoid gate
on the heads' outputs; or queries through a normed latent of their own and a rotation that pairs
neighbours, without a gate. The feed-forward is a mixture of ungated experts (squared ReLU) chosen
by sigmoid scores inside the best groups of experts. A stretch of layers is passed through several
times with the same weights, a learned row per pass added in front of each pass.

``bf16=True`` rounds what an engine holds in bfloat16 (weights are bfloat16 already; the operands
of products, the projections, the cached vectors) and keeps the rest exact: the yardstick for that
mode."""

from __future__ import annotations

import json
from pathlib import Path

import numpy as np


def load_tensors(folder: Path) -> dict[str, np.ndarray]:
    """Every tensor of model.safetensors as float64, read from the file's own layout: 8 bytes of
    header length, a JSON header, then the data."""
    raw = (Path(folder) / "model.safetensors").read_bytes()
    n = int.from_bytes(raw[:8], "little")
    out = {}
    for name, meta in json.loads(raw[8:8 + n]).items():
        if name == "__metadata__":
            continue
        a, b = meta["data_offsets"]
        buf = raw[8 + n + a: 8 + n + b]
        if meta["dtype"] == "BF16":
            arr = (np.frombuffer(buf, dtype="<u2").astype(np.uint32) << 16).view(np.float32).astype(np.float64)
        elif meta["dtype"] == "F32":
            arr = np.frombuffer(buf, dtype="<f4").astype(np.float64)
        else:
            raise ValueError(f"{name}: dtype {meta['dtype']}")
        out[name] = arr.reshape(meta["shape"])
    return out


def to_bf16(x: np.ndarray) -> np.ndarray:
    """Nearest bfloat16, ties to even, as float64."""
    bits = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32).astype(np.uint64)
    bits = (bits + 0x7FFF + ((bits >> 16) & 1)) & 0xFFFF0000
    return bits.astype(np.uint32).view(np.float32).astype(np.float64)


def exact(x: np.ndarray) -> np.ndarray:
    return x


# ------------------------------------------------------------------ small pieces

def rms_norm(x: np.ndarray, w: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def sigmoid(z: np.ndarray) -> np.ndarray:
    return 1.0 / (1.0 + np.exp(-z))


def frequencies(dims: int, base: float) -> np.ndarray:
    return float(base) ** (-2.0 * np.arange(dims // 2, dtype=np.float64) / max(dims, 1))


def rotate(x: np.ndarray, pos: np.ndarray, base: float, halves: bool) -> np.ndarray:
    """x [T, ..., r] turned by pos x frequency; partners are (i, i + r/2) for ``halves``, else (2i, 2i + 1)."""
    r = x.shape[-1]
    ang = pos.astype(np.float64)[:, None] * frequencies(r, base)[None, :]
    ang = ang.reshape((len(pos),) + (1,) * (x.ndim - 2) + (r // 2,))
    out = np.empty_like(x)
    first, second = (slice(0, r // 2), slice(r // 2, r)) if halves else (slice(0, r, 2), slice(1, r, 2))
    u, v = x[..., first], x[..., second]
    out[..., first] = u * np.cos(ang) - v * np.sin(ang)
    out[..., second] = v * np.cos(ang) + u * np.sin(ang)
    return out


def causal_softmax(scores: np.ndarray) -> np.ndarray:
    """scores [H, T, T] -> weights over the keys j <= i."""
    t = scores.shape[-1]
    s = np.where(np.arange(t)[None, :] <= np.arange(t)[:, None], scores, -np.inf)
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


# ------------------------------------------------------------------ mixers, whole sequences

def latent_queries(h: np.ndarray, w: dict, m: dict, eps: float, rnd=exact) -> np.ndarray:
    """[T, heads, dim + rot_dim]: one product, or through a normed latent where the mixer has one."""
    if "dq" in w:
        c = rnd(rms_norm(rnd(h @ w["dq"].T), w["dq.norm"], eps))
        q = c @ w["uq"].T
    else:
        q = h @ w["q"].T
    return rnd(q).reshape(h.shape[0], m["heads"], m["dim"] + m["rot_dim"])


def latent_keys(h: np.ndarray, pos: np.ndarray, w: dict, m: dict, eps: float, halves: bool, rnd=exact):
    """(compressed vectors [T, kv_rank], the rotated key part all heads share [T, rot_dim]): what a cache holds."""
    down = rnd(h @ w["dkv"].T)
    c = rnd(rms_norm(down[:, : m["kv_rank"]], w["dkv.norm"], eps))
    return c, rnd(rotate(down[:, m["kv_rank"]:], pos, m["rot"]["base"], halves))


def latent_attention(h: np.ndarray, pos: np.ndarray, w: dict, m: dict, eps: float, halves: bool, rnd=exact) -> np.ndarray:
    t, heads, d = h.shape[0], m["heads"], m["dim"]
    q = latent_queries(h, w, m, eps, rnd)
    c, shared = latent_keys(h, pos, w, m, eps, halves, rnd)
    turned = rnd(rotate(q[..., d:], pos, m["rot"]["base"], halves))
    keys = rnd(c @ w["uk"].T).reshape(t, heads, d)
    values = rnd(c @ w["uv"].T).reshape(t, heads, m["vdim"])
    scores = np.empty((heads, t, t))
    for a in range(heads):
        scores[a] = (q[:, a, :d] @ keys[:, a].T + turned[:, a] @ shared.T) * m["scale"]
    p = causal_softmax(scores)
    out = np.concatenate([rnd(p[a] @ values[:, a]) for a in range(heads)], axis=-1)
    if "g" in w:
        out = rnd(out * sigmoid(rnd(h @ w["g"].T)))
    return rnd(out @ w["o"].T)


# ------------------------------------------------------------------ experts

def choose(scores: np.ndarray, top: int, groups: dict | None) -> np.ndarray:
    """The ``top`` experts with the largest scores among those of the best groups (neighbouring experts form
    a group, whose score is the sum of its two largest); the lower index among equals. One token."""
    allowed = np.ones(len(scores), dtype=bool)
    if groups:
        per = len(scores) // groups["count"]
        sums = np.array([np.sort(scores[g * per: (g + 1) * per])[::-1][:2].sum() for g in range(groups["count"])])
        best = np.argsort(-sums, kind="stable")[: groups["keep"]]
        allowed = np.isin(np.arange(len(scores)) // per, best)
    return np.argsort(-np.where(allowed, scores, -np.inf), kind="stable")[:top]


def route(h: np.ndarray, w_router: np.ndarray, r: dict) -> tuple[np.ndarray, np.ndarray]:
    """(chosen experts [T, top], their weights): the chosen scores times the router's scale, not renormalized."""
    s = sigmoid(h @ w_router.T)
    chosen = np.stack([choose(row, r["top"], r.get("groups")) for row in s])
    return chosen, np.take_along_axis(s, chosen, axis=1) * r.get("scale", 1.0)


def choice_margin(scores: np.ndarray, top: int, groups: dict | None) -> float:
    """How far the scores of one token would have to move for another choice: the distance between the last
    kept and the first dropped group, or the last chosen and the first unchosen expert, whichever is less."""
    margin, allowed = np.inf, np.ones(len(scores), dtype=bool)
    if groups:
        per = len(scores) // groups["count"]
        sums = np.sort(scores.reshape(groups["count"], per), axis=1)[:, ::-1][:, :2].sum(1)
        order = np.argsort(-sums, kind="stable")
        if groups["keep"] < groups["count"]:
            margin = sums[order[groups["keep"] - 1]] - sums[order[groups["keep"]]]
        allowed = np.isin(np.arange(len(scores)) // per, order[: groups["keep"]])
    inside = np.sort(scores[allowed])[::-1]
    return float(min(margin, inside[top - 1] - inside[top] if top < len(inside) else np.inf))


def expert(h: np.ndarray, up: np.ndarray, down: np.ndarray, rnd=exact) -> np.ndarray:
    return rnd(np.square(np.maximum(h @ up.T, 0.0))) @ down.T


def mixture(h: np.ndarray, w: dict, r: dict, rnd=exact) -> np.ndarray:
    chosen, weight = route(h, w["router"], r)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(chosen[t], weight[t]):
            out[t] += g * expert(h[t], w[f"e{e}.up"], w[f"e{e}.down"], rnd)
    return out


# ------------------------------------------------------------------ the model

HALVES = {"latent_attention": True, "latent_attention_2": False}


class PlainZurolorn:
    def __init__(self, folder: str | Path, bf16: bool = False) -> None:
        folder = Path(folder)
        self.cfg = json.loads((folder / "config.json").read_text())
        self.w = load_tensors(folder)
        self.eps = float(self.cfg["norm"]["eps"])
        self.rnd = to_bf16 if bf16 else exact
        self.margins: list[np.ndarray] = []      # of every layer run with experts of the last call, [T] each

    def part(self, prefix: str) -> dict:
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def mixer(self, i: int, h: np.ndarray, pos: np.ndarray) -> np.ndarray:
        entry = self.cfg["layers"][i]
        return latent_attention(h, pos, self.part(f"l{i}.mix."), entry["mixer"], self.eps, HALVES[entry["type"]], self.rnd)

    def layer(self, i: int, x: np.ndarray, pos: np.ndarray) -> np.ndarray:
        entry = self.cfg["layers"][i]
        x = x + self.w[f"l{i}.ls1"] * self.mixer(i, self.rnd(rms_norm(x, self.w[f"l{i}.norm1"], self.eps)), pos)
        if entry.get("mlp") is not None:
            h = self.rnd(rms_norm(x, self.w[f"l{i}.norm2"], self.eps))
            w, r = self.part(f"l{i}.mlp."), entry["mlp"]["router"]
            x = x + self.w[f"l{i}.ls2"] * mixture(h, w, r, self.rnd)
            self.margins.append(np.array([choice_margin(s, r["top"], r.get("groups")) for s in sigmoid(h @ w["router"].T)]))
        return x

    def runs(self) -> list[tuple[int, int | None]]:
        """(layer, number of the pass it opens or None) in the order the layers run."""
        n, loop = len(self.cfg["layers"]), self.cfg.get("loop")
        if not loop:
            return [(i, None) for i in range(n)]
        out = [(i, None) for i in range(loop["start"])]
        for p in range(loop["times"]):
            out += [(i, p if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
        return out + [(i, None) for i in range(loop["stop"], n)]

    def hidden(self, tokens, every_layer: bool = False):
        toks = np.asarray(tokens)
        pos = np.arange(len(toks))
        x, seen = self.w["embed"][toks] * float(self.cfg["embedding"]["scale"]), []
        self.margins = []
        for i, opens in self.runs():
            if opens is not None:
                x = x + self.w["loop.step"][opens]
            x = self.layer(i, x, pos)
            seen.append(x)
        return seen if every_layer else x

    def close_calls(self, tokens, below: float, last: int = 0) -> int:
        """How many (of the ``last``, or all) tokens have an expert choice somewhere that hangs on less than ``below``."""
        self.hidden(tokens)
        return int((np.min(self.margins, axis=0)[-last:] < below).sum()) if self.margins else 0

    def logits(self, tokens) -> np.ndarray:
        x = self.rnd(rms_norm(self.hidden(tokens), self.w["final.norm"], self.eps))
        return x @ self.w["head"].T * float(self.cfg["logit_scale"])

    def greedy(self, prompt, n: int) -> list[int]:
        toks, out = list(prompt), []
        for _ in range(n):
            out.append(int(np.argmax(self.logits(toks)[-1])))
            toks.append(out[-1])
        return out
