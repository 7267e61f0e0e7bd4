"""A plain, slow Durelix in numpy (float64), whole sequences at a time, one function per mechanism. It shares no code
with the package: it is what the engine is compared with.

Durelix adds to the token table's row a row of a bigram table (hashed from the token and the one in front of it). A sub-layer
reads the stream x itself, and its output is normalized before it is added: x <- x + norm(f(x)). The mixer is two side by side,
half the sum of their normalized outputs: attention in a sliding window (short convolutions, a norm per head in front of the
rotation, a sink per head, a gate on the output) and retention (linear attention with a fixed decay per head). The
feed-forward is a squared-ReLU one or a mixture of gated experts and identity experts. The output matrix is the token table.

``bf16=True`` rounds what an engine holds in bfloat16 (weights are bfloat16 already; what a sub-layer reads, the
projections, the cached keys and values, a sub-layer's inner activations and its output) and keeps the rest exact: the
yardstick for that mode."""

from __future__ import annotations

import json
from pathlib import Path

import numpy as np

from .zurolorn_plain import exact, load_tensors, to_bf16


def sigmoid(z: np.ndarray) -> np.ndarray:
    return 1.0 / (1.0 + np.exp(-z))


def silu(z: np.ndarray) -> np.ndarray:
    return z * sigmoid(z)


def unit_rms(x: np.ndarray, eps: float) -> np.ndarray:
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)


# ------------------------------------------------------------------ token table

def bigram_rows(tokens, buckets: int, mul_prev: int, mul_cur: int) -> list[int]:
    """The bigram table's row for every token of a sequence."""
    toks = [int(t) for t in tokens]
    return [buckets] + [(p * mul_prev + c * mul_cur) % buckets for p, c in zip(toks, toks[1:])]


# ------------------------------------------------------------------ attention

def short_conv(u: np.ndarray, w: np.ndarray) -> np.ndarray:
    """y[t, c] = sum_j w[c, j] u[t - taps + 1 + j, c], u = 0 in front of the sequence."""
    t, taps = u.shape[0], w.shape[1]
    y = np.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < t:
            y[back:] += w[:, j] * u[: t - back]
    return y


def rotate(x: np.ndarray, pos: np.ndarray, dims: int, base: float, halves: bool) -> np.ndarray:
    """x [T, heads, d]: the first ``dims`` dimensions turned; partners (i, i + dims/2) for ``halves``, else (2i, 2i + 1)."""
    out = x.copy()
    for i in range(dims // 2):
        u, v = (i, i + dims // 2) if halves else (2 * i, 2 * i + 1)
        a = pos.astype(np.float64) * float(base) ** (-2.0 * i / dims)
        c, s = np.cos(a)[:, None], np.sin(a)[:, None]
        out[..., u] = x[..., u] * c - x[..., v] * s
        out[..., v] = x[..., v] * c + x[..., u] * s
    return out


def window_mask(t: int, size: int) -> np.ndarray:
    back = np.arange(t)[:, None] - np.arange(t)[None, :]
    return (back >= 0) & (back < size)


def sink_softmax(scores: np.ndarray, seen: np.ndarray, sink: float) -> np.ndarray:
    """[T, T] scores -> weights; exp(sink) joins every row's denominator and has no value."""
    s = np.where(seen, scores, -np.inf)
    top = np.maximum(s.max(-1, keepdims=True), sink)
    e = np.exp(s - top)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - top))


def attention_heads(h: np.ndarray, pos: np.ndarray, w: dict, m: dict, eps: float, rnd=exact):
    """(q [T, heads, dim], k [T, kv_heads, dim], v [T, kv_heads, vdim]) as the softmax and a cache see them."""
    t = h.shape[0]
    q, k, v = (short_conv(rnd(h @ w[n].T), w[n + ".conv"]) for n in ("q", "k", "v"))
    out = []
    for x, heads, norm in ((q, m["heads"], "q.norm"), (k, m["kv_heads"], "k.norm")):
        x = unit_rms(x.reshape(t, heads, m["dim"]), eps) * w[norm]
        rot = m.get("rot")
        out.append(rnd(x if rot is None else rotate(x, pos, rot["dims"], rot["base"], False)))
    return out[0], out[1], rnd(v.reshape(t, m["kv_heads"], m["vdim"]))


def attention_weights(q: np.ndarray, k: np.ndarray, w: dict, m: dict, head: int) -> np.ndarray:
    kv = head // (m["heads"] // m["kv_heads"])
    return sink_softmax(q[:, head] @ k[:, kv].T * m["scale"], window_mask(len(q), m["mask"]["size"]), float(w["sink"][head]))


def window_attention(h: np.ndarray, pos: np.ndarray, w: dict, m: dict, eps: float, rnd=exact) -> np.ndarray:
    q, k, v = attention_heads(h, pos, w, m, eps, rnd)
    per = m["heads"] // m["kv_heads"]
    o = np.concatenate([attention_weights(q, k, w, m, a) @ v[:, a // per] for a in range(m["heads"])], axis=-1)
    return rnd(rnd(o * sigmoid(rnd(h @ w["g"].T))) @ w["o"].T)


# ------------------------------------------------------------------ retention

def retention_scan(q: np.ndarray, k: np.ndarray, v: np.ndarray, decay) -> np.ndarray:
    """Per head S <- decay S + k v^T, o = S^T q, token by token; [T, heads, .] each."""
    t, heads, _ = q.shape
    out = np.zeros((t, heads, v.shape[-1]))
    for a in range(heads):
        s = np.zeros((q.shape[-1], v.shape[-1]))
        for i in range(t):
            s = float(decay[a]) * s + np.outer(k[i, a], v[i, a])
            out[i, a] = s.T @ q[i, a]
    return out


def retention(h: np.ndarray, pos: np.ndarray, w: dict, m: dict, eps: float, rnd=exact) -> np.ndarray:
    t, heads, d = h.shape[0], m["heads"], m["dim"]
    q, k, v, g = (rnd(h @ w[n].T) for n in ("q", "k", "v", "g"))
    q, k = q.reshape(t, heads, d), k.reshape(t, heads, d)
    rot = m.get("rot")
    if rot is not None:
        q, k = (rotate(x, pos, rot["dims"], rot["base"], True) for x in (q, k))
    o = unit_rms(retention_scan(q, k * d ** -0.5, v.reshape(t, heads, m["vdim"]), m["decay"]), eps).reshape(t, -1)
    return rnd(rnd(o * silu(g)) @ w["o"].T)


# ------------------------------------------------------------------ feed-forwards

def dense(h: np.ndarray, w: dict, rnd=exact) -> np.ndarray:
    z = rnd(h @ w["up"].T)
    return rnd(rnd(np.square(np.maximum(z, 0.0))) @ w["down"].T)


def softmax(z: np.ndarray) -> np.ndarray:
    e = np.exp(z - z.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def choose(scores: np.ndarray, top: int, groups: dict | None) -> np.ndarray:
    """The ``top`` largest of one token's choice scores among those of the best groups of neighbours (a group's score is
    its largest); the lower index among equals."""
    allowed = np.ones(len(scores), dtype=bool)
    if groups:
        best = np.argsort(-scores.reshape(groups["count"], -1).max(-1), kind="stable")[: groups["keep"]]
        allowed = np.isin(np.arange(len(scores)) // (len(scores) // groups["count"]), best)
    return np.argsort(-np.where(allowed, scores, -np.inf), kind="stable")[:top]


def choice_margin(scores: np.ndarray, top: int, groups: dict | None) -> float:
    """How far one token's choice scores would have to move for another choice."""
    margin, inside = np.inf, np.sort(scores)[::-1]
    if groups:
        per = scores.reshape(groups["count"], -1)
        order = np.argsort(-per.max(-1), kind="stable")
        if groups["keep"] < groups["count"]:
            margin = per[order[groups["keep"] - 1]].max() - per[order[groups["keep"]]].max()
        inside = np.sort(per[order[: groups["keep"]]].reshape(-1))[::-1]
    return float(min(margin, inside[top - 1] - inside[top] if top < len(inside) else np.inf))


def route(h: np.ndarray, w: dict, r: dict) -> tuple[np.ndarray, np.ndarray]:
    """(chosen [T, top], weights): softmax scores over experts and identity experts, the correction for the choice alone."""
    s = softmax(h @ w["router"].T)
    chosen = np.stack([choose(row, r["top"], r.get("groups")) for row in s + w["correction"]])
    return chosen, np.take_along_axis(s, chosen, axis=1)


def expert(h: np.ndarray, gate: np.ndarray, up: np.ndarray, down: np.ndarray, rnd=exact) -> np.ndarray:
    return rnd(silu(h @ gate.T) * (h @ up.T)) @ down.T


def mixture(h: np.ndarray, w: dict, r: dict, rnd=exact) -> np.ndarray:
    chosen, weight = route(h, w, r)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(chosen[t], weight[t]):
            out[t] += g * (h[t] if e >= r["experts"] else expert(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], rnd))
    return out


# ------------------------------------------------------------------ the model

class PlainDurelix:
    def __init__(self, folder: str | Path, bf16: bool = False) -> None:
        folder = Path(folder)
        self.cfg = json.loads((folder / "config.json").read_text())
        self.w = load_tensors(folder)
        self.eps = float(self.cfg["norm"]["eps"])
        self.rnd = to_bf16 if bf16 else exact
        self.margins: list[np.ndarray] = []      # of every layer with experts of the last call, [T] each

    def part(self, prefix: str) -> dict:
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def embed(self, tokens) -> np.ndarray:
        b = self.cfg["embedding"]["bigram"]
        rows = bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])
        return self.w["embed"][np.asarray(tokens, dtype=int)] + self.w["bigram"][rows]

    def mixer(self, i: int, h: np.ndarray, pos: np.ndarray) -> np.ndarray:
        m = self.cfg["layers"][i]["mixer"]
        left = window_attention(h, pos, self.part(f"l{i}.mix.left."), m["left"], self.eps, self.rnd)
        right = retention(h, pos, self.part(f"l{i}.mix.right."), m["right"], self.eps, self.rnd)
        return 0.5 * (unit_rms(left, self.eps) * self.w[f"l{i}.mix.left.out"] + unit_rms(right, self.eps) * self.w[f"l{i}.mix.right.out"])

    def layer(self, i: int, x: np.ndarray, pos: np.ndarray) -> np.ndarray:
        f = self.cfg["layers"][i].get("mlp")
        x = x + unit_rms(self.mixer(i, self.rnd(x), pos), self.eps) * self.w[f"l{i}.norm1"]
        if f is None:
            return x
        h, w = self.rnd(x), self.part(f"l{i}.mlp.")
        if f["kind"] == "dense":
            y = dense(h, w, self.rnd)
        else:
            y, r = mixture(h, w, f["router"], self.rnd), f["router"]
            self.margins.append(np.array([choice_margin(s, r["top"], r.get("groups")) for s in softmax(h @ w["router"].T) + w["correction"]]))
        return x + unit_rms(y, self.eps) * self.w[f"l{i}.norm2"]

    def hidden(self, tokens, every_layer: bool = False):
        pos = np.arange(len(tokens))
        x, seen = self.embed(tokens), []
        self.margins = []
        for i in range(len(self.cfg["layers"])):
            x = self.layer(i, x, pos)
            seen.append(x)
        return seen if every_layer else x

    def close_calls(self, tokens, below: float, last: int = 0) -> int:
        """How many (of the ``last``, or all) tokens have an expert choice somewhere that hangs on less than ``below``."""
        self.hidden(tokens)
        return int((np.min(self.margins, axis=0)[-last:] < below).sum()) if self.margins else 0

    def logits(self, tokens) -> np.ndarray:
        x = self.rnd(unit_rms(self.hidden(tokens), self.eps) * self.w["final.norm"])
        return x @ self.w["embed"].T

    def greedy(self, prompt, n: int) -> list[int]:
        toks, out = list(prompt), []
        for _ in range(n):
            out.append(int(np.argmax(self.logits(toks)[-1])))
            toks.append(out[-1])
        return out
