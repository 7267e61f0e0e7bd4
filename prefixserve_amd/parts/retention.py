"""Retention: linear attention with a fixed decay per head and a matrix per head as fixed-size state."""

from __future__ import annotations

from typing import TYPE_CHECKING, Any, Mapping, Sequence

import torch

from .attention import head_slots
from .base import Mixer, PositionEncoding, RotaryTable, Runtime, StateNeed, WeightWant, register_mixer

if TYPE_CHECKING:
    from prefixserve_amd.engine.batch import StepContext


def decay_powers(decays: Sequence[float], count: int) -> torch.Tensor:
    """[heads, count] float32: every decay to the powers 0 .. count - 1, formed in float64 and rounded once."""
    g = torch.tensor([float(d) for d in decays], dtype=torch.float64)
    n = torch.arange(count, dtype=torch.float64)
    return torch.pow(g[:, None], n[None, :]).to(torch.float32).contiguous()


def padded(size: int) -> int:
    """The size the kernels run a head of ``size`` dimensions with."""
    return -(-int(size) // 16) * 16


class Retention(Mixer):
    """q, k = W x (``num_heads`` x ``head_dim``), v = W x (``num_heads`` x ``value_dim``), without biases;
    q and k are rotated (the table of the encoding ``position``: pairs (i, i + r/2) of the first r
    dimensions), k also times head_dim^-1/2. With a fixed decay g per head (``decays``) and no softmax or
    denominator
        S <- g S + k v^T;   o = S^T q        (read after the write)
    then o / rms(o) per head without a weight, times silu(W_g x), then the output matrix.

    Rotation, recurrence, state and norm are 32-bit in every mode. The per-request state is S as [heads,
    head_dim, value_dim], sizes rounded up to multiples of 16: the matrices' rows are laid out so, with
    zeros, the rotation's partners half a head apart (the encoding is made for heads of that size,
    ``padded``). Because the decay does not depend on the token, a portion runs in pieces side by side on
    the matrix cores. ``names``: "q", "k", "v", "gate", "o"."""

    state_in_graphs = True
    state_align = 4                  # the kernels read and write four values of the state at a time
    takes_input_rows = True

    def __init__(self, hidden_size: int, positions: Mapping[str, PositionEncoding], num_heads: int, head_dim: int, value_dim: int,
                 decays: Sequence[float], names: Mapping[str, str], norm_eps: float, position: str) -> None:
        self.hidden_size = int(hidden_size)
        self.num_heads, self.head_dim, self.value_dim = int(num_heads), int(head_dim), int(value_dim)
        self.decays = tuple(float(d) for d in decays)
        self.norm_eps = float(norm_eps)
        if self.num_heads < 1 or not 1 <= self.head_dim <= 256 or not 1 <= self.value_dim <= 256:
            raise ValueError(f"{num_heads} heads of {head_dim} and {value_dim} (at most 256 each)")
        if len(self.decays) != self.num_heads:
            raise ValueError(f"{len(self.decays)} decays for {num_heads} heads")
        self.dim_p, self.vdim_p = padded(self.head_dim), padded(self.value_dim)
        self.pos = positions[position]
        if not isinstance(self.pos, RotaryTable) or self.pos.head_dim != self.dim_p:
            raise ValueError(f"retention applies a rotation table made for heads of {self.dim_p}")
        rotary = self.dim_p if self.pos.rotary_dim is None else int(self.pos.rotary_dim)
        if rotary > self.head_dim:
            raise ValueError(f"{rotary} rotating dimensions in a head of {self.head_dim}")
        self.index = head_slots(self.head_dim, rotary, self.dim_p)
        self.names = dict(names)
        self.key_size, self.value_size = self.num_heads * self.dim_p, self.num_heads * self.vdim_p

    def weights(self) -> dict[str, WeightWant]:
        h, n, hd = self.hidden_size, self.names, self.num_heads
        return {n["q"]: WeightWant((hd * self.head_dim, h)), n["k"]: WeightWant((hd * self.head_dim, h)),
                n["v"]: WeightWant((hd * self.value_dim, h)), n["gate"]: WeightWant((hd * self.value_dim, h)),
                n["o"]: WeightWant((h, hd * self.value_dim))}

    def state_need(self) -> StateNeed:
        return StateNeed((self.num_heads * self.dim_p * self.vdim_p,), torch.float32)

    def _laid_out(self, w: torch.Tensor, size: int, slots: int, index: "list[int] | None" = None) -> torch.Tensor:
        """Rows [heads * size, K] laid into [heads * slots, K]; ``index``: slot of each row of a head."""
        out = torch.zeros((self.num_heads, slots, w.shape[1]), dtype=w.dtype)
        out[:, list(range(size)) if index is None else index] = w.view(self.num_heads, size, w.shape[1])
        return out.view(self.num_heads * slots, w.shape[1])

    def input_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        """Rows of q, k, v and the gate, heads laid into their slots."""
        n = self.names
        return torch.cat([self._laid_out(tensors[n[key]], size, slots, index) for key, size, slots, index in (
            ("q", self.head_dim, self.dim_p, self.index), ("k", self.head_dim, self.dim_p, self.index),
            ("v", self.value_dim, self.vdim_p, None), ("gate", self.value_dim, self.vdim_p, None))], dim=0)

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        Mixer.bind(self, tensors, rt)
        self.w_in = None if self.input_elsewhere else rt.ops.prepare_matrix(self.input_matrix(tensors), rt)
        o = tensors[self.names["o"]]
        self.w_o = rt.ops.prepare_matrix(self._laid_out(o.t().contiguous(), self.value_dim, self.vdim_p).t().contiguous(), rt)
        self.powers = decay_powers(self.decays, rt.ops.retention_powers()).to(rt.device)

    def weight_bytes(self) -> int:
        return sum(w.numel() * w.element_size() for w in (self.w_in, self.w_o) if w is not None)

    def forward(self, x: torch.Tensor, ctx: "StepContext", cache: Any, state: torch.Tensor | None,
                writes_cache: bool) -> torch.Tensor | None:
        rows = self.rt.workspace.get("retention.in", (x.shape[0], 2 * (self.key_size + self.value_size)), self.rt.dtype)
        self.rt.ops.linear(x, self.w_in, rows)
        return self.forward_rows(rows, 0, ctx, cache, state, writes_cache)

    def forward_rows(self, rows: torch.Tensor, col: int, ctx: "StepContext", cache: Any, state: torch.Tensor | None,
                     writes_cache: bool) -> torch.Tensor | None:
        """From the product's rows, [q | k | v | gate] from column ``col`` on."""
        rt, ops = self.rt, self.rt.ops
        assert state is not None, "retention keeps its state in a slot"
        out = rt.workspace.get("retention.out", (rows.shape[0], self.value_size), rt.dtype)
        k_col = col + self.key_size
        v_col = k_col + self.key_size
        ops.retention(rows, col, k_col, v_col, v_col + self.value_size, self.pos.table, self.powers,
                      self.head_dim ** -0.5, state, self.state_base, ctx, self.num_heads, self.dim_p, self.vdim_p, self.value_dim,
                      self.norm_eps, out)
        return ops.linear_to_residual(out, self.w_o, "retention.delta", getattr(ctx, "residual", None))


register_mixer("retention", Retention)
