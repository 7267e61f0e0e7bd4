"""A decoder built from a ``ModelSpec``: token table, layers run in the listed order,
final norm, output matrix. This is the one forward pass of the package: generation, the
scheduler's engine and trace replay all call ``DecoderModel.step``."""

from __future__ import annotations

from typing import TYPE_CHECKING, Any, Mapping

import torch

from . import attention as _attention  # noqa: F401  (registers the built-in parts)
from . import block as _block  # noqa: F401
from . import delta as _delta  # noqa: F401
from . import hyper as _hyper  # noqa: F401
from . import latent as _latent  # noqa: F401
from . import mlp as _mlp  # noqa: F401
from . import moe as _moe  # noqa: F401
from . import norm as _norm  # noqa: F401
from . import parallel as _parallel  # noqa: F401
from . import recurrent as _recurrent  # noqa: F401
from . import retention as _retention  # noqa: F401
from . import rope as _rope  # noqa: F401
from . import ssm as _ssm  # noqa: F401
from . import stream as _stream  # noqa: F401
from .base import CacheNeed, Part, Runtime, StateNeed, WeightWant, make
from .spec import ModelSpec

if TYPE_CHECKING:
    from prefixserve_amd.engine.batch import StepContext


class DecoderModel:
    def __init__(self, spec: ModelSpec) -> None:
        spec.validate()
        self.spec = spec
        self.positions = {name: make("position", ps.kind, **ps.params) for name, ps in spec.positions.items()}
        self.blocks = []
        for layer in spec.layers:
            h = spec.hidden_size
            mixer = make("mixer", layer.mixer.kind, hidden_size=h, positions=self.positions, **layer.mixer.params)
            ff = n2 = None
            if layer.feed_forward is not None:
                ff = make("feed_forward", layer.feed_forward.kind, hidden_size=h, **layer.feed_forward.params)
            n1 = make("norm", layer.mixer_norm.kind, hidden_size=h, **layer.mixer_norm.params)
            if layer.feed_forward_norm is not None:
                n2 = make("norm", layer.feed_forward_norm.kind, hidden_size=h, **layer.feed_forward_norm.params)
            extra = {name: make("norm", ps.kind, hidden_size=h, **ps.params) for name, ps in layer.extra_norms.items()}
            self.blocks.append(make("block", layer.block, mixer=mixer, feed_forward=ff, mixer_norm=n1,
                                    feed_forward_norm=n2, **extra, **layer.block_params))
        self.final_norm = make("norm", spec.final_norm.kind, hidden_size=spec.hidden_size, **spec.final_norm.params)
        sizes = dict(hidden_size=spec.hidden_size, vocab_size=spec.vocab_size)
        self.embedding_transforms = [make("transform", ps.kind, **sizes, **ps.params) for ps in spec.embedding_transforms]
        # A constant in front of everything else is the gather's own factor.
        self.embedding_factor = getattr(self.embedding_transforms[0], "embedding_factor", None) if self.embedding_transforms else None
        for tr in self.embedding_transforms[1:]:
            if tr.gather is not None or tr.state_need() is not None:
                raise ValueError("a transform that does the gather or keeps state comes first behind the token table")
        # The block of the first run reads the stream's copy in the activation dtype: a gather may write it as well.
        self.gather_copies = bool(self.blocks) and getattr(self.blocks[spec.order[0].layer], "reads_stream_copy", False) \
            and len(self.embedding_transforms) == 1
        self.logit_transforms = [make("transform", ps.kind, **sizes, **ps.params) for ps in spec.logit_transforms]
        self.stream_transforms = {name: make("transform", ps.kind, **sizes, **ps.params)
                                  for name, ps in spec.stream_transforms.items()}
        # The token table's output (behind its transforms) is kept for the step if a transform asks.
        self.keeps_embedding_output = any(getattr(tr, "needs_embedding_output", False)
                                          for tr in self.stream_transforms.values())
        self.caches: dict[int, Any] = {}
        self.states: dict[int, torch.Tensor] = {}
        self.rt: Runtime | None = None

    # ---------------------------------------------------------------- weights

    def _named_parts(self) -> list[tuple[str, Part]]:
        out: list[tuple[str, Part]] = []
        for layer, blk in zip(self.spec.layers, self.blocks):
            out += [(layer.prefix, p) for p in blk.parts()]
        out.append((self.spec.final_norm_prefix, self.final_norm))
        out += [("", tr) for tr in self.embedding_transforms + self.logit_transforms + list(self.stream_transforms.values())]
        return out

    def weights(self) -> dict[str, WeightWant]:
        """Every tensor the model wants, by full name."""
        s = self.spec
        want: dict[str, WeightWant] = {s.embedding: WeightWant((s.vocab_size, s.hidden_size), "embedding")}
        for prefix, part in self._named_parts():
            for rel, w in part.weights().items():
                want[prefix + rel] = w
        if s.head is not None:
            want[s.head] = WeightWant((s.vocab_size, s.hidden_size), "matrix")
        return want

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime, max_position: int) -> None:
        """Hands each part its tensors and builds position tables up to ``max_position``."""
        s = self.spec
        if max_position > s.max_position:
            raise ValueError(f"max_position {max_position} > the model's limit {s.max_position}")
        self.rt = rt
        for pos in self.positions.values():
            pos.bind({}, rt)
            pos.prepare(max_position)
        for prefix, part in self._named_parts():
            part.bind({rel: tensors[prefix + rel] for rel in part.weights()}, rt)
        self.embedding = rt.ops.prepare_matrix(tensors[s.embedding], rt)
        # Tied output matrix = the very same storage (prefixserve/model/weights.py:133-136).
        self.head = self.embedding if s.head is None else rt.ops.prepare_matrix(tensors[s.head], rt)
        self.max_position = int(max_position)

    def step_weight_bytes(self) -> int:
        """Bytes of weights one decode step reads: every layer's matrices and norm weights in
        each run, the final norm and the output matrix. The token table is only gathered from
        (a few rows), unless it is also the output matrix."""
        total = 0
        for run in self.spec.order:
            total += sum(p.weight_bytes() for p in self.blocks[run.layer].parts())
        total += self.final_norm.weight_bytes()
        total += self.head.numel() * self.head.element_size()
        return total

    # ------------------------------------------------------------------ cache

    def cache_needs(self) -> dict[int, CacheNeed]:
        """cache entry -> what its writing run's mixer needs."""
        needs: dict[int, CacheNeed] = {}
        for run in self.spec.order:
            need = self.blocks[run.layer].mixer.cache_need()
            if need is None:
                continue
            if run.writes_cache:
                needs[run.cache] = need
        # A mixer's further entries get numbers of their own behind every run's.
        for key, need in self._aux_entries().items():
            needs[self._aux_ids[key]] = need
        return needs

    def _aux_entries(self) -> dict[tuple[int, str], CacheNeed]:
        """(cache entry of the writing run, the mixer's name for it) -> need, and their entry numbers."""
        out: dict[tuple[int, str], CacheNeed] = {}
        for run in self.spec.order:
            if run.writes_cache:
                for name, need in self.blocks[run.layer].mixer.aux_cache_needs().items():
                    out[(run.cache, name)] = need
        base = 1 + max((run.cache for run in self.spec.order), default=0)
        self._aux_ids = {key: base + i for i, key in enumerate(sorted(out))}
        return out

    def state_needs(self) -> dict[int, StateNeed]:
        """index into ``spec.order`` -> fixed-size per-request state its mixer keeps; -1: that of the first transform
        behind the token table."""
        needs: dict[int, StateNeed] = {}
        if self.embedding_transforms and self.embedding_transforms[0].state_need() is not None:
            needs[-1] = self.embedding_transforms[0].state_need()
        for i, run in enumerate(self.spec.order):
            need = self._block_state_need(self.blocks[run.layer])
            if need is not None:
                needs[i] = need
        return needs

    @staticmethod
    def _block_state_need(blk: Any) -> StateNeed | None:
        """A block may keep state of its own around its mixer's (``state_need`` of the block);
        otherwise the run's state is the mixer's."""
        own = getattr(blk, "state_need", None)
        return own() if own is not None else blk.mixer.state_need()

    def state_in_graphs(self) -> bool:
        """Whether every part that keeps state lets a captured decode step update it."""
        if any(tr.state_need() is not None and not tr.state_in_graphs for tr in self.embedding_transforms[:1]):
            return False
        return all(getattr(blk, "state_in_graphs", blk.mixer.state_in_graphs) for blk in self.blocks
                   if self._block_state_need(blk) is not None)

    def attach(self, caches: Mapping[int, Any], states: Mapping[int, torch.Tensor]) -> None:
        self.caches = dict(caches)
        self.states = dict(states)
        for (entry, name), _need in self._aux_entries().items():
            main, aux = self.caches.get(entry), self.caches.get(self._aux_ids[(entry, name)])
            if main is not None and aux is not None:
                main.aux = {**(main.aux or {}), name: aux}

    # ------------------------------------------------------------------- step

    def step(self, ctx: "StepContext") -> torch.Tensor | None:
        """Runs the tokens of ``ctx`` as one batch from the cache and returns float32 logits
        ``[S, vocab]`` at the wanted rows (None when no row is wanted: nothing to wait for).
        Rows first, then the norm, then the product: only S rows pay for the vocabulary
        (prefixserve/model/llama.py:96-101,123-126)."""
        rt = self.rt
        assert rt is not None, "bind() first"
        s, ws, ops = self.spec, rt.workspace, rt.ops
        t = ctx.num_tokens
        with ops.step_scope():
            if s.streams > 1:
                # Every copy of the stream starts as the token table's output; blocks get all of them.
                streams = ws.get("residual", (s.streams, t, s.hidden_size), torch.float32)
                residual = streams[0]
            else:
                streams = residual = ws.get("residual", (t, s.hidden_size), torch.float32)
            copy = None
            first = self.embedding_transforms[0] if self.embedding_transforms else None
            if first is not None and first.gather is not None:
                if self.gather_copies and rt.dtype != torch.float32:
                    copy = ws.get("block.x", (t, s.hidden_size), rt.dtype)
                first.gather(ctx.token_ids, self.embedding, residual, ctx, self.states.get(-1), copy)
            elif self.embedding_factor is not None:
                ops.embed(ctx.token_ids, self.embedding, residual, factor=self.embedding_factor)
            else:
                ops.embed(ctx.token_ids, self.embedding, residual)
            done = first is not None and (first.gather is not None or self.embedding_factor is not None)
            for tr in self.embedding_transforms[1 if done else 0:]:
                tr.apply(residual, ctx, None)
            if s.streams > 1:
                streams[1:].copy_(residual.unsqueeze(0).expand(s.streams - 1, t, s.hidden_size))
            ctx.residual = residual
            ctx.residual_scale = None
            ctx.stream_copy = copy           # a context may be stepped twice (a graph's eager run, then its capture)
            if self.keeps_embedding_output:
                ctx.embedding_output = ws.get("embedding.output", (t, s.hidden_size), torch.float32)
                ctx.embedding_output.copy_(residual)
            pending = None
            for i, run in enumerate(s.order):
                if run.before:
                    # A transform reads and writes the stream itself: what the last sub-layer left to
                    # be added goes in first.
                    ctx.stream_copy = None
                    ctx.pass_index = run.pass_index
                    todo = [self.stream_transforms[name] for name in run.before]
                    if pending is not None:
                        if todo[0].add_pending is not None:
                            todo.pop(0).add_pending(residual, pending, ctx)
                        else:
                            ops.residual_add(residual, pending)
                        pending = None
                    for tr in todo:
                        tr.apply(residual, ctx, None)
                pending = self.blocks[run.layer].forward(streams, pending, ctx, self.caches.get(run.cache),
                                                         self.states.get(i), run.writes_cache)
            if ctx.num_logit_rows == 0:
                return None
            if s.streams > 1:
                # The final norm reads the sum of the copies: the others join the first as slices to be added.
                assert pending is None, "a block over several streams leaves nothing pending"
                pending = streams[1:]
            x = self.final_norm.add_norm_rows(residual, pending, ctx.logit_rows, "final.x", lazy=True)
            logits = ws.get("logits", (ctx.num_logit_rows, s.vocab_size), torch.float32)
            ops.linear(x, self.head, logits)
            for tr in self.logit_transforms:
                tr.apply(logits, ctx, ctx.logit_rows)
            return logits
