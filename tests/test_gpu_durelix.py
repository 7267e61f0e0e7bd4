"""Durelix on the GPU: the kernels it brought, each against a plain float64 computation, and the model in both dtypes
against the plain implementation in tests/plain/durelix_plain.py: every cutting, mixed batches on reused pages and slots,
prompts of many runs of retention, captured decode steps, generation, and the programs a user starts."""

from __future__ import annotations

import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import traces
from durelix_configs import DURELIX, attention, dense, layer, model, moe, retention, write_durelix
from plain import durelix_plain as plain
from prefixserve_amd.engine.batch import GroupMeta, StepItem, StepPacker
from prefixserve_amd.engine.replay import TraceReplayer
from prefixserve_amd.engine.runner import ModelRunner
from prefixserve_amd.parts.attention import head_slots
from prefixserve_amd.parts.base import NormedDeltas
from prefixserve_amd.parts.retention import decay_powers
from test_durelix_host import SHARP, carrying_keys, sharp
from test_gpu_kernels import paged_case

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
DEV = "cuda:0"
F32_TOL = 3e-5
# bfloat16: a row's largest error over its largest logit, against the plain model with what an engine holds in bfloat16
# rounded to it (``bf16_bars``): the median and the ninth decile of a trace's rows, and how many rows lie far out. A router's
# close call (choice scores within CLOSE of another choice) falls the other way after rounding, in the yardstick as in the
# engine but not at the same token, and moves that row by tenths and rows behind it a little.
BF16_FACTOR, BF16_TAIL_FACTOR, BF16_FAR_FACTOR, BF16_FAR_SHARE, CLOSE = 1.5, 2.5, 2.0, 0.03, 3e-3


@pytest.fixture(scope="module")
def ops():
    from prefixserve_amd.kernels.ops import HipOps
    from prefixserve_amd.parts.base import Workspace

    return HipOps(torch.device(DEV), Workspace(torch.device(DEV)))


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: write_durelix(tmp_path_factory.mktemp(f"durelix-{name}"), name) for name in DURELIX}


def rnd(*shape, dtype=torch.float32, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype).to(DEV)


def rel(got, want):
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    return float(np.abs(got - want).max() / max(np.abs(want).max(), 1e-30))


def f64(t):
    return t.double().cpu().numpy()


def tol_of(act):
    return 2e-5 if act == torch.float32 else 1e-2


def runner_for(folder, pages, dtype, slots=4, graphs=False):
    return ModelRunner(folder, dtype=dtype, device=DEV, num_blocks=pages, max_seq_len=pages * 16, max_num_seqs=slots,
                       use_graphs=graphs)


class Requests:
    """Steps of a few requests on pages in a scrambled order and in slots of their own, packed as the engine packs them."""

    def __init__(self, ops, pages=80, slots=5, vocab=100):
        self.packer = StepPacker(torch.device(DEV), [GroupMeta(pages)], vocab, pages * 16, slots, ops.PREFILL_TILE_Q)
        self.free = torch.randperm(pages, generator=torch.Generator().manual_seed(5)).tolist()
        self.tables, self.done = {}, {}
        self.slot = {r: (3 * r + 2) % slots for r in range(slots)}

    def step(self, portions: dict[int, int], tokens=None):
        items = []
        for r, n in portions.items():
            start = self.done.get(r, 0)
            table = self.tables.setdefault(r, [])
            while len(table) * 16 < start + n:
                table.append(self.free.pop())
            toks = [1] * n if tokens is None else tokens[r][start: start + n]
            items.append(StepItem(key=r, tokens=toks, start=start, block_tables=[table], slot=self.slot[r], want=[]))
            self.done[r] = start + n
        ctx = self.packer.pack(items)
        torch.cuda.synchronize()
        return ctx


# Portions of requests step by step: prompts of several runs of 128 tokens, single tokens, twos, beside each other.
STEPS = [{0: 300, 1: 1}, {0: 1, 1: 2, 2: 37}, {0: 129, 2: 1}, {1: 1, 0: 1, 2: 1}, {2: 256, 1: 3}, {0: 2, 1: 128, 2: 33}]


def by_request(steps):
    """Flat rows of every step -> for each request the (step, row) places in the order of its tokens."""
    places: dict[int, list] = {}
    for k, portions in enumerate(steps):
        t = 0
        for r, n in portions.items():
            places.setdefault(r, []).extend((k, t + i) for i in range(n))
            t += n
    return places


# ------------------------------------------------------------------ kernels

@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("hidden,buckets,mul_prev,mul_cur", [(64, 37, 5, 3), (50, 1, 9, 2), (1000, 4001, 65537, 257), (2048, 12, 1, 0)])
def test_gather_with_a_bigram_table(ops, act, hidden, buckets, mul_prev, mul_cur):
    vocab = 100
    table, bigram = rnd(vocab, hidden, dtype=act, seed=1), rnd(buckets + 1, hidden, dtype=act, seed=2)
    rng = np.random.default_rng(3)
    toks = {r: rng.integers(0, vocab, 600).tolist() for r in range(3)}
    state = torch.full((5, 1), 77, dtype=torch.int32, device=DEV)          # slots hold junk: the runner clears them
    reqs = Requests(ops)
    state[[reqs.slot[r] for r in range(3)]] = 0
    got = {r: [] for r in toks}
    for portions in STEPS:
        ctx = reqs.step(portions, toks)
        t = ctx.num_tokens
        out, copy = torch.empty(t, hidden, device=DEV), torch.empty(t, hidden, dtype=act, device=DEV)
        ops.embed_bigram(ctx.token_ids, table, bigram, out, copy, state, ctx, mul_prev, mul_cur)
        assert torch.equal(copy, out.to(act))
        at = 0
        for r, n in portions.items():
            got[r].append(out[at: at + n])
            at += n
    for r, parts in got.items():
        rows = torch.cat(parts)
        seq = toks[r][: len(rows)]
        want = table[torch.tensor(seq)].double() + bigram[torch.tensor(plain.bigram_rows(seq, buckets, mul_prev, mul_cur))].double()
        assert rel(rows.cpu(), want.cpu()) < 1e-6
        assert int(state[reqs.slot[r], 0]) == seq[-1] + 1
    assert int((state == 77).sum()) == 2


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("hidden", [64, 50, 1000, 1028, 2048, 4104, 7000, 8200])
@pytest.mark.parametrize("sa,sb", [(0, None), (1, None), (9, None), (0, 0), (3, 0), (8, 8)])
def test_norm_on_an_output(ops, act, hidden, sa, sb):
    """stream += norm(y) * w, y one tensor or slices, or half the sum of two outputs that are normalized first."""
    t = 5
    if sb is not None and hidden > 8192:
        pytest.skip("two rows of this width do not fit in LDS")
    resid, w = rnd(t, hidden, seed=1), 1 + rnd(hidden, seed=2, scale=0.2)

    def output(s, seed):
        d = rnd(t, hidden, dtype=act, seed=seed, scale=0.3) if s == 0 else rnd(s, t, hidden, seed=seed, scale=0.3)
        return d, f64(d) if s == 0 else f64(d).sum(0)

    a, ya = output(sa, 3)
    delta, y = a, ya
    if sb is not None:
        b, yb = output(sb, 4)
        wa, wb = rnd(hidden, seed=5), rnd(hidden, seed=6)
        delta = NormedDeltas([(a, wa), (b, wb)], 0.5, 1e-4)
        y = 0.5 * (plain.unit_rms(ya, 1e-4) * f64(wa) + plain.unit_rms(yb, 1e-4) * f64(wb))
    want = f64(resid) + plain.unit_rms(y, 1e-5) * f64(w)
    for out in (torch.empty(t, hidden, dtype=act, device=DEV), None):
        got = resid.clone()
        ops.output_norm(got, delta, w, 1e-5, out)
        assert rel(got.cpu(), want) < 3e-6
        assert out is None or torch.equal(out, got.to(act))


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("hq,hkv,d,dim,taps,rot,norm", [(4, 2, 64, 64, 3, 64, True), (3, 1, 32, 24, 4, 10, True), (2, 2, 256, 200, 2, 128, True),
                                                       (6, 3, 48, 48, 1, 0, True), (5, 5, 16, 9, 7, 4, False), (2, 1, 96, 96, 16, 96, True),
                                                       (16, 4, 128, 128, 4, 64, True), (1, 1, 160, 150, 5, 0, False)])
def test_short_convolutions_norm_rotation_and_cache_write(ops, act, hq, hkv, d, dim, taps, rot, norm):
    """Over several steps in slots of junk, from the middle of wider rows: every request's q, k and v are those of its whole
    sequence, and nothing but its places in the pages and its slot is written."""
    from prefixserve_amd.parts.attention import head_slots

    channels = (hq + 2 * hkv) * d
    slots_of = head_slots(dim, rot, d, neighbours=True)
    real = np.zeros((hq + 2 * hkv, d), dtype=bool)
    real[:, slots_of] = True                                               # values in the same slots as keys here
    conv = rnd(taps, channels, seed=1) * torch.tensor(real.reshape(-1), device=DEV)
    qw, kw = (rnd(d, seed=s) for s in (2, 3)) if norm else (None, None)
    table = None
    if rot:
        ang = np.zeros((1300, d // 2))
        ang[:, : rot // 2] = np.arange(1300)[:, None] * 500.0 ** (-2.0 * np.arange(rot // 2) / rot)
        table = torch.tensor(np.stack([np.cos(ang), np.sin(ang)], -1), dtype=torch.float32, device=DEV)
    state = torch.full((5, 7 + (taps - 1) * channels + 2), 3e4, device=DEV)
    reqs = Requests(ops)
    for r in range(3):
        state[reqs.slot[r], 7: 7 + (taps - 1) * channels] = 0
    junk = state.clone()
    kv = torch.full((80, 2, hkv, 16 * d), 9.0, dtype=act, device=DEV)
    ins, outs = [], []
    for k, portions in enumerate(STEPS):
        ctx = reqs.step(portions)
        rows = rnd(ctx.num_tokens, 8 + channels + 5, dtype=act, seed=10 + k)
        q = torch.empty(ctx.num_tokens, hq * d, dtype=act, device=DEV)
        ops.qkv_conv_append(rows, 8, conv, hq, hkv, d, ctx.positions, table, dim if norm else 0, 1e-5, qw, kw, q, kv,
                            ctx.groups[0].write_slot, state, 7, ctx)
        ins.append(f64(rows)[:, 8: 8 + channels])
        outs.append(f64(q))
    written = 0
    for r, places in by_request(STEPS).items():
        u = np.stack([ins[k][i] for k, i in places])
        n = len(u)
        y = plain.short_conv(u, f64(conv).T).reshape(n, hq + 2 * hkv, d)
        heads = y[:, : hq + hkv]
        if norm:
            heads = heads / np.sqrt((heads * heads).sum(-1, keepdims=True) / dim + 1e-5)
            heads = np.concatenate([heads[:, :hq] * f64(qw), heads[:, hq:] * f64(kw)], axis=1)
        if rot:
            laid = plain.rotate(heads[..., slots_of], np.arange(n), rot, 500.0, False)
            other = heads
            heads = np.zeros_like(other)
            heads[..., slots_of] = laid
        q = np.stack([outs[k][i] for k, i in places]).reshape(n, hq, d)
        assert rel(q, heads[:, :hq]) < tol_of(act), r
        pos = torch.arange(n)
        page, off = torch.tensor(reqs.tables[r])[pos // 16].to(DEV), (pos % 16).to(DEV)
        assert rel(f64(kv[:, 0].view(80, hkv, 16, d)[page, :, off]), heads[:, hq:]) < tol_of(act)
        assert rel(f64(kv[:, 1].view(80, hkv, d, 16)[page, :, :, off]), y[:, hq + hkv:]) < tol_of(act)
        written += 2 * n * hkv * d
        if taps > 1:
            saved = state[reqs.slot[r], 7: 7 + (taps - 1) * channels].view(taps - 1, channels)
            assert np.array_equal(f64(saved), u[n - taps + 1:])
            junk[reqs.slot[r], 7: 7 + (taps - 1) * channels] = saved.reshape(-1)
    assert torch.equal(state, junk) and int((kv != 9.0).sum()) <= written


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,dim,vdim,rot", [(3, 32, 32, 32), (2, 64, 128, 64), (4, 128, 128, 64), (1, 256, 256, 128), (5, 6, 5, 4), (2, 33, 17, 10),
                                                (2, 48, 80, 0), (3, 16, 200, 16), (2, 200, 24, 200), (1, 96, 64, 96), (2, 20, 130, 12), (1, 130, 48, 2)])
def test_retention_continues_from_its_slot(ops, act, heads, dim, vdim, rot):
    """Prompts of several runs, single tokens and portions of two beside each other, over steps: outputs and states are those
    of the walk token by token over the whole sequence."""
    dim_p, vdim_p = -(-dim // 16) * 16, -(-vdim // 16) * 16
    decays = [0.999, 0.9, 1.0, 0.3, 0.0][:heads]
    powers = decay_powers(decays, ops.retention_powers()).to(DEV)
    index = head_slots(dim, rot, dim_p)                                    # where a head's dimensions stand in its row
    ang = np.zeros((1300, dim_p // 2))                                     # pairs that do not turn
    if rot:
        ang[:, : rot // 2] = np.arange(1300)[:, None] * 900.0 ** (-2.0 * np.arange(rot // 2) / rot)[None]
    table = torch.tensor(np.stack([np.cos(ang), np.sin(ang)], -1), dtype=torch.float32, device=DEV)
    size = heads * dim_p * vdim_p
    state = torch.full((5, 8 + size + 4), 3e4, device=DEV)
    reqs = Requests(ops)
    for r in range(3):
        state[reqs.slot[r], 8: 8 + size] = 0
    cols = [4, 4 + heads * dim_p, 4 + 2 * heads * dim_p, 4 + 2 * heads * dim_p + heads * vdim_p]
    width = 4 + 2 * heads * (dim_p + vdim_p) + 4
    mask = np.zeros(width, dtype=bool)
    for c, at, p in ((cols[0], index, dim_p), (cols[1], index, dim_p), (cols[2], range(vdim), vdim_p), (cols[3], range(vdim), vdim_p)):
        for h in range(heads):
            mask[[c + h * p + i for i in at]] = True
    ins, outs = [], []
    for k, portions in enumerate(STEPS):
        ctx = reqs.step(portions)
        rows = rnd(ctx.num_tokens, width, dtype=act, seed=10 + k, scale=0.7) * torch.tensor(mask, dtype=act, device=DEV)
        out = torch.empty(ctx.num_tokens, heads * vdim_p, dtype=act, device=DEV)
        ops.retention(rows, *cols, table, powers, dim ** -0.5, state, 8, ctx, heads, dim_p, vdim_p, vdim, 1e-5, out)
        ins.append(f64(rows))
        outs.append(f64(out))
    for r, places in by_request(STEPS).items():
        x = np.stack([ins[k][i] for k, i in places])
        got = np.stack([outs[k][i] for k, i in places]).reshape(-1, heads, vdim_p)
        n = len(x)
        q, k_ = (x[:, c: c + heads * dim_p].reshape(n, heads, dim_p)[..., index] for c in cols[:2])
        v, g = (x[:, c: c + heads * vdim_p].reshape(n, heads, vdim_p)[..., :vdim] for c in cols[2:])
        if rot:
            q, k_ = (plain.rotate(y, np.arange(n), rot, 900.0, True) for y in (q, k_))
        k_ = k_ * dim ** -0.5
        want = plain.unit_rms(plain.retention_scan(q, k_, v, decays), 1e-5) * plain.silu(g)
        assert rel(got[..., :vdim], want) < (1e-4 if act == torch.float32 else 1e-2), r
        assert not got[..., vdim:].any()
        s = np.zeros((heads, dim, vdim))
        for i in range(n):
            s = np.asarray(decays)[:, None, None] * s + k_[i][:, :, None] * v[i][:, None, :]
        kept = f64(state[reqs.slot[r], 8: 8 + size]).reshape(heads, dim_p, vdim_p)
        assert rel(kept[:, index, :vdim], s) < 2e-5 and not kept[:, :, vdim:].any()
        assert not kept[:, [i for i in range(dim_p) if i not in index]].any()
    assert bool((state[:, :8] == 3e4).all()) and bool((state[:, 8 + size:] == 3e4).all())


@pytest.mark.parametrize("hq,hkv,d,new,old,window", [
    (8, 2, 64, [37, 1, 130, 1, 2, 16, 1, 1], [0, 15, 50, 31, 94, 16, 0, 200], 70),      # decode, and the per-head kernel for portions
    (32, 8, 64, [2040], [0], 500),                                                       # grouped, a window
    (32, 8, 128, [100], [1948], None),                                                   # grouped in runs, the merge kernel
    (8, 8, 128, [100, 40], [5000, 300], None),                                           # per head in runs
    (32, 16, 64, [300, 70, 1, 2, 129], [0, 500, 77, 40, 1000], 250),                     # two tiles per workgroup
    (6, 3, 48, [5, 1], [300, 700], 64), (6, 2, 256, [150, 1], [90, 300], 40), (5, 1, 32, [33, 1], [7, 1000], None),
    (4, 2, 144, [70, 1], [20, 100], 50),                                                 # the generic kernel
])
@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
def test_attention_with_a_sink_and_a_gate_on_its_output(ops, act, hq, hkv, d, new, old, window):
    pages = sum(-(-(n + o) // 16) for n, o in zip(new, old)) + 8
    sink = rnd(hq, seed=3) + 2.0
    for exact in (True, False):
        for given in (sink, None):
            got, want = paged_case(ops, act, hq, hkv, d, new, old, window=window, seed=hq + d, num_blocks=pages, sink=given, gated=True,
                                   exact_weights=exact)
            assert rel(f64(got), f64(want)) < (2e-5 if act == torch.float32 else 2e-2)


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("t,k,e,identity,top,count,keep", [(1, 96, 6, 2, 3, 4, 2), (9, 64, 12, 0, 2, 3, 1), (70, 128, 60, 4, 8, 8, 4), (3, 200, 120, 10, 8, 13, 5),
                                                           (333, 256, 33, 7, 6, 40, 9), (17, 100, 2, 4, 6, 2, 2), (40, 64, 256, 0, 4, 0, 0), (16, 128, 300, 20, 8, 5, 2),
                                                           (5, 72, 9, 3, 4, 0, 0)])
def test_router_scores_by_a_softmax_over_all_and_chooses_with_a_correction(ops, act, t, k, e, identity, top, count, keep):
    x, n = rnd(t, k, dtype=act, seed=7), e + identity
    w = rnd(n, k, seed=8, scale=0.2).to(torch.bfloat16).float()
    corr = rnd(n, seed=9, scale=0.3) - 0.2                                 # choice scores of both signs
    chosen, weight = torch.empty(t, top, dtype=torch.int32, device=DEV), torch.empty(t, top, device=DEV)
    s = plain.softmax(f64(x) @ f64(w).T)
    groups = {"count": count, "keep": keep} if count else None
    for router in (w.to(act), None):                                       # product + choice; one kernel for both
        for c in (corr, None):
            ops.moe_route(x, w, chosen, weight, router, mode=2, groups=count, keep=keep, group_max=True, identity=identity,
                          **({} if c is None else {"correction": c}))
            got = chosen.cpu().numpy().astype(np.int64)
            score = s if c is None else s + f64(c)
            for i in range(t):
                assert len(set(got[i].tolist())) == top
                if plain.choice_margin(score[i], top, groups) > 1e-5:      # sums that differ by rounding alone may fall either way
                    assert set(got[i].tolist()) == set(plain.choose(score[i], top, groups).tolist()), i
            np.testing.assert_allclose(weight.cpu().numpy(), np.take_along_axis(s, got, -1), rtol=2e-5, atol=1e-7)


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("t,k,f,e,identity,top", [(1, 96, 40, 4, 1, 2), (2, 64, 16, 2, 2, 3), (9, 64, 56, 3, 1, 3), (70, 128, 24, 8, 1, 1), (4, 100, 33, 2, 1, 3),
                                                  (300, 128, 72, 5, 1, 2), (40, 200, 64, 12, 4, 4), (700, 64, 96, 1, 1, 1), (8, 1024, 256, 6, 2, 4)])
def test_experts_beside_identity_experts(ops, act, t, k, f, e, identity, top):
    x = rnd(t, k, dtype=act, seed=9)
    w_in, down = rnd(e, 2 * f, k, dtype=act, seed=10, scale=0.15), rnd(e, k, f, dtype=act, seed=11, scale=0.15)
    gen = torch.Generator().manual_seed(12)
    chosen = torch.stack([torch.randperm(e + identity, generator=gen)[:top] for _ in range(t)]).to(torch.int32).to(DEV)
    weight = (0.1 + torch.rand(t, top, generator=gen)).to(DEV)
    act_buf, out = torch.empty(t * top, f, dtype=act, device=DEV), torch.full((top, t, k), 3.0, device=DEV)
    plain_args = (0.0 + 1.0, float("inf"), 0.0)
    ops.moe_experts(x, chosen, weight, w_in, down, act_buf, out, *plain_args, weight_on_output=True, identity=identity)
    want = np.zeros((top, t, k))
    xs, c, wt = f64(x), chosen.cpu().numpy(), f64(weight)
    for i in range(t):
        for j in range(top):
            ex = c[i, j]
            y = xs[i] if ex >= e else plain.expert(xs[i], f64(w_in[ex, :f]), f64(w_in[ex, f:]), f64(down[ex]))
            want[j, i] = wt[i, j] * y
    assert rel(out.cpu(), want) < (1e-5 if act == torch.float32 else 2e-2)
    if act == torch.bfloat16 and t <= 70:
        resid = rnd(t, k, seed=13)
        got = resid.clone()
        ops.moe_experts(x, chosen, weight, w_in, down, act_buf, None, *plain_args, weight_on_output=True, identity=identity, residual=got)
        assert rel((got - resid).cpu(), f64(out).sum(0)) < 1e-4


def test_kernels_refuse_what_they_do_not_take(ops):
    from prefixserve_amd.kernels.ops import KernelError

    x, i32 = rnd(2, 64), dict(dtype=torch.int32, device=DEV)
    chosen, weight = torch.empty(2, 2, **i32), torch.empty(2, 2, device=DEV)
    for kw in ({"mode": 0, "correction": rnd(8)}, {"mode": 2, "correction": rnd(7)}, {"mode": 3}, {"mode": 2, "groups": 3, "keep": 1},
               {"mode": 2, "groups": 8, "keep": 1}, {"mode": 2, "identity": 8}):
        with pytest.raises(KernelError):
            ops.moe_route(x, rnd(8, 64), chosen, weight, **kw)
    with pytest.raises(KernelError):
        ops.output_norm(x.clone(), rnd(3, 64), rnd(64), 1e-5, None)
    with pytest.raises(KernelError):
        ops.output_norm(x.clone(), NormedDeltas([(x, rnd(64))], 0.5, 1e-5), rnd(64), 1e-5, None)
    ctx = Requests(ops).step({0: 2})
    still = torch.tensor([1.0, 0.0], device=DEV).expand(9, 8, 2).contiguous()
    with pytest.raises(KernelError):                                       # a state row that is no multiple of four
        ops.retention(rnd(2, 64), 0, 16, 32, 48, still, decay_powers([0.5], ops.retention_powers()).to(DEV), 1.0, torch.zeros(5, 257, device=DEV), 0,
                      ctx, 1, 16, 16, 16, 1e-5, torch.empty(2, 16, device=DEV))
    with pytest.raises(KernelError):                                       # columns outside the rows
        ops.retention(rnd(2, 60), 0, 16, 32, 48, still, decay_powers([0.5], ops.retention_powers()).to(DEV), 1.0, torch.zeros(5, 256, device=DEV), 0,
                      ctx, 1, 16, 16, 16, 1e-5, torch.empty(2, 16, device=DEV))
    with pytest.raises(KernelError):
        ops.qkv_conv_append(rnd(2, 48), 0, rnd(3, 48), 1, 1, 16, ctx.positions, None, 16, 1e-5, None, None, torch.empty(2, 16, device=DEV),
                            None, None, torch.zeros(5, 95, device=DEV), 0, ctx)
    with pytest.raises(KernelError):
        ops.embed_bigram(ctx.token_ids, rnd(9, 16), rnd(5, 16), torch.empty(2, 16, device=DEV), None, torch.zeros(5, 1, device=DEV), ctx, 1, 1)


# ------------------------------------------------------------------ whole models

LENGTHS = [70, 33, 97, 18, 64, 45, 1, 52, 2, 81, 29, 3]


def bf16_bars(folder, truth, reqs, last=0):
    """(median, ninth decile, 99th percentile) of the rows (the ``last`` ones of each request, or all) of a plain bfloat16 run
    against the plain model in float64, and the number of close calls."""
    rough = plain.PlainDurelix(folder, bf16=True)
    rows = np.concatenate([np.abs(rough.logits(t)[-last:] - w[-last:]).max(-1) / np.abs(w[-last:]).max(-1) for t, w in zip(reqs, truth)])
    close = sum(plain.PlainDurelix(folder).close_calls(t, CLOSE, last) for t in reqs)
    return (*(float(np.quantile(rows, q)) for q in (0.5, 0.9, 0.99)), close)


def check_rows(errors, dtype, bars=None, tol=F32_TOL):
    if dtype == "float32":
        assert max(errors) < tol, max(errors)
    else:
        e = np.asarray(errors)
        far = int((e > BF16_FAR_FACTOR * bars[2]).sum())
        assert np.isfinite(e).all() and np.median(e) < BF16_FACTOR * bars[0] and np.quantile(e, 0.9) < BF16_TAIL_FACTOR * bars[1] \
            and far <= max(1, BF16_FAR_SHARE * len(e)) + 2 * bars[3], (float(np.median(e)), float(np.quantile(e, 0.9)), far, len(e), bars, float(e.max()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(DURELIX))
def test_every_cutting_matches_the_plain_model(name, dtype, folders):
    rng = np.random.default_rng(4)
    reqs = [rng.integers(0, DURELIX[name]["vocab"], n).tolist() for n in LENGTHS]
    pm = plain.PlainDurelix(folders[name])
    truth = [pm.logits(t) for t in reqs]
    bars = bf16_bars(folders[name], truth, reqs) if dtype == "bfloat16" else None
    runner = runner_for(folders[name], 32, dtype)
    for build in (traces.whole, traces.decode_tail, traces.portions):
        steps, expect = build(reqs)
        errors: list = []
        traces.compare(TraceReplayer(runner).run_step, steps, expect, truth, 10.0, errors)
        check_rows(errors, dtype, bars)
    steps, expect, peak = traces.mixed(reqs, max_live=3, seed=2)
    small = runner_for(folders[name], peak // 16, dtype, slots=3)
    for t in small.pools.tensors:
        t.fill_(3e4)                                        # a page that is used again never holds zeros
    for t in small.states.values():
        t.fill_(7)                                          # nor does a slot
    rp = TraceReplayer(small)
    errors = []
    traces.compare(rp.run_step, steps, expect, truth, 10.0, errors)
    check_rows(errors, dtype, bars)
    assert all(rp.cache.num_free(g) == peak // 16 for g in range(rp.cache.num_groups))


def test_cuttings_agree_with_each_other_in_32_bit(folders):
    """A position's 32-bit logits do not depend on how its prompt was cut, beyond rounding."""
    toks = np.random.default_rng(8).integers(0, 90, 300).tolist()
    runner = runner_for(folders["A"], 24, "float32")
    rows = {}
    for build in (traces.whole, traces.decode_tail, traces.portions):
        steps, expect = build([toks])
        rp = TraceReplayer(runner)
        got = np.concatenate([r for r in (rp.run_step(s) for s in steps) if r is not None])
        rows[build.__name__] = {p: got[k] for k, (_, p) in enumerate(e for exp in expect for e in exp)}
    for p in rows["decode_tail"]:
        assert rel(rows["decode_tail"][p], rows["whole"][p]) < 1e-5 and rel(rows["portions"][p], rows["whole"][p]) < 1e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_windows_and_far_keys(dtype, tmp_path):
    """1,310 tokens under scores with which single keys at the far end of the window carry the weight, and decays with which
    retention sees a thousand tokens back: a prompt of several runs, a portion of twenty tokens behind it, and decoding, beside
    another request on interleaved pages."""
    folder = write_durelix(tmp_path, SHARP, seed=6, std=0.3, edit=sharp)
    toks = np.random.default_rng(5).integers(0, 48, 1310).tolist()
    other = np.random.default_rng(6).integers(0, 48, 40).tolist()
    pm = plain.PlainDurelix(folder)
    truth = [pm.logits(toks), pm.logits(other)]
    assert sum(b > 100 for i, b in carrying_keys(pm, toks).items() if i >= 1280) >= 1
    runner = runner_for(folder, 100, dtype)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:700], "want": [100, 699]}, {"id": "b", "tokens": other[:17], "want": [16]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[700:1280], "want": [579]}, {"id": "b", "tokens": other[17:20], "want": [2]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[1280:1300], "want": list(range(20))}], "end": []}]
    expect = [[(0, 100), (0, 699), (1, 16)], [(0, 1279), (1, 19)], [(0, p) for p in range(1280, 1300)]]
    for i in range(10):
        steps.append({"step": 3 + i, "entries": [{"id": "a", "tokens": [toks[1300 + i]], "want": [0]}, {"id": "b", "tokens": [other[20 + i]], "want": [0]}],
                      "end": []})
        expect.append([(0, 1300 + i), (1, 20 + i)])
    errors: list = []
    traces.compare(TraceReplayer(runner).run_step, steps, expect, truth, 10.0, errors)
    check_rows(errors, dtype, bf16_bars(folder, truth, [toks, other], last=40) if dtype == "bfloat16" else None, tol=1e-4)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes_at_the_kernels_limits(dtype, tmp_path):
    """Heads of 256 on both sides, sixteen taps, a window beyond the prompt, 255 experts and an identity expert in 128 groups."""
    cfg = model(90, 128, 1e-5, (9000, 999983, 1009), [
        layer(attention(2, 1, 256, 200, 16, 1000, 0.06, (256, 1e4)), retention(1, 256, 256, (0.99,), (256, 1e4)), moe(255, 1, 6, 16, (128, 5))),
        layer(attention(20, 1, 16, 256, 2, 30, 0.25, (2, 1e4)), retention(9, 16, 144, [0.9 + 0.01 * i for i in range(9)], (2, 1e4)), moe(2, 0, 2, 200, (1, 1)))])
    folder = write_durelix(tmp_path, cfg, seed=9)
    toks = np.random.default_rng(5).integers(0, 90, 160).tolist()
    truth = plain.PlainDurelix(folder).logits(toks)
    steps, expect = traces.decode_tail([toks], tail=12)
    errors: list = []
    traces.compare(TraceReplayer(runner_for(folder, 12, dtype)).run_step, steps, expect, [truth], 10.0, errors)
    check_rows(errors, dtype, bf16_bars(folder, [truth], [toks], last=13) if dtype == "bfloat16" else None)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes_that_are_multiples_of_nothing(dtype, tmp_path):
    """A width of 90, a vocabulary of 77, inner sizes of 13 and 7, heads of 5, 9 and 11 numbers: the products' and the norms'
    narrow forms, rows that start at odd addresses."""
    cfg = model(77, 90, 1e-6, (13, 3, 4), [
        layer(attention(3, 1, 5, 9, 3, 21, 0.5, (2, 30.0)), retention(3, 7, 11, (0.5, 0.9, 0.99), (6, 60.0)), moe(5, 1, 2, 13, (2, 1))),
        layer(attention(1, 1, 11, 3, 5, 50, 0.4, (10, 900.0)), retention(1, 19, 1, (0.95,)), dense(21)),
        layer(attention(7, 7, 2, 2, 2, 9, 0.7, (2, 900.0)), retention(2, 1, 23, (0.9, 0.8)), moe(4, 1, 5, 7))])
    folder = write_durelix(tmp_path, cfg, seed=13)
    rng = np.random.default_rng(5)
    reqs = [rng.integers(0, 77, n).tolist() for n in (75, 40, 9)]
    pm = plain.PlainDurelix(folder)
    truth = [pm.logits(t) for t in reqs]
    steps, expect, peak = traces.mixed(reqs, max_live=3, seed=1)
    errors: list = []
    traces.compare(TraceReplayer(runner_for(folder, peak // 16, dtype, slots=3)).run_step, steps, expect, truth, 10.0, errors)
    check_rows(errors, dtype, bf16_bars(folder, truth, reqs) if dtype == "bfloat16" else None)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decoding_through_graphs(dtype, folders):
    """Two requests decode side by side through captured steps, then one alone (another graph), for a hundred and twenty tokens;
    the capture's second run of a step leaves no trace in the states."""
    rng = np.random.default_rng(3)
    reqs = [rng.integers(0, 90, n).tolist() for n in (140, 155)]
    pm = plain.PlainDurelix(folders["A"])
    truth = [pm.logits(t) for t in reqs]
    runner = runner_for(folders["A"], 24, dtype, graphs=True)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": reqs[0][:20], "want": [19]}, {"id": "b", "tokens": reqs[1][:31], "want": [30]}], "end": []}]
    expect = [[(0, 19), (1, 30)]]
    for k in range(120):
        steps.append({"step": len(steps), "entries": [{"id": "a", "tokens": [reqs[0][20 + k]], "want": [0]},
                                                     {"id": "b", "tokens": [reqs[1][31 + k]], "want": [0]}], "end": ["a"] if k == 119 else []})
        expect.append([(0, 20 + k), (1, 31 + k)])
    for k in range(151, 155):
        steps.append({"step": len(steps), "entries": [{"id": "b", "tokens": [reqs[1][k]], "want": [0]}], "end": ["b"] if k == 154 else []})
        expect.append([(1, k)])
    errors: list = []
    traces.compare(TraceReplayer(runner).run_step, steps, expect, truth, 10.0, errors)
    check_rows(errors, dtype, bf16_bars(folders["A"], truth, reqs) if dtype == "bfloat16" else None)
    assert runner.use_graphs and len(runner._graphs) == 2


@pytest.mark.parametrize("batch", [3, 12, 20, 40, 70])
def test_decode_batches_of_every_form(batch, folders):
    """Experts pair by pair and grouped, the choice with and without the sorting, products by kernels and by the library."""
    rng = np.random.default_rng(batch)
    reqs = [rng.integers(0, 70, int(n)).tolist() for n in rng.integers(6, 30, batch)]
    pm = plain.PlainDurelix(folders["C"])
    truth = [pm.logits(t) for t in reqs]
    runner = runner_for(folders["C"], 2 * batch, "bfloat16", slots=batch, graphs=True)
    steps = [{"step": i, "entries": [{"id": f"r{i}", "tokens": t[:-4], "want": []}], "end": []} for i, t in enumerate(reqs)]
    expect = [[] for _ in reqs]
    for k in range(4):
        steps.append({"step": len(steps), "entries": [{"id": f"r{i}", "tokens": [t[len(t) - 4 + k]], "want": [0]} for i, t in enumerate(reqs)], "end": []})
        expect.append([(i, len(t) - 4 + k) for i, t in enumerate(reqs)])
    errors: list = []
    traces.compare(TraceReplayer(runner).run_step, steps, expect, truth, 10.0, errors)
    check_rows(errors, "bfloat16", bf16_bars(folders["C"], truth, reqs))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_generation_through_the_entry_point(dtype, folders):
    """Portions under a budget, few pages; in bfloat16 ``warm_up()`` and eight decode steps a round too, whose tokens reach the
    bigram table without the host seeing them."""
    from prefixserve_amd.engine.engine import Engine, EngineConfig
    from prefixserve_amd.generation import generate

    pm = plain.PlainDurelix(folders["A"])
    rng = np.random.default_rng(12)
    prompts = [rng.integers(0, 90, n).tolist() for n in (34, 5, 23, 40, 9, 35)]
    eng = Engine(EngineConfig(model_path=str(folders["A"]), dtype=dtype, max_num_seqs=3, max_prefill_tokens=16,
                              max_seq_len=128, num_blocks=12, **({"decode_steps": 8} if dtype == "bfloat16" else {})))
    if dtype == "bfloat16":
        eng.warm_up()
    outs, _ = generate(eng, prompts, 12, temperature=0.0, ignore_eos=True)
    if dtype == "float32":
        for p, o in zip(prompts, outs):
            assert list(o.tokens) == pm.greedy(p, 12)
    else:
        rough = bf16_bars(folders["A"], [pm.logits(p) for p in prompts], prompts)[2]
        for p, o in zip(prompts, outs):                     # every token is the plain model's best, or as good to within rounding
            rows = pm.logits(p + list(o.tokens))[len(p) - 1: -1]
            for row, tok in zip(rows, o.tokens):
                assert row.max() - row[tok] <= 4.0 * rough * np.abs(row).max()


def test_pools_sized_from_a_measured_step_leave_room_for_many_short_portions(folders):
    """The largest step a scheduler asks for is one long portion; a step of many portions of two tokens has more runs of retention."""
    runner = ModelRunner(folders["A"], dtype="bfloat16", device=DEV, num_blocks=None, max_seq_len=512, max_num_seqs=24, max_prefill_tokens=256,
                         reserve_bytes=200 << 30)
    version = runner.workspace.version
    items = [StepItem(key=i, tokens=[i, i + 1], start=0, block_tables=[[i]] * len(runner.layer_groups), slot=i, want=[1]) for i in range(24)]
    got = runner.step(items)
    pm = plain.PlainDurelix(folders["A"])
    want = np.stack([pm.logits([i, i + 1])[-1] for i in range(24)])
    assert rel(got.cpu(), want) < 0.1
    kept = runner.workspace._bufs["retention.sums"].numel()
    assert kept >= 24 * 4 * 16 * 16 and runner.workspace.version - version <= 8


def test_trace_run_and_the_command_line_as_programs(folders, tmp_path):
    rng = np.random.default_rng(7)
    reqs = [rng.integers(0, 90, n).tolist() for n in (40, 70, 25, 90, 33)]
    pm = plain.PlainDurelix(folders["A"])
    truth = [pm.logits(t) for t in reqs]
    steps, expect, peak = traces.mixed(reqs, max_live=3, seed=5)
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / f"out-{dtype}"
        proc = subprocess.run([str(ROOT / "bin" / "trace_run"), "--model", str(folders["A"]), "--dtype", dtype, "--out", str(out),
                               "--max-tokens", str(peak)], input="".join(json.dumps(s) + "\n" for s in steps), text=True,
                              capture_output=True, env=dict(os.environ), timeout=600)
        assert proc.returncode == 0, proc.stderr[-2000:]
        assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
        errors = []
        for s, exp in zip(steps, expect):
            if exp:
                got = np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(len(exp), -1)
                errors += [rel(row, truth[i][p]) for row, (i, p) in zip(got, exp)]
        check_rows(errors, dtype, bf16_bars(folders["A"], truth, reqs) if dtype == "bfloat16" else None)
    prompt = [5, 17, 3, 80, 41, 7, 7, 19, 0, 64, 11]
    proc = subprocess.run(
        [sys.executable, "-m", "prefixserve_amd.cli", "generate", "--model", str(folders["A"]), "--dtype", "float32",
         "--max-seq-len", "128", "--num-blocks", "16", "--max-running-requests", "2", "--chunked-prefill-size", "5",
         "--max-tokens", "6", "--ignore-eos", "--prompt-ids", ",".join(map(str, prompt))],
        capture_output=True, text=True, cwd=ROOT, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert json.loads(proc.stdout.strip().splitlines()[-1])["outputs"][0]["tokens"] == pm.greedy(prompt, 6)


def random_durelix(rng) -> dict:
    """A configuration drawn at random: widths that are no multiples of 16, one to four layers, any feed-forward or none."""
    layers = []
    for _ in range(int(rng.integers(1, 5))):
        kv = int(rng.integers(1, 4))
        dim, rdim = int(rng.choice([6, 16, 20, 34, 64])), int(rng.choice([4, 16, 22, 50]))
        heads = int(rng.integers(1, 6))
        left = attention(kv * int(rng.integers(1, 4)), kv, dim, int(rng.choice([5, 16, 24, 64])), int(rng.integers(1, 6)), int(rng.choice([1, 8, 16, 31, 200])),
                         float(rng.choice([0.1, 0.3, 0.8])), None if rng.random() < 0.2 else (2 * int(rng.integers(1, dim // 2 + 1)), float(rng.choice([20.0, 1e4]))))
        right = retention(heads, rdim, int(rng.choice([3, 16, 40])), rng.uniform(0.5, 1.0, heads).tolist(),
                          None if rng.random() < 0.2 else (2 * int(rng.integers(1, rdim // 2 + 1)), float(rng.choice([20.0, 1e6]))))
        mlp = None if rng.random() < 0.2 else dense(int(rng.choice([17, 40, 96])))
        if rng.random() < 0.6:
            count, per = int(rng.choice([1, 2, 3, 5])), int(rng.choice([1, 2, 4, 7]))
            keep = int(rng.integers(1, count + 1))
            identity = int(rng.integers(0, min(4, count * per)))
            mlp = moe(count * per - identity, identity, int(rng.integers(1, keep * per + 1)), int(rng.choice([8, 20, 24, 40])), (count, keep) if rng.random() < 0.7 else None)
        layers.append(layer(left, right, mlp))
    return model(int(rng.choice([50, 131, 250])), int(rng.choice([40, 72, 100, 136])), float(rng.choice([1e-5, 1e-6])),
                 (int(rng.choice([1, 30, 997])), int(rng.integers(1, 50)), int(rng.integers(1, 50))), layers)


def first_close_call(pm, toks, below=1e-2) -> int:
    """The first token some layer's choice for which hangs on less than ``below``; the number of tokens if there is none."""
    pm.hidden(toks)
    close = np.min(pm.margins, axis=0) < below if pm.margins else np.zeros(len(toks), dtype=bool)
    return int(np.argmax(close)) if close.any() else len(toks)


@pytest.mark.parametrize("seed", range(10))
def test_random_configurations_in_both_dtypes(seed, tmp_path):
    rng = np.random.default_rng(500 + seed)
    cfg = random_durelix(rng)
    folder = write_durelix(tmp_path, cfg, seed=seed)
    reqs = [rng.integers(0, cfg["vocab"], n).tolist() for n in (90, 17, 45, 3)]
    pm = plain.PlainDurelix(folder)
    truth = [pm.logits(t) for t in reqs]
    steps, expect, peak = traces.mixed(reqs, max_live=3, seed=seed)
    for dtype in ("float32", "bfloat16"):
        errors: list = []
        traces.compare(TraceReplayer(runner_for(folder, peak // 16, dtype, slots=3)).run_step, steps, expect, truth, 10.0, errors)
        if dtype == "float32":
            assert max(errors) < F32_TOL, (cfg, max(errors))
            continue
        # A choice that falls the other way moves its row and, through the recurrence's state, every later one of that request:
        # rows in front of a request's first close call are judged, in the yardstick as well.
        cut = [first_close_call(pm, t) for t in reqs]
        rough = plain.PlainDurelix(folder, bf16=True)
        rows = np.concatenate([np.abs(rough.logits(t) - w).max(-1)[:n] / np.abs(w).max(-1)[:n] for t, w, n in zip(reqs, truth, cut)])
        kept = [e for e, (i, p) in zip(errors, (at for exp in expect for at in exp)) if p < cut[i]]
        assert np.isfinite(errors).all() and len(kept) <= len(rows)
        if len(kept) > 20:
            check_rows(kept, dtype, (*(float(np.quantile(rows, q)) for q in (0.5, 0.9, 0.99)), 0))
