"""Zurolorn on the GPU: the kernels it brought, each against a plain float32 computation, and the
model in both dtypes against the plain implementation in tests/plain/zurolorn_plain.py: every cutting,
mixed batches on reused pages, contexts long enough for the attention kernels to cut their keys into
runs, captured decode steps, generation, and the programs a user starts."""

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
from plain import zurolorn_plain as plain
from prefixserve_amd.engine.replay import TraceReplayer
from prefixserve_amd.engine.runner import ModelRunner
from prefixserve_amd.parts.base import ScaledDelta
from test_zurolorn_host import SHARP, far_places, sharp
from zurolorn_configs import ZUROLORN, latent, layer, model, moe, write_zurolorn

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
DEV = "cuda:0"
F32_TOL = 3e-5
# bfloat16: a row's largest error over its largest logit, against the plain model with its products and
# activations rounded to bfloat16 (``bf16_bars``): the median and the ninth decile of a trace's rows, and
# how many rows lie far out. A router's close call (scores within CLOSE of another choice) falls the other way
# after rounding, in the yardstick as in the engine but not at the same token, and moves that row by tenths
# and one behind it a little; the plain model says how many such tokens there are.
BF16_FACTOR, BF16_TAIL_FACTOR, BF16_FAR_FACTOR, BF16_FAR_SHARE, CLOSE = 1.5, 2.5, 2.0, 0.03, 3e-3


@pytest.fixture(scope="module")
def ops():
    from prefixserve_amd.kernels.ops import HipOps
    from prefixserve_amd.parts.base import Workspace

    return HipOps(torch.device(DEV), Workspace(torch.device(DEV)))


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: write_zurolorn(tmp_path_factory.mktemp(f"zurolorn-{name}"), name) for name in ZUROLORN}


def rnd(*shape, dtype=torch.float32, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype).to(DEV)


def rel(got, want):
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    return float(np.abs(got - want).max() / max(np.abs(want).max(), 1e-30))


def f64(t):
    return t.double().cpu().numpy()


def runner_for(folder, pages, dtype, slots=4, graphs=False):
    return ModelRunner(folder, dtype=dtype, device=DEV, num_blocks=pages, max_seq_len=pages * 16, max_num_seqs=slots,
                       use_graphs=graphs)


# ------------------------------------------------------------------ kernels

@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("hidden", [64, 50, 1000, 2048, 4104, 9000])
@pytest.mark.parametrize("slices", [0, 1, 3, 9])
def test_sums_with_factors_per_column(ops, act, hidden, slices):
    """residual += factors * delta in the fused add + norm (whole and for picked rows) and in the plain sum."""
    t = 5
    resid, scale, w = rnd(t, hidden, seed=1), rnd(hidden, seed=2), 1 + rnd(hidden, seed=3, scale=0.1)
    delta = rnd(t, hidden, dtype=act, seed=4) if slices == 0 else rnd(slices, t, hidden, seed=4)
    whole = delta.float().sum(0) if slices else delta.float()
    want = resid.double() + scale.double() * whole.double()
    normed = want / torch.sqrt((want * want).mean(-1, keepdim=True) + 1e-5) * w.double()
    tol_out = 1e-5 if act == torch.float32 else 1e-2
    got, out = resid.clone(), torch.empty(t, hidden, dtype=act, device=DEV)
    ops.add_rmsnorm(got, ScaledDelta(delta, scale), w, 1e-5, out)
    assert rel(got.cpu(), want.cpu()) < 2e-6 and rel(out.float().cpu(), normed.cpu()) < tol_out
    rows = torch.tensor([3, 0, 3], dtype=torch.int32, device=DEV)
    kept, out = resid.clone(), torch.empty(3, hidden, dtype=act, device=DEV)
    ops.add_rmsnorm_rows(kept, ScaledDelta(delta, scale), rows, w, 1e-5, out)
    assert torch.equal(kept, resid) and rel(out.float().cpu(), normed[rows.long()].cpu()) < tol_out
    row = rnd(hidden, seed=5)
    got = resid.clone()
    ops.residual_add(got, ScaledDelta(delta, scale), row=row)
    assert rel(got.cpu(), (want + row.double()).cpu()) < 2e-6
    got = resid.clone()
    ops.residual_add(got, delta, row=row)
    assert rel(got.cpu(), (resid.double() + whole.double() + row.double()).cpu()) < 2e-6


@pytest.mark.parametrize("m,n,k", [(1, 64, 96), (8, 2048, 1024), (16, 320, 72), (5, 4096, 2048), (3, 40, 8)])
def test_a_small_product_into_the_stream_with_factors_per_column(ops, m, n, k):
    x, w = rnd(m, k, dtype=torch.bfloat16, seed=1), rnd(n, k, dtype=torch.bfloat16, seed=2, scale=0.1)
    resid, scale = rnd(m, n, seed=3), rnd(n, seed=4)
    got = resid.clone()
    res = ops.linear_to_residual(x, w, "t.delta", got, col_scale=scale)
    y = x.double() @ w.double().T
    if ops.fuses_norm(m, n, torch.bfloat16):
        assert res is None and rel(got.cpu(), (resid.double() + scale.double() * y).cpu()) < 1e-5
    else:
        assert torch.equal(got, resid)                      # handed back without the factors
        assert rel((res.float().sum(0) if res.dim() == 3 else res.float()).cpu(), y.cpu()) < 1e-2


def test_a_large_product_with_factors_is_handed_back(ops):
    """Where the library would add into the stream it cannot multiply columns: the output comes back instead."""
    m, n, k = 1100, 256, 128
    x, w = rnd(m, k, dtype=torch.bfloat16, seed=1), rnd(n, k, dtype=torch.bfloat16, seed=2, scale=0.1)
    resid = rnd(m, n, seed=3)
    got = resid.clone()
    res = ops.linear_to_residual(x, w, "t.delta2", got, col_scale=rnd(n, seed=4))
    assert torch.equal(got, resid) and rel(res.float().cpu(), (x.double() @ w.double().T).cpu()) < 1e-2


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("t,k,e,top,count,keep,factor", [(1, 96, 8, 3, 4, 2, 2.5), (9, 64, 12, 2, 3, 1, 1.0), (70, 128, 64, 8, 8, 4, 0.5),
                                                         (3, 200, 130, 8, 13, 5, 1.5), (333, 256, 40, 6, 40, 9, 2.0), (17, 100, 6, 6, 2, 2, 1.0),
                                                         (40, 64, 256, 4, 128, 70, 3.0), (64, 128, 320, 8, 5, 2, 1.2)])
def test_router_chooses_inside_the_best_groups(ops, act, t, k, e, top, count, keep, factor):
    x = rnd(t, k, dtype=act, seed=7)
    w = rnd(e, k, seed=8, scale=0.2).to(torch.bfloat16).float()
    if e // count >= 2:
        w[1] = w[0]                                                    # equal scores: the lower index wins
    chosen = torch.empty(t, top, dtype=torch.int32, device=DEV)
    weight = torch.empty(t, top, device=DEV)
    s = plain.sigmoid(f64(x) @ f64(w).T)
    for router in (w.to(act), None):                                   # product + choice; one kernel for both
        ops.moe_route(x, w, chosen, weight, router, groups=count, keep=keep, factor=factor)
        got = chosen.cpu().numpy()
        sums = np.sort(s.reshape(t, count, -1), axis=-1)[:, :, -2:].sum(-1)
        for i in range(t):
            assert len(set(got[i].tolist())) == top
            inside = {int(g) for g in got[i] // (e // count)}
            # groups and experts whose 32-bit sums differ by rounding alone may fall either way
            floor = np.sort(sums[i])[::-1][keep - 1] - 2e-6
            assert all(sums[i][g] >= floor for g in inside)
            want = plain.choose(s[i], top, {"count": count, "keep": keep})
            assert np.allclose(s[i][got[i]], s[i][want], atol=4e-6), i
            order = list(got[i])
            if 0 in order and 1 in order and e // count >= 2:
                assert order.index(0) < order.index(1)
        np.testing.assert_allclose(weight.cpu().numpy(), factor * np.take_along_axis(s, got.astype(np.int64), -1), rtol=1e-5, atol=1e-6)


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("t,k,f,e,top", [(1, 96, 40, 5, 2), (2, 64, 16, 3, 2), (9, 64, 56, 4, 3), (70, 128, 24, 9, 1), (4, 100, 33, 3, 3),
                                         (300, 128, 72, 6, 2), (40, 200, 64, 16, 4), (700, 64, 96, 2, 1), (8, 2048, 1024, 8, 4)])
def test_ungated_experts_into_slices_and_into_the_stream(ops, act, t, k, f, e, top):
    x = rnd(t, k, dtype=act, seed=9)
    up, down = rnd(e, f, k, dtype=act, seed=10, scale=0.15), rnd(e, k, f, dtype=act, seed=11, scale=0.15)
    gen = torch.Generator().manual_seed(12)
    chosen = torch.stack([torch.randperm(e, generator=gen)[:top] for _ in range(t)]).to(torch.int32).to(DEV)
    weight = (0.4 + 2.0 * torch.rand(t, top, generator=gen)).to(DEV)
    act_buf, out = torch.empty(t * top, f, dtype=act, device=DEV), torch.full((top, t, k), 3.0, device=DEV)
    ops.moe_experts(x, chosen, weight, up, down, act_buf, out, 0.0, 0.0, 0.0, weight_on_output=True, kind="squared_relu")
    want = torch.zeros(top, t, k, dtype=torch.float64, device=DEV)
    for ex in range(e):
        hidden = torch.relu(x.double() @ up[ex].double().T).square()
        y = hidden @ down[ex].double().T
        for j in range(top):
            rows = chosen[:, j] == ex
            want[j, rows] = weight[rows, j: j + 1].double() * y[rows]
    assert rel(out.cpu(), want.cpu()) < (1e-5 if act == torch.float32 else 2e-2)
    if act == torch.bfloat16 and t <= 70:
        resid, scale = rnd(t, k, seed=13), rnd(k, seed=14)
        for factors in (scale, None):
            got = resid.clone()
            ops.moe_experts(x, chosen, weight, up, down, act_buf, None, 0.0, 0.0, 0.0, weight_on_output=True, kind="squared_relu",
                            residual=got, col_scale=factors)
            total = out.double().sum(0) * (1.0 if factors is None else factors.double())
            assert rel((got - resid).cpu(), total.cpu()) < 1e-4


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m,heads,n,k", [(1, 3, 40, 24), (8, 2, 128, 256), (16, 5, 72, 192), (37, 2, 8, 70), (200, 5, 65, 17), (64, 1, 64, 64), (130, 3, 96, 320)])
def test_heads_product_with_a_gate(ops, act, m, heads, n, k):
    x, w = rnd(m, heads * (k + 8), dtype=act, seed=1), rnd(heads, n, k, dtype=act, seed=2, scale=0.2)
    gate = rnd(m, 5 + heads * n + 3, dtype=act, seed=3, scale=2.0)
    for gated in (True, False):
        out = torch.full((m, heads * n), 7.0, dtype=act, device=DEV)
        ops.heads_linear(x, 0, k + 8, w, out, 0, n, **({"gate": gate, "gate_offset": 5, "gate_head": n} if gated else {}))
        want = torch.cat([x[:, h * (k + 8): h * (k + 8) + k].double() @ w[h].double().T for h in range(heads)], dim=1)
        if gated:
            want = want * torch.sigmoid(gate[:, 5: 5 + heads * n].double())
        assert rel(out.float().cpu(), want.cpu()) < (1e-5 if act == torch.float32 else 1e-2)


def pairs_table(rot, base=30.0, positions=64):
    ang = torch.arange(positions, dtype=torch.float64)[:, None] * torch.tensor(plain.frequencies(rot, base))[None, :]
    return torch.stack([ang.cos(), ang.sin()], dim=-1).float().contiguous().to(DEV)


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("halves", [True, False])
@pytest.mark.parametrize("hq,dim,rot,rank,slots,c_rank", [(3, 12, 6, 20, 32, 18), (1, 8, 0, 16, 16, 40), (8, 64, 16, 96, 112, 300), (2, 0, 8, 24, 32, 7),
                                                          (5, 128, 64, 192, 256, 64)])
def test_latent_cache_write_and_queries(ops, act, halves, hq, dim, rot, rank, slots, c_rank):
    """The page, the queries' normed latent, and the query in the compressed space, from rows that hold
    [queries' latent | compressed | shared part | more]; and the form whose queries lie in the rows."""
    t, blocks = 67, 5
    rows = rnd(t, c_rank + rank + rot + 3, dtype=act, seed=1)
    w, cw = 1 + rnd(rank, seed=2, scale=0.2), 1 + rnd(c_rank, seed=3, scale=0.2)
    table = pairs_table(rot) if rot else None
    pos = torch.tensor(np.random.default_rng(1).integers(0, 64, t).astype(np.int32), device=DEV)
    kv = torch.full((blocks, 2, 1, 16 * slots), 9.0, dtype=act, device=DEV)
    ws = torch.tensor(np.random.default_rng(2).permutation(blocks * 16)[:t].astype(np.int32), device=DEV)
    c_q = torch.empty(t, c_rank, dtype=act, device=DEV)
    ops.latent_kv_append(rows, None, hq, dim, rot, rank, slots, pos, table, w, 1e-5, kv, ws, halves=halves, low_col=c_rank,
                         q_latent=(c_rank, cw, c_q))
    p = pos.cpu().numpy()
    turn = lambda v: plain.rotate(v, p, 30.0, halves) if rot else v
    low = f64(rows)[:, c_rank: c_rank + rank + rot]
    key, val = np.zeros((t, slots)), np.zeros((t, slots))
    key[:, :rank] = val[:, :rank] = plain.rms_norm(low[:, :rank], f64(w), 1e-5)
    key[:, rank: rank + rot] = turn(low[:, rank:])
    tol = 1e-5 if act == torch.float32 else 1e-2
    page, off = (ws // 16).long(), (ws % 16).long()
    assert rel(kv[:, 0].view(blocks, 16, slots)[page, off].float().cpu(), key) < tol
    assert rel(kv[:, 1].view(blocks, slots, 16)[page, :, off].float().cpu(), val) < tol
    assert int((kv != 9.0).sum()) <= 2 * t * slots                     # nothing else was written
    assert rel(c_q.float().cpu(), plain.rms_norm(f64(rows)[:, :c_rank], f64(cw), 1e-5)) < tol

    q, fold = rnd(t, hq * (dim + rot), dtype=act, seed=4), rnd(hq, rank, dim, dtype=act, seed=5, scale=0.2)
    want = np.zeros((t, hq, slots))
    heads = f64(q).reshape(t, hq, dim + rot)
    for h in range(hq):
        want[:, h, :rank] = heads[:, h, :dim] @ f64(fold)[h].T
    want[:, :, rank: rank + rot] = turn(heads[..., dim:])
    for count in (t, 16, 1):
        q_lat = torch.full((count, hq * slots), 5.0, dtype=act, device=DEV)
        ops.latent_query(q[:count].contiguous(), fold, q_lat, hq, dim, rot, rank, slots, pos[:count].contiguous(), table, halves=halves)
        assert rel(q_lat.float().view(count, hq, slots).cpu(), want[:count]) < tol
    both = torch.cat([q, rows[:, c_rank:]], dim=1).contiguous()
    q_lat = torch.full((t, hq * slots), 5.0, dtype=act, device=DEV)
    kv2 = torch.full_like(kv, 9.0)
    ops.latent_kv_append(both, q_lat, hq, dim, rot, rank, slots, pos, table, w, 1e-5, kv2, ws, halves=halves)
    assert torch.equal(kv2, kv)
    got = q_lat.float().view(t, hq, slots).cpu().numpy()
    assert np.all(got[:, :, :rank] == 5.0) and (slots == rank or rel(got[:, :, rank:], want[:, :, rank:]) < tol or rot == 0)


def test_kernels_refuse_what_they_do_not_take(ops):
    from prefixserve_amd.kernels.ops import KernelError

    x, i32 = rnd(2, 64), dict(dtype=torch.int32, device=DEV)
    for count, keep, top in ((3, 1, 1), (4, 5, 1), (4, 1, 3)):
        with pytest.raises(KernelError):
            ops.moe_route(x, rnd(8, 64), torch.empty(2, top, **i32), torch.empty(2, top, device=DEV), groups=count, keep=keep)
    with pytest.raises(KernelError):
        ops.moe_route(x, rnd(8, 64), torch.empty(2, 1, **i32), torch.empty(2, 1, device=DEV), mode=1, groups=2, keep=1)
    with pytest.raises(KernelError):                                   # a 32-bit step keeps its slices
        ops.moe_experts(x, torch.zeros(2, 1, **i32), torch.ones(2, 1, device=DEV), rnd(2, 8, 64), rnd(2, 64, 8), torch.empty(2, 8, device=DEV),
                        None, 0.0, 0.0, 0.0, kind="squared_relu", residual=x.clone())
    with pytest.raises(KernelError):
        ops.residual_add(x.clone(), ScaledDelta(rnd(2, 64), rnd(32)))
    with pytest.raises(KernelError):
        ops.heads_linear(x, 0, 32, rnd(2, 8, 32), torch.empty(2, 16, device=DEV), 0, 8, gate=rnd(2, 15), gate_head=8)
    with pytest.raises(KernelError):
        ops.latent_query(x, rnd(2, 16, 24), torch.empty(2, 64, device=DEV), 2, 24, 8, 16, 32, torch.zeros(2, **i32), None)


# ------------------------------------------------------------------ whole models

LENGTHS = [70, 33, 97, 18, 64, 45, 1, 52, 2, 81, 29, 3]


def bf16_bars(folder, truth, reqs, last=0):
    """(median, ninth decile, 99th percentile) of the rows (the ``last`` ones of each request, or all) of a
    plain bfloat16 run against the plain model in float64, and the number of close calls."""
    rough = plain.PlainZurolorn(folder, bf16=True)
    rows = np.concatenate([np.abs(rough.logits(t)[-last:] - w[-last:]).max(-1) / np.abs(w[-last:]).max(-1) for t, w in zip(reqs, truth)])
    close = sum(plain.PlainZurolorn(folder).close_calls(t, CLOSE, last) for t in reqs)
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
@pytest.mark.parametrize("name", list(ZUROLORN))
def test_every_cutting_matches_the_plain_model(name, dtype, folders):
    rng = np.random.default_rng(4)
    reqs = [rng.integers(0, ZUROLORN[name]["vocab"], n).tolist() for n in LENGTHS]
    pm = plain.PlainZurolorn(folders[name])
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
    rp = TraceReplayer(small)
    errors = []
    traces.compare(rp.run_step, steps, expect, truth, 10.0, errors)
    check_rows(errors, dtype, bars)
    assert all(rp.cache.num_free(g) == peak // 16 for g in range(rp.cache.num_groups))


def test_cuttings_agree_with_each_other_in_32_bit(folders):
    """A position's 32-bit logits do not depend on how its prompt was cut, beyond rounding."""
    toks = np.random.default_rng(8).integers(0, 96, 90).tolist()
    runner = runner_for(folders["A"], 16, "float32")
    rows = {}
    for build in (traces.whole, traces.decode_tail, traces.portions):
        steps, expect = build([toks])
        rp = TraceReplayer(runner)
        got = np.concatenate([r for r in (rp.run_step(s) for s in steps) if r is not None])
        rows[build.__name__] = {p: got[k] for k, (_, p) in enumerate(e for exp in expect for e in exp)}
    for p in rows["decode_tail"]:
        assert rel(rows["decode_tail"][p], rows["whole"][p]) < 5e-6 and rel(rows["portions"][p], rows["whole"][p]) < 5e-6


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_contexts_and_far_keys(dtype, tmp_path):
    """2,100 keys, so that the decode attention and the attention of a short portion cut their keys into
    runs, under scores with which single keys hundreds of tokens back carry the weight; a prompt, a portion
    of twenty tokens behind it, and decoding, also two requests side by side on interleaved pages."""
    folder = write_zurolorn(tmp_path, SHARP, seed=6, std=0.3, edit=sharp)
    toks = np.random.default_rng(5).integers(0, 48, 2110).tolist()
    other = np.random.default_rng(6).integers(0, 48, 40).tolist()
    pm = plain.PlainZurolorn(folder)
    truth = [pm.logits(toks), pm.logits(other)]
    assert len([f for f in far_places(pm, toks, back=500) if f[0] >= 2080]) >= 2
    runner = runner_for(folder, 140, dtype)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:1000], "want": [100, 999]}, {"id": "b", "tokens": other[:17], "want": [16]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[1000:2080], "want": [1079]}, {"id": "b", "tokens": other[17:20], "want": [2]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[2080:2100], "want": list(range(20))}], "end": []}]
    expect = [[(0, 100), (0, 999), (1, 16)], [(0, 2079), (1, 19)], [(0, p) for p in range(2080, 2100)]]
    for i in range(10):
        steps.append({"step": 3 + i, "entries": [{"id": "a", "tokens": [toks[2100 + i]], "want": [0]}, {"id": "b", "tokens": [other[20 + i]], "want": [0]}],
                      "end": []})
        expect.append([(0, 2100 + i), (1, 20 + i)])
    errors: list = []
    traces.compare(TraceReplayer(runner).run_step, steps, expect, truth, 10.0, errors)
    check_rows(errors, dtype, bf16_bars(folder, truth, [toks, other], last=40) if dtype == "bfloat16" else None, tol=1e-4)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes_at_the_kernels_limits(dtype, tmp_path):
    """A cache entry of 256 and ones wider than the matrix-core attention takes (332 and 576 numbers), a queries'
    latent wider than the model, 256 experts in 128 groups, a head of 256 value dimensions."""
    cfg = model(90, 128, 1e-5, 2.0, 1.0, [layer(latent(2, 64, 64, 256, 192, 0.1, 1e4), moe(256, 6, 16, 2.0, (128, 5))),
                                          layer(latent(3, 32, 32, 16, 300, 0.1, 1e4, q_rank=200), moe(2, 2, 200, 1.0, (1, 1))),
                                          layer(latent(2, 16, 64, 16, 512, 0.1, 1e4), None)])
    folder = write_zurolorn(tmp_path, cfg, seed=9)
    toks = np.random.default_rng(5).integers(0, 90, 60).tolist()
    truth = plain.PlainZurolorn(folder).logits(toks)
    steps, expect = traces.decode_tail([toks], tail=12)
    errors: list = []
    traces.compare(TraceReplayer(runner_for(folder, 8, dtype)).run_step, steps, expect, [truth], 10.0, errors)
    check_rows(errors, dtype, bf16_bars(folder, [truth], [toks]) if dtype == "bfloat16" else None)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes_that_are_multiples_of_nothing(dtype, tmp_path):
    """A width of 90, a vocabulary of 77, inner sizes of 13 and 7, heads of 5, 9 and 11 numbers, latents of 19
    and 3: the products' and the norms' narrow forms, rows that start at odd addresses."""
    cfg = model(77, 90, 1e-6, 1.3, 0.9, [layer(latent(3, 5, 2, 9, 19, 0.5, 30.0), moe(6, 2, 13, 1.1, (2, 1))),
                                         layer(latent(2, 11, 6, 5, 7, 0.4, 900.0, q_rank=3), moe(5, 5, 7)),
                                         layer(latent(1, 9, 10, 11, 3, 0.4, 900.0), None)], loop=(1, 3, 2))
    folder = write_zurolorn(tmp_path, cfg, seed=13)
    rng = np.random.default_rng(5)
    reqs = [rng.integers(0, 77, n).tolist() for n in (75, 40, 9)]
    pm = plain.PlainZurolorn(folder)
    truth = [pm.logits(t) for t in reqs]
    steps, expect, peak = traces.mixed(reqs, max_live=3, seed=1)
    errors: list = []
    traces.compare(TraceReplayer(runner_for(folder, peak // 16, dtype, slots=3)).run_step, steps, expect, truth, 10.0, errors)
    check_rows(errors, dtype, bf16_bars(folder, truth, reqs) if dtype == "bfloat16" else None)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decoding_through_graphs(dtype, folders):
    """Two requests decode side by side through captured steps, then one alone (another graph), for a hundred
    and twenty tokens."""
    rng = np.random.default_rng(3)
    reqs = [rng.integers(0, 96, n).tolist() for n in (140, 155)]
    pm = plain.PlainZurolorn(folders["A"])
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


@pytest.mark.parametrize("batch", [3, 12, 20, 40])
def test_decode_batches_of_every_form(batch, folders):
    """Up to 16 tokens a step adds into the stream and normalizes in the products; above, norm kernels and slices."""
    rng = np.random.default_rng(batch)
    reqs = [rng.integers(0, 70, int(n)).tolist() for n in rng.integers(6, 30, batch)]
    pm = plain.PlainZurolorn(folders["C"])
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
    """Portions under a budget, few pages, a shared prefix; in bfloat16 ``warm_up()`` and eight decode steps a round too."""
    from prefixserve_amd.engine.engine import Engine, EngineConfig
    from prefixserve_amd.generation import generate

    pm = plain.PlainZurolorn(folders["D"])
    rng = np.random.default_rng(12)
    head = rng.integers(0, 52, 32).tolist()
    prompts = [head + [1, 2]] + [rng.integers(0, 52, n).tolist() for n in (5, 23, 40, 9)] + [head + [3, 4, 5]]
    eng = Engine(EngineConfig(model_path=str(folders["D"]), dtype=dtype, max_num_seqs=3, max_prefill_tokens=16,
                              max_seq_len=128, num_blocks=16, **({"decode_steps": 8} if dtype == "bfloat16" else {})))
    if dtype == "bfloat16":
        eng.warm_up()
    outs, _ = generate(eng, prompts, 12, temperature=0.0, ignore_eos=True)
    if dtype == "float32":
        for p, o in zip(prompts, outs):
            assert list(o.tokens) == pm.greedy(p, 12)
    else:
        rough = bf16_bars(folders["D"], [pm.logits(p) for p in prompts], prompts)[2]
        for p, o in zip(prompts, outs):                     # every token is the plain model's best, or as good to within rounding
            rows = pm.logits(p + list(o.tokens))[len(p) - 1: -1]
            for row, tok in zip(rows, o.tokens):
                assert row.max() - row[tok] <= 4.0 * rough * np.abs(row).max()
    assert outs[-1].cached_tokens == 32


def test_trace_run_and_the_command_line_as_programs(folders, tmp_path):
    rng = np.random.default_rng(7)
    reqs = [rng.integers(0, 96, n).tolist() for n in (40, 70, 25, 90, 33)]
    pm = plain.PlainZurolorn(folders["A"])
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
    prompt = [5, 17, 3, 90, 41, 7, 7, 19, 0, 64, 11]
    proc = subprocess.run(
        [sys.executable, "-m", "prefixserve_amd.cli", "generate", "--model", str(folders["A"]), "--dtype", "float32",
         "--max-seq-len", "128", "--num-blocks", "16", "--max-running-requests", "2", "--chunked-prefill-size", "5",
         "--max-tokens", "6", "--ignore-eos", "--prompt-ids", ",".join(map(str, prompt))],
        capture_output=True, text=True, cwd=ROOT, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert json.loads(proc.stdout.strip().splitlines()[-1])["outputs"][0]["tokens"] == pm.greedy(prompt, 6)


def random_zurolorn(rng) -> dict:
    """A configuration drawn at random: widths that are no multiples of 16, one to five layers of both kinds, any
    repeated stretch or none, any grouping of the experts or none."""
    width = int(rng.choice([40, 72, 100, 136]))
    layers = []
    for _ in range(int(rng.integers(1, 6))):
        rot = int(rng.choice([0, 2, 8, 16, 20]))
        dim = int(rng.choice([8, 12, 32, 50] if rot == 0 else [0, 4, 16, 24, 40]))
        mixer = latent(int(rng.integers(1, 6)), dim, rot, int(rng.choice([4, 16, 20, 48])), int(rng.choice([5, 16, 40, 64, 100])),
                       float(rng.choice([0.1, 0.3, 0.6])), float(rng.choice([20.0, 1e4, 1e6])),
                       q_rank=None if rng.random() < 0.5 else int(rng.choice([6, 24, 64, 90])))
        mlp = None
        if rng.random() < 0.8:
            count, per = int(rng.choice([1, 2, 3, 5])), int(rng.choice([1, 2, 4, 7]))
            keep = int(rng.integers(1, count + 1))
            mlp = moe(count * per, int(rng.integers(1, keep * per + 1)), int(rng.choice([8, 20, 24, 40])), float(rng.choice([1.0, 0.5, 2.5])),
                      (count, keep) if rng.random() < 0.7 else None)
        layers.append(layer(mixer, mlp))
    loop = None
    if rng.random() < 0.6:
        start = int(rng.integers(0, len(layers)))
        loop = (start, int(rng.integers(start + 1, len(layers) + 1)), int(rng.integers(1, 4)))
    return model(int(rng.choice([50, 131, 256])), width, float(rng.choice([1e-5, 1e-6])), float(rng.choice([1.0, 4.0])), float(rng.choice([0.3, 1.0, 2.0])),
                 layers, loop)


@pytest.mark.parametrize("seed", range(10))
def test_random_configurations_in_both_dtypes(seed, tmp_path):
    rng = np.random.default_rng(300 + seed)
    cfg = random_zurolorn(rng)
    folder = write_zurolorn(tmp_path, cfg, seed=seed)
    reqs = [rng.integers(0, cfg["vocab"], n).tolist() for n in (90, 17, 45, 3)]
    pm = plain.PlainZurolorn(folder)
    truth = [pm.logits(t) for t in reqs]
    steps, expect, peak = traces.mixed(reqs, max_live=3, seed=seed)
    for dtype in ("float32", "bfloat16"):
        errors: list = []
        traces.compare(TraceReplayer(runner_for(folder, peak // 16, dtype, slots=3)).run_step, steps, expect, truth, 10.0, errors)
        if dtype == "float32":
            assert max(errors) < F32_TOL, (cfg, max(errors))
        else:
            check_rows(errors, dtype, bf16_bars(folder, truth, reqs))
