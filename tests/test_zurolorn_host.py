"""Zurolorn on the host: its configuration, the model built from it, and the whole engine path
(packing, pages, the repeated stretch, replay, scheduler, prefix cache, generation) with the kernel
library's CPU stand-in, against the plain implementation in tests/plain/zurolorn_plain.py."""

from __future__ import annotations

import copy
import math

import numpy as np
import pytest
import torch

import traces
from emulated_ops import EmulatedOps
from plain import zurolorn_plain as plain
from prefixserve_amd.config import UnsupportedModelError, ZurolornConfig, read_model_dir
from prefixserve_amd.engine.batch import StepItem
from prefixserve_amd.engine.replay import TraceReplayer
from prefixserve_amd.engine.runner import ModelRunner
from prefixserve_amd.models.zurolorn import build_zurolorn_spec
from prefixserve_amd.parts.base import Runtime, ScaledDelta, Workspace
from prefixserve_amd.parts.moe import RoutedExperts
from prefixserve_amd.weights import WeightLoadError, load_weights
from zurolorn_configs import ZUROLORN, latent, layer, model, moe, spread_scales, write_zurolorn

TOL = 3e-5


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: write_zurolorn(tmp_path_factory.mktemp(f"zurolorn-{name}"), name) for name in ZUROLORN}


def runner_for(folder, pages, dtype="float32", slots=4):
    return ModelRunner(folder, dtype=dtype, device="cpu", num_blocks=pages, max_seq_len=pages * 16, max_num_seqs=slots,
                       use_graphs=False, ops=EmulatedOps())


def whole(runner, toks, want=None):
    want = list(range(len(toks))) if want is None else want
    return TraceReplayer(runner).run_step({"step": 0, "entries": [{"id": "a", "tokens": list(toks), "want": want}], "end": ["a"]})


def close(got, want, tol=TOL):
    return float(np.abs(got - want).max()) <= tol * float(np.abs(want).max())


# ------------------------------------------------------------------ configuration and spec

def test_configuration_reads_every_key_and_refuses_what_it_does_not_know():
    cfg = ZurolornConfig.from_dicts(ZUROLORN["A"])
    assert (cfg.vocab_size, cfg.hidden_size, cfg.norm_eps, cfg.embedding_scale, cfg.logit_scale) == (96, 64, 1e-5, 3.0, 0.5)
    assert (cfg.loop.start, cfg.loop.stop, cfg.loop.times) == (1, 3, 3)
    m, two, e = cfg.layers[0].mixer, cfg.layers[1].mixer, cfg.layers[0].mlp
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale, m.rot_base, m.q_rank) == (4, 16, 8, 24, 40, 0.3, 500.0, None)
    assert two.q_rank == 48 and cfg.layers[1].mlp is None
    assert (e.experts, e.top, e.ff, e.scale, e.groups, e.keep) == (8, 3, 24, 1.5, 4, 2)
    for name in ZUROLORN:
        one = ZurolornConfig.from_dicts(ZUROLORN[name])
        assert ZurolornConfig.from_dicts(one.to_config_json()) == one
    assert ZurolornConfig.from_dicts(ZUROLORN["B"]).loop is None and ZurolornConfig.from_dicts(ZUROLORN["B"]).layers[1].mlp.groups is None
    for path, value in [(("layers", 0, "mixer", "q_rank"), 8), (("layers", 0, "mlp", "kind"), "dense"), (("layers", 0, "type"), "attention"),
                        (("layers", 0, "mixer", "rot", "dims"), 6), (("layers", 0, "mixer", "rot", "scaling"), {}), (("loop", "stop"), 9),
                        (("loop", "times"), 0), (("sink",), True), (("layers", 0, "mixer", "mask"), {"size": 4}),
                        (("layers", 0, "mlp", "router", "groups", "count"), 3), (("layers", 0, "mlp", "router", "groups", "keep"), 5),
                        (("layers", 2, "mlp", "router", "top"), 3), (("layers", 0, "mlp", "shared"), {"ff": 8}),
                        (("layers", 0, "mixer", "heads"), 0), (("layers", 1, "mixer", "q_rank"), 0)]:
        raw = copy.deepcopy(ZUROLORN["A"])
        at = raw
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        with pytest.raises(UnsupportedModelError):
            ZurolornConfig.from_dicts(raw)


def test_a_repeated_stretch_is_listed_once_per_pass_with_caches_of_its_own(folders):
    spec = build_zurolorn_spec(read_model_dir(folders["A"])[1])
    assert [(r.layer, r.before, r.pass_index) for r in spec.order] == [
        (0, (), 0), (1, ("pass",), 0), (2, (), 0), (1, ("pass",), 1), (2, (), 1), (1, ("pass",), 2), (2, (), 2), (3, (), 0)]
    assert sorted(r.cache for r in spec.order) == list(range(8)) and all(r.writes_cache for r in spec.order)
    runner = runner_for(folders["A"], 8)
    # entries of 48 (40 + 8), 48 (24 + 16), 32 (16 + 12), 32 (20 + 6): two layer groups, nothing kept in slots, no window
    assert sorted(len(g.entries) for g in runner.layer_groups) == [4, 4] and not runner.model.state_needs()
    assert runner.windows == [None, None] and runner.state_bytes_per_slot == 0
    assert not build_zurolorn_spec(read_model_dir(folders["B"])[1]).stream_transforms
    assert [r.before for r in build_zurolorn_spec(read_model_dir(folders["C"])[1]).order] == [("pass",), ()]
    assert [(r.layer, r.pass_index) for r in build_zurolorn_spec(read_model_dir(folders["D"])[1]).order] == [(0, 0), (1, 0), (1, 1)]


def test_weights_are_checked_by_name_and_shape(folders):
    arch, cfg, _ = read_model_dir(folders["A"])
    from prefixserve_amd.parts.model import DecoderModel

    want = DecoderModel(arch.build_spec(cfg)).weights()
    assert want["l0.mix.g"].shape == (96, 64) and want["l1.mix.uq"].shape == (80, 48) and want["loop.step"].shape == (3, 64)
    assert "l0.mlp.e0.gate" not in want and "l1.norm2" not in want and "l1.ls2" not in want and "l1.ls1" in want
    wrong = {**want, "l0.mix.q": want["l0.mix.dkv"], "l7.norm1": want["l0.norm1"]}
    with pytest.raises(WeightLoadError) as err:
        load_weights(folders["A"], wrong)
    assert err.value.missing == ["l7.norm1"] and [n for n, _, _ in err.value.wrong_shape] == ["l0.mix.q"]


def test_a_layer_without_feed_forward_ignores_a_norm_and_a_scale_that_nothing_reads(tmp_path):
    from safetensors.torch import load_file, save_file

    folder = write_zurolorn(tmp_path, "A")
    toks = np.random.default_rng(2).integers(0, 96, 20).tolist()
    want = whole(runner_for(folder, 4), toks)
    tensors = load_file(str(folder / "model.safetensors"))
    tensors["l1.norm2"], tensors["l1.ls2"] = torch.full((64,), 5.0), torch.full((64,), 7.0)
    save_file(tensors, str(folder / "model.safetensors"))
    assert np.array_equal(whole(runner_for(folder, 4), toks), want)


# ------------------------------------------------------------------ mechanisms, one at a time

def test_the_plain_mechanisms_agree_with_their_definitions_written_out():
    """The oracle's own functions against the equations entry by entry."""
    rng = np.random.default_rng(5)
    x = rng.normal(size=(3, 6))
    for halves in (True, False):
        got = plain.rotate(x, np.array([0, 4, 11]), 50.0, halves)
        for t, p in enumerate((0, 4, 11)):
            for i in range(3):
                a = p * 50.0 ** (-2.0 * i / 6)
                u, v = (i, i + 3) if halves else (2 * i, 2 * i + 1)
                assert math.isclose(got[t, u], x[t, u] * math.cos(a) - x[t, v] * math.sin(a), abs_tol=1e-12)
                assert math.isclose(got[t, v], x[t, v] * math.cos(a) + x[t, u] * math.sin(a), abs_tol=1e-12)
    m = {"heads": 2, "dim": 2, "rot_dim": 4, "vdim": 3, "kv_rank": 5, "scale": 0.7, "rot": {"base": 9.0, "dims": 4}}
    h = rng.normal(size=(4, 6))
    shared = {"dkv": rng.normal(size=(9, 6)), "dkv.norm": rng.normal(size=5), "uk": rng.normal(size=(4, 5)), "uv": rng.normal(size=(6, 5)),
              "o": rng.normal(size=(6, 6))}
    for w in ({**shared, "q": rng.normal(size=(12, 6)), "g": rng.normal(size=(6, 6))},
              {**shared, "dq": rng.normal(size=(7, 6)), "dq.norm": rng.normal(size=7), "uq": rng.normal(size=(12, 7))}):
        halves = "q" in w
        got = plain.latent_attention(h, np.arange(4), w, m, 1e-6, halves)
        turn = lambda v, p: plain.rotate(v[None], np.array([p]), 9.0, halves)[0]
        norm = lambda v, g: v / math.sqrt((v * v).mean() + 1e-6) * g
        for i in range(4):
            out = np.zeros(6)
            q = w["q"] @ h[i] if halves else w["uq"] @ norm(w["dq"] @ h[i], w["dq.norm"])
            for a in range(2):
                qa = q[6 * a: 6 * a + 6]
                scores, vals = [], []
                for j in range(i + 1):
                    d = w["dkv"] @ h[j]
                    c = norm(d[:5], w["dkv.norm"])
                    scores.append(0.7 * (qa[:2] @ (w["uk"] @ c)[2 * a: 2 * a + 2] + turn(qa[2:], i) @ turn(d[5:], j)))
                    vals.append((w["uv"] @ c)[3 * a: 3 * a + 3])
                p = np.exp(scores) / np.exp(scores).sum()
                out[3 * a: 3 * a + 3] = sum(pj * vj for pj, vj in zip(p, vals))
            if halves:
                out = out / (1 + np.exp(-(w["g"] @ h[i])))
            assert np.allclose(got[i], w["o"] @ out, rtol=1e-10, atol=1e-12)
    up, down = rng.normal(size=(5, 6)), rng.normal(size=(6, 5))
    z = up @ h[0]
    assert np.allclose(plain.expert(h[0], up, down), down @ np.where(z > 0, z * z, 0.0))


def test_the_choice_inside_groups_by_hand():
    s = np.array([0.9, 0.1, 0.2, 0.6, 0.5, 0.5, 0.4, 0.3])          # groups of two: 1.0, 0.8, 1.0, 0.7
    assert plain.choose(s, 2, {"count": 4, "keep": 1}).tolist() == [0, 1]            # equal groups: the first
    assert plain.choose(s, 3, {"count": 4, "keep": 2}).tolist() == [0, 4, 5]         # expert 3 is better than 4, but its group is not kept
    assert plain.choose(s, 3, None).tolist() == [0, 3, 4]
    assert plain.choose(s, 3, {"count": 2, "keep": 1}).tolist() == [0, 3, 2]         # groups of four: 1.5 and 1.0, the two largest alone
    assert plain.choose(s, 2, {"count": 8, "keep": 3}).tolist() == [0, 3]            # groups of one
    chosen, weight = plain.route(np.eye(8), np.log(s / (1 - s))[:, None] * np.ones((8, 8)), {"top": 2, "scale": 2.5})
    assert chosen.tolist() == [[0, 3]] * 8 and np.allclose(weight, [2.25, 1.5])


@pytest.mark.parametrize("experts,top,groups", [(8, 2, (4, 2)), (8, 3, None), (12, 4, (3, 2)), (6, 2, (6, 3)), (9, 9, (3, 3)), (16, 1, (2, 1))])
@pytest.mark.parametrize("scale", [1.0, 2.5])
def test_routed_experts_alone(experts, top, groups, scale):
    """The part against the plain mixture: choice, weights and output."""
    names = {"router": "router", "up": "e{e}.up", "down": "e{e}.down"}
    part = RoutedExperts(20, experts, top, 12, names, expert="squared_relu", weight_on="output", weight_scale=scale,
                         groups=None if groups is None else {"count": groups[0], "keep": groups[1]})
    rng = np.random.default_rng(experts + top)
    w = {name: rng.normal(size=want.shape) * 0.4 for name, want in part.weights().items()}
    rt = Runtime(torch.device("cpu"), torch.float32, EmulatedOps(), Workspace(torch.device("cpu")))
    rt.ops.ws = rt.workspace
    part.bind({k: torch.tensor(v, dtype=torch.float32) for k, v in w.items()}, rt)
    h = rng.normal(size=(33, 20)).astype(np.float32)
    ctx = type("Ctx", (), {"residual": None})()
    got = part.forward(torch.tensor(h), ctx).sum(0).numpy()
    r = {"top": top, "scale": scale, "groups": None if groups is None else {"count": groups[0], "keep": groups[1]}}
    assert close(got, plain.mixture(h.astype(np.float64), w, r))


def test_experts_refuse_groups_that_do_not_fit():
    names = {"router": "r", "up": "u{e}", "down": "d{e}", "gate": "g{e}"}
    for kw in ({"groups": {"count": 3, "keep": 1}}, {"groups": {"count": 4, "keep": 5}}, {"groups": {"count": 4, "keep": 1}, "top_k": 3},
               {"groups": {"count": 4, "keep": 2}, "score": "softmax_of_chosen"}, {"expert": "relu"}):
        args = {"top_k": 2, **kw}
        with pytest.raises(ValueError):
            RoutedExperts(16, 8, intermediate_size=8, names=names, **args)


ONE_LAYER = {
    "direct": latent(3, 12, 6, 10, 20, 0.4, 300.0), "direct-one-head": latent(1, 8, 8, 24, 8, 0.6, 10000.0),
    "direct-no-rotation": latent(2, 16, 0, 8, 12, 0.4, 1.0), "direct-all-rotated": latent(2, 0, 12, 8, 12, 0.4, 40.0),
    "latent-queries": latent(3, 12, 6, 10, 20, 0.4, 300.0, q_rank=18), "latent-queries-rank-one": latent(2, 8, 4, 6, 1, 0.5, 90.0, q_rank=3),
}


@pytest.mark.parametrize("kind", list(ONE_LAYER))
@pytest.mark.parametrize("ff", [None, moe(6, 2, 24, 1.7, (3, 2))])
def test_each_mixer_alone(kind, ff, tmp_path):
    """A model of one layer: whatever differs from the plain model is that mixer's (or the block's)."""
    folder = write_zurolorn(tmp_path, model(50, 32, 1e-5, 2.0, 3.0, [layer(ONE_LAYER[kind], ff)]), seed=8)
    toks = np.random.default_rng(1).integers(0, 50, 45).tolist()
    assert close(whole(runner_for(folder, 4), toks), plain.PlainZurolorn(folder).logits(toks))


def test_a_block_hands_a_scaled_output_to_whoever_adds_it(folders):
    """The factors per column reach the sum whether the feed-forward hands its output back or there is none."""
    runner = runner_for(folders["A"], 8)
    seen = []
    for blk in runner.model.blocks:
        inner = blk.forward
        blk.forward = lambda *a, _inner=inner, **kw: seen.append(_inner(*a, **kw)) or seen[-1]
    whole(runner, [1, 2, 3])
    assert len(seen) == 8 and all(isinstance(s, ScaledDelta) for s in seen)
    assert seen[0].delta.dim() == 3 and seen[1].delta.dim() == 2             # experts' slices; a mixer's rows


# ------------------------------------------------------------------ whole models

LENGTHS = [70, 33, 97, 18, 64, 45, 1, 52, 2, 81, 29, 3]


@pytest.mark.parametrize("name", list(ZUROLORN))
def test_every_cutting_matches_the_plain_model_on_the_host(name, folders):
    rng = np.random.default_rng(4)
    reqs = [rng.integers(0, ZUROLORN[name]["vocab"], n).tolist() for n in LENGTHS]
    pm = plain.PlainZurolorn(folders[name])
    truth = [pm.logits(t) for t in reqs]
    runner = runner_for(folders[name], 32)
    for build in (traces.whole, traces.decode_tail, traces.portions):
        steps, expect = build(reqs)
        assert traces.compare(TraceReplayer(runner).run_step, steps, expect, truth, TOL) < TOL
    steps, expect, peak = traces.mixed(reqs, max_live=3, seed=2)
    assert sum(len(r) for r in reqs) > 1.3 * peak
    small = runner_for(folders[name], peak // 16, slots=3)
    for t in small.pools.tensors:
        t.fill_(1e30)                                       # a page that is used again never holds zeros
    rp = TraceReplayer(small)
    assert traces.compare(rp.run_step, steps, expect, truth, TOL) < TOL
    assert all(rp.cache.num_free(g) == peak // 16 for g in range(rp.cache.num_groups))


@pytest.mark.parametrize("name", list(ZUROLORN))
def test_layers_follow_the_plain_model_one_by_one(name, folders):
    """The stream behind every run of a layer: a fault shows in the run that makes it."""
    toks = np.random.default_rng(9).integers(0, ZUROLORN[name]["vocab"], 37).tolist()
    want = plain.PlainZurolorn(folders[name]).hidden(toks, every_layer=True)
    runner = runner_for(folders[name], 8)
    seen = []
    for blk in runner.model.blocks:
        inner = blk.forward

        def forward(residual, *a, _inner=inner, **kw):
            out = _inner(residual, *a, **kw)
            seen.append((residual + EmulatedOps._whole(out) if out is not None else residual).clone().numpy())
            return out

        blk.forward = forward
    tables = [[0, 1, 2]] * len(runner.layer_groups)
    runner.step([StepItem(key="a", tokens=toks, start=0, block_tables=tables, slot=0, want=[36])])
    assert len(seen) == len(want)
    for i, (got, exp) in enumerate(zip(seen, want)):
        assert close(got, exp), f"run {i}"


def test_faults_would_show(tmp_path):
    """Each fault in one mechanism, planted in the plain model, moves the logits by a hundred tolerances."""
    cfg = model(60, 32, 1e-5, 2.0, 1.7, [layer(latent(2, 8, 8, 12, 16, 1.0, 60.0), moe(8, 2, 16, 1.6, (4, 2))),
                                         layer(latent(3, 8, 4, 8, 12, 1.0, 40.0, q_rank=10), moe(6, 2, 16, 1.3, (3, 1)))], loop=(0, 1, 2))
    folder = write_zurolorn(tmp_path, cfg, seed=2, std=0.3)
    toks = np.random.default_rng(3).integers(0, 60, 60).tolist()
    truth = plain.PlainZurolorn(folder).logits(toks)
    assert close(whole(runner_for(folder, 4), toks), truth)

    def moved(change) -> float:
        other = plain.PlainZurolorn(folder)
        change(other)
        return float(np.abs(other.logits(toks) - truth).max() / np.abs(truth).max())

    def tensor(name, f):
        return lambda m: m.w.__setitem__(name, f(m.w[name]))

    def key(path, value):
        def change(m):
            at = m.cfg
            for k in path[:-1]:
                at = at[k]
            at[path[-1]] = value
        return change

    mix = lambda i, k, v: key(("layers", i, "mixer", k), v)
    router = lambda i, k, v: key(("layers", i, "mlp", "router", k), v)
    changes = {
        "gate": tensor("l0.mix.g", lambda t: t * 0), "norm of c": tensor("l0.mix.dkv.norm", np.ones_like),
        "norm of the queries' latent": tensor("l1.mix.dq.norm", np.ones_like), "mixer's factors": tensor("l0.ls1", np.ones_like),
        "experts' factors": tensor("l1.ls2", np.ones_like), "a pass's row": tensor("loop.step", lambda t: t[::-1]),
        "no rows": tensor("loop.step", lambda t: t * 0), "one pass more": lambda m: (key(("loop", "times"), 3)(m), tensor("loop.step", lambda t: t[[0, 1, 1]])(m)),
        "base": mix(0, "rot", {"base": 75.0, "dims": 8}), "scale": mix(1, "scale", 1.06), "router's scale": router(0, "scale", 1.7),
        "kept groups": router(0, "groups", {"count": 4, "keep": 3}), "other groups": router(1, "groups", {"count": 2, "keep": 1}),
        "no groups": router(1, "groups", None), "embedding": key(("embedding", "scale"), 2.1), "logits": key(("logit_scale",), 1.72),
        "eps": lambda m: setattr(m, "eps", 0.05),
    }
    for name, change in changes.items():
        assert moved(change) > 100 * TOL, name
    for kind in ("latent_attention", "latent_attention_2"):
        plain.HALVES[kind] ^= True                          # the other pairing of the rotation
        try:
            assert moved(lambda m: None) > 100 * TOL, kind
        finally:
            plain.HALVES[kind] ^= True


def sharp(tensors):
    """Queries and compressed vectors large: single keys carry the softmax."""
    spread_scales(tensors)
    for name, t in tensors.items():
        if name.endswith((".uk", ".mix.q", ".mix.uq")):
            t.mul_(2.0)


SHARP = model(48, 32, 1e-5, 3.0, 1.0, [layer(latent(2, 16, 4, 12, 24, 1.2, 1e4), None), layer(latent(2, 16, 4, 8, 24, 1.2, 1e4, q_rank=24), moe(4, 1, 16))])


def far_places(pm, toks, back=200):
    """(query, key) places of head 0 of layer 0 that carry more than half the weight from more than ``back`` tokens back."""
    m, w = pm.cfg["layers"][0]["mixer"], pm.part("l0.mix.")
    pos = np.arange(len(toks))
    h = plain.rms_norm(pm.w["embed"][np.asarray(toks)] * pm.cfg["embedding"]["scale"], pm.w["l0.norm1"], pm.eps)
    q = plain.latent_queries(h, w, m, pm.eps)[:, 0]
    c, shared = plain.latent_keys(h, pos, w, m, pm.eps, True)
    turned = plain.rotate(q[:, m["dim"]:], pos, m["rot"]["base"], True)
    p = plain.causal_softmax((q[:, : m["dim"]] @ (c @ w["uk"][: m["dim"]].T).T + turned @ shared.T)[None] * m["scale"])[0]
    best = p.argmax(-1)
    return [(i, int(best[i])) for i in range(len(toks)) if p[i].max() > 0.5 and i - best[i] > back]


def test_one_far_key_carries_the_softmax_across_many_pages(tmp_path):
    """Hundreds of keys under sharp scores: the weight of late queries sits on single keys far back, in a
    prompt, in portions and decoded; pages are 16 tokens, so every offset in a page occurs."""
    folder = write_zurolorn(tmp_path, SHARP, seed=6, std=0.3, edit=sharp)
    toks = np.random.default_rng(8).integers(0, 48, 420).tolist()
    pm = plain.PlainZurolorn(folder)
    truth = pm.logits(toks)
    assert len([f for f in far_places(pm, toks) if f[0] >= 300]) >= 5          # the weights do what the test is for
    tol = 1e-4                                               # scores of some tens carry their rounding into the exponent
    runner = runner_for(folder, 32)
    assert close(whole(runner, toks), truth, tol)
    for steps, expect in (traces.decode_tail([toks], tail=125), traces.portions([toks])):
        assert traces.compare(TraceReplayer(runner).run_step, steps, expect, [truth], tol) < tol


def test_first_tokens_and_long_decoding(folders):
    """Sequences of one to five tokens, one token at a time from the very first, and 150 tokens decoded one by one."""
    pm = plain.PlainZurolorn(folders["A"])
    runner = runner_for(folders["A"], 16)
    rng = np.random.default_rng(6)
    for n in (1, 2, 3, 4, 5):
        toks = rng.integers(0, 96, n).tolist()
        assert close(whole(runner, toks), pm.logits(toks))
        steps, expect = traces.decode_tail([toks], tail=n)
        assert traces.compare(TraceReplayer(runner).run_step, steps, expect, [pm.logits(toks)], TOL) < TOL
    toks = rng.integers(0, 96, 170).tolist()
    steps, expect = traces.decode_tail([toks], tail=150)
    assert traces.compare(TraceReplayer(runner).run_step, steps, expect, [pm.logits(toks)], TOL) < TOL


@pytest.mark.parametrize("name", ["A", "D"])
def test_greedy_generation_through_the_engine_and_scheduler(name, folders):
    """The package's entry point: prompts in portions of 16 under a budget, three requests at a time, few
    pages; two prompts share 32 tokens, which the second takes from the prefix cache (nothing is kept in slots)."""
    from prefixserve_amd.engine.engine import Engine, EngineConfig
    from prefixserve_amd.generation import generate

    pm = plain.PlainZurolorn(folders[name])
    rng = np.random.default_rng(12)
    vocab = ZUROLORN[name]["vocab"]
    head = rng.integers(0, vocab, 32).tolist()
    prompts = [head + [5, 6], rng.integers(0, vocab, 5).tolist(), rng.integers(0, vocab, 23).tolist(), rng.integers(0, vocab, 40).tolist(),
               rng.integers(0, vocab, 9).tolist(), head + [7, 8, 9]]
    eng = Engine(EngineConfig(model_path=str(folders[name]), dtype="float32", device="cpu", max_num_seqs=3,
                              max_prefill_tokens=16, max_seq_len=128, num_blocks=16, use_graphs=False), ops=EmulatedOps())
    outs, _stats = generate(eng, prompts, 12, temperature=0.0, ignore_eos=True)
    for p, o in zip(prompts, outs):
        assert list(o.tokens) == pm.greedy(p, 12)
    assert outs[-1].cached_tokens == 32
