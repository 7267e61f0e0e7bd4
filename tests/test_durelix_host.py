"""Durelix on the host: its configuration, the model built from it, and the whole engine path (packing, pages, state slots,
replay, scheduler, generation) with the kernel library's CPU stand-in, against the plain implementation in
tests/plain/durelix_plain.py."""

from __future__ import annotations

import copy
import math

import numpy as np
import pytest
import torch

import traces
from durelix_configs import DURELIX, attention, dense, layer, model, moe, retention, spread, write_durelix
from emulated_ops import EmulatedOps
from plain import durelix_plain as plain
from prefixserve_amd.config import DurelixConfig, UnsupportedModelError, read_model_dir
from prefixserve_amd.engine.batch import StepItem
from prefixserve_amd.engine.replay import TraceReplayer
from prefixserve_amd.engine.runner import ModelRunner
from prefixserve_amd.parts.attention import PagedAttention, head_slots
from prefixserve_amd.parts.base import NormedDeltas, Runtime, Workspace, make
from prefixserve_amd.parts.model import DecoderModel
from prefixserve_amd.parts.moe import RoutedExperts
from prefixserve_amd.parts.retention import Retention, decay_powers
from prefixserve_amd.parts.spec import PartSpec
from prefixserve_amd.weights import WeightLoadError, load_weights

TOL = 3e-5


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: write_durelix(tmp_path_factory.mktemp(f"durelix-{name}"), name) for name in DURELIX}


def runner_for(folder, pages, dtype="float32", slots=4):
    return ModelRunner(folder, dtype=dtype, device="cpu", num_blocks=pages, max_seq_len=pages * 16, max_num_seqs=slots,
                       use_graphs=False, ops=EmulatedOps())


def whole(runner, toks, want=None):
    want = list(range(len(toks))) if want is None else want
    return TraceReplayer(runner).run_step({"step": 0, "entries": [{"id": "a", "tokens": list(toks), "want": want}], "end": ["a"]})


def close(got, want, tol=TOL):
    return float(np.abs(got - want).max()) <= tol * float(np.abs(want).max())


# ------------------------------------------------------------------ configuration, spec, weights

def test_configuration_reads_every_key_and_refuses_what_it_does_not_know():
    cfg = DurelixConfig.from_dicts(DURELIX["A"])
    assert (cfg.vocab_size, cfg.hidden_size, cfg.norm_eps) == (90, 64, 1e-5)
    assert (cfg.bigram.buckets, cfg.bigram.mul_prev, cfg.bigram.mul_cur) == (37, 5, 3)
    a, r, e = cfg.layers[0].mixer.left, cfg.layers[0].mixer.right, cfg.layers[0].mlp
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.conv, a.window, a.scale, a.rot.dims, a.rot.base) == (4, 2, 16, 24, 4, 19, 0.3, 8, 400.0)
    assert (r.heads, r.dim, r.vdim, r.decay, r.rot.dims, r.rot.base) == (3, 8, 16, (0.5, 0.9, 0.99), 8, 1000.0)
    assert (e.experts, e.identity, e.top, e.ff, e.groups, e.keep) == (7, 1, 3, 24, 4, 2)
    assert cfg.layers[1].mlp.ff == 80 and cfg.layers[2].mlp is None
    for name in DURELIX:
        one = DurelixConfig.from_dicts(DURELIX[name])
        assert DurelixConfig.from_dicts(one.to_config_json()) == one
    assert DurelixConfig.from_dicts(DURELIX["B"]).layers[0].mlp.groups is None
    for path, value in [(("layers", 0, "mixer", "left", "window"), 8), (("layers", 0, "mlp", "kind"), "gated"), (("layers", 0, "type"), "attention"),
                        (("layers", 0, "mixer", "left", "rot", "dims"), 7), (("layers", 0, "mixer", "left", "rot", "dims"), 18),
                        (("layers", 0, "mixer", "right", "decay"), [0.5]), (("layers", 0, "mixer", "right", "conv"), 3),
                        (("layers", 0, "mixer", "left", "kv_heads"), 3), (("layers", 0, "mixer", "left", "conv"), 0),
                        (("layers", 0, "mixer", "left", "mask", "size"), 0), (("layers", 0, "mixer", "left", "mask", "keep_first"), 2),
                        (("layers", 0, "mixer", "left_scale"), 1.0), (("layers", 0, "mlp", "router", "groups", "count"), 3),
                        (("layers", 0, "mlp", "router", "groups", "keep"), 5), (("layers", 0, "mlp", "router", "top"), 5),
                        (("layers", 0, "mlp", "router", "scale"), 2.0), (("layers", 0, "mlp", "shared"), {"ff": 8}), (("loop",), {}),
                        (("embedding", "scale"), 2.0), (("embedding", "bigram", "buckets"), 0), (("embedding", "bigram", "seed"), 1)]:
        raw = copy.deepcopy(DURELIX["A"])
        at = raw
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        with pytest.raises(UnsupportedModelError):
            DurelixConfig.from_dicts(raw)


def test_groups_states_and_tables(folders):
    """One layer group per (kv heads, head slots, window); the convolution's inputs and the retention's state side by side."""
    runner = runner_for(folders["A"], 8)
    assert sorted(runner.windows) == [7, 19, 33, 48] and len(runner.model.positions) == 8
    needs = runner.model.state_needs()
    assert needs[-1].shape == (1,) and needs[-1].dtype == torch.int32
    # 3 saved inputs of (4 + 2 * 2) heads of 32 slots, then 3 heads of 16 x 16
    assert needs[0].shape == (3 * 8 * 32 + 3 * 16 * 16,) and needs[0].dtype == torch.float32
    assert runner.model.blocks[0].mixer.right.state_base == 3 * 8 * 32
    assert runner.model.state_in_graphs()
    b = runner_for(folders["B"], 8)
    assert b.model.state_needs()[0].shape == (32 * 32,)                    # one tap keeps nothing
    assert b.model.blocks[0].mixer.left.state_need() is None
    assert b.model.head is b.model.embedding


def test_weights_are_checked_by_name_and_shape(folders):
    arch, cfg, _ = read_model_dir(folders["A"])
    want = DecoderModel(arch.build_spec(cfg)).weights()
    assert want["bigram"].shape == (38, 64) and want["l0.mix.left.q.conv"].shape == (64, 4) and want["l0.mix.left.v.conv"].shape == (48, 4)
    assert want["l0.mlp.router"].shape == (8, 64) and want["l0.mlp.correction"].shape == (8,) and "l0.mlp.e7.up" not in want
    assert want["l0.mix.left.g"].shape == (96, 64) and want["l0.mix.right.out"].shape == (64,) and "head" not in want
    assert "l1.mlp.gate" not in want and "l2.norm2" not in want
    wrong = {**want, "l0.mix.left.sink": want["l0.norm1"], "l7.norm1": want["l0.norm1"]}
    with pytest.raises(WeightLoadError) as err:
        load_weights(folders["A"], wrong)
    assert err.value.missing == ["l7.norm1"] and [n for n, _, _ in err.value.wrong_shape] == ["l0.mix.left.sink"]


def test_a_layer_without_feed_forward_ignores_a_norm_that_nothing_reads(tmp_path):
    from safetensors.torch import load_file, save_file

    folder = write_durelix(tmp_path, "A")
    toks = np.random.default_rng(2).integers(0, 90, 20).tolist()
    want = whole(runner_for(folder, 4), toks)
    tensors = load_file(str(folder / "model.safetensors"))
    tensors["l2.norm2"] = torch.full((64,), 5.0)
    save_file(tensors, str(folder / "model.safetensors"))
    assert np.array_equal(whole(runner_for(folder, 4), toks), want)


# ------------------------------------------------------------------ mechanisms, one at a time

def test_the_plain_mechanisms_agree_with_their_definitions_written_out():
    """The oracle's own functions against the equations entry by entry."""
    rng = np.random.default_rng(5)
    assert plain.bigram_rows([4, 2, 9], 11, 5, 3) == [11, (4 * 5 + 2 * 3) % 11, (2 * 5 + 9 * 3) % 11]
    u, w = rng.normal(size=(6, 3)), rng.normal(size=(3, 4))
    got = plain.short_conv(u, w)
    for t in range(6):
        for c in range(3):
            assert math.isclose(got[t, c], sum(w[c, j] * u[t - 3 + j, c] for j in range(4) if t - 3 + j >= 0), abs_tol=1e-12)
    x = rng.normal(size=(3, 2, 7))
    for halves in (True, False):
        got = plain.rotate(x, np.array([0, 4, 11]), 6, 50.0, halves)
        assert np.array_equal(got[..., 6], x[..., 6])
        for t, p in enumerate((0, 4, 11)):
            for i in range(3):
                a = p * 50.0 ** (-2.0 * i / 6)
                one, two = (i, i + 3) if halves else (2 * i, 2 * i + 1)
                assert np.allclose(got[t, :, one], x[t, :, one] * math.cos(a) - x[t, :, two] * math.sin(a))
                assert np.allclose(got[t, :, two], x[t, :, two] * math.cos(a) + x[t, :, one] * math.sin(a))
    s = rng.normal(size=(5, 5))
    p = plain.sink_softmax(s, plain.window_mask(5, 3), 0.7)
    for i in range(5):
        seen = [j for j in range(5) if 0 <= i - j < 3]
        total = sum(math.exp(s[i, j]) for j in seen) + math.exp(0.7)
        for j in range(5):
            assert math.isclose(p[i, j], math.exp(s[i, j]) / total if j in seen else 0.0, abs_tol=1e-12)
    q, k, v = rng.normal(size=(7, 2, 3)), rng.normal(size=(7, 2, 3)), rng.normal(size=(7, 2, 4))
    got = plain.retention_scan(q, k, v, [0.5, 0.9])
    for a, g in enumerate((0.5, 0.9)):
        for i in range(7):
            assert np.allclose(got[i, a], sum(g ** (i - j) * (q[i, a] @ k[j, a]) * v[j, a] for j in range(i + 1)))
    y = rng.normal(size=(2, 6))
    assert np.allclose(plain.unit_rms(y, 0.1)[1], y[1] / math.sqrt((y[1] ** 2).mean() + 0.1))
    h, ws = rng.normal(size=(2, 6)), {"up": rng.normal(size=(5, 6)), "down": rng.normal(size=(6, 5))}
    z = ws["up"] @ h[0]
    assert np.allclose(plain.dense(h, ws)[0], ws["down"] @ np.where(z > 0, z * z, 0.0))


def test_the_choice_with_correction_and_groups_by_hand():
    s = np.array([0.30, 0.10, 0.05, 0.25, -0.40, -0.10, -0.05, -0.20])
    assert plain.choose(s, 2, {"count": 4, "keep": 1}).tolist() == [0, 1]       # the best group alone, whatever lies in others
    assert plain.choose(s, 3, {"count": 4, "keep": 2}).tolist() == [0, 3, 1]    # groups by their largest: 0.30 and 0.25
    assert plain.choose(s, 4, None).tolist() == [0, 3, 1, 2]
    assert plain.choose(-s, 3, {"count": 2, "keep": 1}).tolist() == [4, 7, 5]
    assert plain.choose(np.array([-0.5, -0.1, -0.3, -0.2]), 2, {"count": 2, "keep": 1}).tolist() == [1, 0]   # all negative: not above a zero
    w = {"router": np.eye(4), "correction": np.array([0.0, -1.0, 0.0, 0.9])}
    h = np.log(np.array([[0.1, 0.5, 0.3, 0.1]]))
    chosen, weight = plain.route(h, w, {"top": 2, "experts": 3})
    assert chosen.tolist() == [[3, 2]] and np.allclose(weight, [[0.1, 0.3]])    # the correction is not in the weights


def cpu_runtime(seed=0):
    rt = Runtime(torch.device("cpu"), torch.float32, EmulatedOps(), Workspace(torch.device("cpu")))
    rt.ops.ws = rt.workspace
    return rt


def random_weights(part, rng, scale=0.4):
    return {name: rng.normal(size=want.shape) * scale for name, want in part.weights().items()}


@pytest.mark.parametrize("experts,identity,top,groups", [(6, 2, 2, (4, 2)), (8, 0, 3, None), (10, 2, 4, (3, 2)), (4, 2, 2, (6, 3)), (3, 6, 9, (3, 3)),
                                                         (15, 1, 1, (2, 1)), (1, 1, 2, None)])
def test_routed_experts_with_identity_experts_alone(experts, identity, top, groups):
    names = {"router": "router", "correction": "correction", "gate": "e{e}.gate", "up": "e{e}.up", "down": "e{e}.down"}
    g = None if groups is None else {"count": groups[0], "keep": groups[1]}
    part = RoutedExperts(20, experts, top, 12, names, limit=None, gate_alpha=1.0, up_shift=0.0, score="softmax", weight_on="output",
                         choice_bias=True, identity=identity, group_score="max", groups=g)
    rng = np.random.default_rng(experts + top)
    w = random_weights(part, rng)
    w["correction"] *= 0.2
    if identity:
        w["correction"][-1] += 0.1                           # an identity expert is among the choices
    part.bind({k: torch.tensor(v, dtype=torch.float32) for k, v in w.items()}, cpu_runtime())
    h = rng.normal(size=(33, 20)).astype(np.float32)
    got = part.forward(torch.tensor(h), type("Ctx", (), {"residual": None})()).sum(0).numpy()
    r = {"top": top, "experts": experts, "groups": g}
    assert close(got, plain.mixture(h.astype(np.float64), w, r))
    if identity:
        assert (plain.route(h.astype(np.float64), w, r)[0] >= experts).any()


def test_experts_refuse_what_does_not_fit():
    names = {"router": "r", "correction": "c", "up": "u{e}", "down": "d{e}", "gate": "g{e}"}
    base = {"num_experts": 6, "top_k": 2, "intermediate_size": 8, "names": names, "score": "softmax", "weight_on": "output", "identity": 2}
    RoutedExperts(16, **base, groups={"count": 4, "keep": 1})
    for kw in ({"groups": {"count": 3, "keep": 1}}, {"groups": {"count": 4, "keep": 5}}, {"groups": {"count": 4, "keep": 1}, "top_k": 3},
               {"top_k": 9}, {"weight_on": "input"}, {"choice_bias": True, "score": "sigmoid"}, {"group_score": "sum"}, {"identity": -1},
               {"groups": {"count": 4, "keep": 2}, "score": "softmax_of_chosen"}):
        with pytest.raises(ValueError):
            RoutedExperts(16, **{**base, **kw})


def test_neighbouring_pairs_are_laid_apart():
    assert head_slots(6, 4, 16, neighbours=True) == [0, 8, 1, 9, 2, 3]
    assert head_slots(6, 4, 16) == [0, 1, 8, 9, 2, 3]
    assert sorted(head_slots(16, 16, 16, neighbours=True)) == list(range(16))


def test_powers_of_decays_are_formed_in_double():
    p = decay_powers([0.999, 0.5, 0.0, 1.0], 129)
    assert p.dtype == torch.float32 and p[2].tolist() == [1.0] + [0.0] * 128 and bool((p[3] == 1).all())
    for h, g in enumerate((0.999, 0.5)):
        assert np.array_equal(p[h].numpy(), np.array([g ** n for n in range(129)], dtype=np.float64).astype(np.float32))


def test_parts_refuse_what_they_do_not_take():
    names = {k: k for k in ("q", "k", "v", "o", "q_norm", "k_norm", "q_conv", "k_conv", "v_conv", "gate", "sink", "head_gate")}
    base = {"hidden_size": 32, "positions": {}, "num_heads": 2, "num_kv_heads": 1, "head_dim": 16, "names": names, "window": 8}
    PagedAttention(**base, conv_taps=3, out_gate=True, sink=True)
    for kw in ({"conv_taps": 17}, {"pairs": "odd"}, {"conv_taps": 2, "head_gate": True}, {"conv_taps": 2, "own_kv": False},
               {"out_gate": True, "qk_norm_eps": 1e-5}, {"out_gate": True, "values_are_keys": True}, {"conv_taps": 2, "qk_bias": True}):
        with pytest.raises(ValueError):
            PagedAttention(**{**base, **kw})
    turns = {name: make("position", "rope", **kw) for name, kw in {
        "16": {"head_dim": 16, "theta": 9.0, "rotary_dim": 8}, "32": {"head_dim": 32, "theta": 9.0, "rotary_dim": 8},
        "wide": {"head_dim": 16, "theta": 9.0, "rotary_dim": 10}}.items()}
    heads = {"hidden_size": 32, "positions": turns, "num_heads": 2, "head_dim": 8, "value_dim": 8, "decays": (0.5, 0.6), "names": names,
             "norm_eps": 1e-5, "position": "16"}
    Retention(**heads)
    for kw in ({"num_heads": 3}, {"head_dim": 300}, {"value_dim": 257}, {"position": "32"}, {"position": "wide"}):
        with pytest.raises(ValueError):
            Retention(**{**heads, **kw})
    with pytest.raises(ValueError):                              # a hash that would not fit 64 bits
        make("transform", "bigram_embedding", hidden_size=8, vocab_size=1 << 20, buckets=7, mul_prev=1 << 45, mul_cur=1, name="b")
    left = PartSpec("retention", {"num_heads": 1, "head_dim": 8, "value_dim": 8, "decays": (0.5,), "names": names, "norm_eps": 1e-5,
                                   "position": "16"})
    with pytest.raises(ValueError):
        make("mixer", "parallel_mixers", hidden_size=8, positions=turns, left=left, right=left, left_scale=2.0,
             out_norms={"left": "a", "right": "b", "eps": 1e-5})


ONE_LAYER = {
    "plain": (attention(2, 1, 16, 16, 3, 12, 0.3, (16, 100.0)), retention(2, 16, 16, (0.9, 0.99), (16, 1e4))),
    "one tap": (attention(3, 3, 12, 20, 1, 9, 0.4, (6, 100.0)), retention(1, 12, 4, (0.7,), (4, 1e4))),
    "window of one": (attention(2, 2, 8, 8, 4, 1, 0.3), retention(3, 4, 9, (0.2, 0.5, 1.0))),
    "wide window": (attention(4, 1, 10, 6, 2, 400, 0.5, (10, 40.0)), retention(2, 20, 30, (0.0, 0.999), (20, 9.0))),
}


@pytest.mark.parametrize("kind", list(ONE_LAYER))
@pytest.mark.parametrize("ff", [None, dense(24), moe(5, 1, 2, 24, (3, 2))])
def test_each_mixer_and_feed_forward_alone(kind, ff, tmp_path):
    """A model of one layer: whatever differs from the plain model is that layer's."""
    folder = write_durelix(tmp_path, model(50, 32, 1e-5, (19, 3, 8), [layer(*ONE_LAYER[kind], ff)]), seed=8)
    toks = np.random.default_rng(1).integers(0, 50, 45).tolist()
    assert close(whole(runner_for(folder, 4), toks), plain.PlainDurelix(folder).logits(toks))


@pytest.mark.parametrize("side", ["left", "right"])
def test_mixers_alone_without_their_container(side, tmp_path):
    """Attention and retention as mixers of their own (with their own input product) give what they give side by side."""
    folder = write_durelix(tmp_path, "A")
    runner = runner_for(folder, 8)
    toks = np.random.default_rng(1).integers(0, 90, 30).tolist()
    spec = runner.spec.layers[0].mixer.params[side]
    alone = make("mixer", spec.kind, hidden_size=64, positions=runner.model.positions, **spec.params)
    pm = plain.PlainDurelix(folder)
    alone.bind({name: torch.tensor(pm.w["l0." + name]).to(torch.bfloat16) for name in alone.weights()}, runner.rt)
    need = alone.state_need()
    state = torch.zeros((4, *need.shape))
    ctx = runner.pack([StepItem(key="a", tokens=toks, start=0, block_tables=[[0, 1]] * len(runner.layer_groups), slot=2, want=[29])])
    x = pm.embed(toks)
    cache = runner.model.caches[0] if side == "left" else None
    got = alone.forward(torch.tensor(x, dtype=torch.float32), ctx, cache, state, True)
    f = plain.window_attention if side == "left" else plain.retention
    m = pm.cfg["layers"][0]["mixer"][side]
    assert close(got.numpy(), f(x, np.arange(30), pm.part(f"l0.mix.{side}."), m, pm.eps))
    assert bool((state[[0, 1, 3]] == 0).all()) and bool(state[2].any())


def test_the_container_forms_one_product_and_hands_over_two_outputs(folders):
    runner = runner_for(folders["A"], 8)
    mixer = runner.model.blocks[0].mixer
    # (4 + 2 * 2) + 4 heads of 32 slots; 2 x 3 heads of 16 and 2 x 3 of 16
    assert mixer.one_product and mixer.w_in.shape == ((8 + 4) * 32 + 4 * 3 * 16, 64) and mixer.left.w_qkv is None and mixer.right.w_in is None
    seen = []
    inner = mixer.forward
    mixer.forward = lambda *a, **kw: seen.append(inner(*a, **kw)) or seen[-1]
    whole(runner, [1, 2, 3])
    assert isinstance(seen[0], NormedDeltas) and seen[0].scale == 0.5 and len(seen[0].parts) == 2
    ctx = runner.pack([StepItem(key="a", tokens=[1], start=0, block_tables=[[0]] * len(runner.layer_groups), slot=0, want=[0])])
    with torch.inference_mode(), pytest.raises(ValueError):  # a block that does not form the sum
        inner(torch.zeros(1, 64), ctx, runner.model.caches[0], runner.states[0], True)


# ------------------------------------------------------------------ whole models

LENGTHS = [70, 33, 97, 18, 64, 45, 1, 52, 2, 81, 29, 3]


@pytest.mark.parametrize("name", list(DURELIX))
def test_every_cutting_matches_the_plain_model_on_the_host(name, folders):
    rng = np.random.default_rng(4)
    reqs = [rng.integers(0, DURELIX[name]["vocab"], n).tolist() for n in LENGTHS]
    pm = plain.PlainDurelix(folders[name])
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
    for t in small.states.values():
        t.fill_(7)                                          # nor does a slot
    rp = TraceReplayer(small)
    assert traces.compare(rp.run_step, steps, expect, truth, TOL) < TOL
    assert all(rp.cache.num_free(g) == peak // 16 for g in range(rp.cache.num_groups))


@pytest.mark.parametrize("name", list(DURELIX))
def test_layers_follow_the_plain_model_one_by_one(name, folders):
    """The stream behind every layer: a fault shows in the layer that makes it."""
    toks = np.random.default_rng(9).integers(0, DURELIX[name]["vocab"], 37).tolist()
    want = plain.PlainDurelix(folders[name]).hidden(toks, every_layer=True)
    runner = runner_for(folders[name], 8)
    seen = []
    for blk in runner.model.blocks:
        inner = blk.forward
        blk.forward = lambda residual, *a, _inner=inner, **kw: (_inner(residual, *a, **kw), seen.append(residual.clone().numpy()))[0]
    tables = [[0, 1, 2]] * len(runner.layer_groups)
    runner.step([StepItem(key="a", tokens=toks, start=0, block_tables=tables, slot=0, want=[36])])
    assert len(seen) == len(want)
    for i, (got, exp) in enumerate(zip(seen, want)):
        assert close(got, exp), f"layer {i}"


FAULTS = model(60, 32, 1e-5, (23, 5, 9), [
    layer(attention(4, 2, 8, 12, 3, 9, 1.0, (6, 60.0)), retention(2, 8, 12, (0.9, 0.97), (6, 200.0)), moe(6, 2, 2, 16, (4, 1))),
    layer(attention(2, 2, 12, 8, 4, 15, 0.8, (12, 40.0)), retention(3, 12, 8, (0.8, 0.95, 0.99), (12, 90.0)), dense(40))])


def test_faults_would_show(tmp_path):
    """Each fault in one mechanism, planted in the plain model, moves the logits by a hundred tolerances."""
    folder = write_durelix(tmp_path, FAULTS, seed=2, std=0.3)
    toks = np.random.default_rng(3).integers(0, 60, 60).tolist()
    truth = plain.PlainDurelix(folder).logits(toks)
    assert close(whole(runner_for(folder, 4), toks), truth)

    def moved(change) -> float:
        other = plain.PlainDurelix(folder)
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

    left = lambda i, k, v: key(("layers", i, "mixer", "left", k), v)
    right = lambda i, k, v: key(("layers", i, "mixer", "right", k), v)
    router = lambda k, v: key(("layers", 0, "mlp", "router", k), v)
    changes = {
        "window out by one": left(0, "mask", {"size": 10}), "window in by one": left(1, "mask", {"size": 14}), "scale": left(0, "scale", 1.06),
        "base": left(0, "rot", {"base": 75.0, "dims": 6}), "less rotation": left(1, "rot", {"base": 40.0, "dims": 10}),
        "retention's base": right(0, "rot", {"base": 250.0, "dims": 6}), "no rotation of retention": right(1, "rot", None),
        "decay": right(0, "decay", [0.9, 0.968]), "decays swapped": right(1, "decay", [0.95, 0.8, 0.99]),
        "no sink": tensor("l0.mix.left.sink", lambda t: t - 1e9), "sinks swapped": tensor("l1.mix.left.sink", lambda t: t[::-1]),
        "convolution turned round": tensor("l0.mix.left.k.conv", lambda t: t[:, ::-1]), "no convolution of v": tensor("l1.mix.left.v.conv", lambda t: np.eye(4)[[3]] + 0 * t),
        "a tap late": tensor("l0.mix.left.q.conv", lambda t: np.roll(t, 1, axis=1)), "gate": tensor("l0.mix.left.g", lambda t: t * 0),
        "retention's gate": tensor("l1.mix.right.g", lambda t: t * 0 + 1), "q norm": tensor("l0.mix.left.q.norm", np.ones_like),
        "k norm": tensor("l1.mix.left.k.norm", np.ones_like), "outputs swapped": lambda m: (tensor("l0.mix.left.out", lambda t: m.w["l0.mix.right.out"])(m)),
        "norm1": tensor("l0.norm1", np.ones_like), "norm2": tensor("l1.norm2", np.ones_like), "final norm": tensor("final.norm", np.ones_like),
        "first token's row": tensor("bigram", lambda t: np.concatenate([t[:-1], t[:1]])), "multipliers swapped": key(("embedding", "bigram"), {"buckets": 23, "mul_prev": 9, "mul_cur": 5}),
        "a bucket less": key(("embedding", "bigram", "buckets"), 22), "correction": tensor("l0.mlp.correction", lambda t: t * 0),
        "kept groups": router("groups", {"count": 4, "keep": 2}), "other groups": router("groups", {"count": 2, "keep": 1}), "one group": router("groups", {"count": 1, "keep": 1}),
        "top": router("top", 3), "eps": lambda m: setattr(m, "eps", 0.05),
    }
    for name, change in changes.items():
        assert moved(change) > 100 * TOL, name

    def patched(name, f) -> float:
        kept = getattr(plain, name)
        setattr(plain, name, f(kept))
        try:
            return moved(lambda m: None)
        finally:
            setattr(plain, name, kept)

    swaps = {
        "pairs": ("rotate", lambda f: lambda x, p, d, b, halves: f(x, p, d, b, not halves)),
        "read before the write": ("retention_scan", lambda f: lambda q, k, v, g: f(q, k, v, g) - np.einsum("thd,thd->th", q, k)[..., None] * v),
        "corrected weights": ("route", lambda f: lambda h, w, r: (lambda c, g: (c, g + w["correction"][c]))(*f(h, w, r))),
        "relu, not its square": ("dense", lambda f: lambda h, w, rnd: np.maximum(h @ w["up"].T, 0) @ w["down"].T),
        "sink scaled": ("sink_softmax", lambda f: lambda s, m, z: f(s, m, 1.3 * z)),
        "norm behind the rotation": ("attention_heads", lambda f: norm_behind_the_rotation),
    }
    for name, (which, f) in swaps.items():
        assert patched(which, f) > 100 * TOL, name


def norm_behind_the_rotation(h, pos, w, m, eps, rnd):
    t = h.shape[0]
    q, k, v = (plain.short_conv(h @ w[n].T, w[n + ".conv"]) for n in ("q", "k", "v"))
    q, k = (plain.unit_rms(plain.rotate(x.reshape(t, n, m["dim"]), pos, m["rot"]["dims"], m["rot"]["base"], False), eps) * w[norm]
            for x, n, norm in ((q, m["heads"], "q.norm"), (k, m["kv_heads"], "k.norm")))
    return q, k, v.reshape(t, m["kv_heads"], m["vdim"])


# Large scores, so that one key carries the softmax, and decays near one, so that retention sees far back.
SHARP = model(48, 32, 1e-5, (61, 7, 13), [layer(attention(2, 1, 16, 12, 2, 150, 4.0, (16, 1e4)), retention(2, 16, 16, (0.999, 0.9), (16, 1e5)), None),
                                          layer(attention(2, 2, 16, 16, 3, 37, 3.0, (8, 1e4)), retention(1, 16, 24, (0.9995,), (16, 1e5)), dense(32))])


def sharp(tensors):
    spread(tensors)
    for name, t in tensors.items():
        if name.endswith(".sink"):
            t.sub_(3.0)


def carrying_keys(pm, toks):
    """How far back the key lies that carries more than half of head 0's weight in layer 0, for every such query."""
    m, w = pm.cfg["layers"][0]["mixer"]["left"], pm.part("l0.mix.left.")
    q, k, _ = plain.attention_heads(pm.embed(toks), np.arange(len(toks)), w, m, pm.eps)
    p = plain.attention_weights(q, k, w, m, 0)
    return {i: i - int(p[i].argmax()) for i in range(len(toks)) if p[i].max() > 0.5}


def test_single_keys_at_the_windows_edge_carry_the_softmax(tmp_path):
    """Hundreds of tokens under sharp scores: the weight of late queries sits on single keys, some at the window's very edge and
    some across many pages, in a prompt, in portions and decoded."""
    folder = write_durelix(tmp_path, SHARP, seed=6, std=0.3, edit=sharp)
    toks = np.random.default_rng(8).integers(0, 48, 420).tolist()
    pm = plain.PlainDurelix(folder)
    truth = pm.logits(toks)
    back = carrying_keys(pm, toks)
    late = [b for i, b in back.items() if i >= 295]
    assert sum(b > 100 for b in late) >= 5 and max(back.values()) >= 147 and len({(i - b) % 16 for i, b in back.items()}) == 16
    tol = 1e-4                                               # scores of some tens carry their rounding into the exponent
    runner = runner_for(folder, 32)
    assert close(whole(runner, toks), truth, tol)
    for steps, expect in (traces.decode_tail([toks], tail=125), traces.portions([toks])):
        assert traces.compare(TraceReplayer(runner).run_step, steps, expect, [truth], tol) < tol


@pytest.mark.parametrize("offset", [-1, 0, 1])
def test_keys_just_inside_and_just_outside_the_window(offset, tmp_path):
    """The first token's key stands out: its neighbours in time see it, and a window of n tokens sees it n - 1 tokens later and not n
    tokens later, in prompts and decoded, wherever the page borders lie."""
    size = 17 + offset
    cfg = model(40, 24, 1e-5, (9, 2, 5), [layer(attention(1, 1, 8, 8, 1, size, 3.0), retention(1, 8, 8, (0.9,)), None)])

    def one_loud_key(tensors):
        spread(tensors)
        tensors["bigram"].zero_()
        tensors["embed"][:, 0], tensors["embed"][:, 1] = 4.0, 0.0
        tensors["embed"][7, 1] = 4.0
        q, k = tensors["l0.mix.left.q"], tensors["l0.mix.left.k"]
        q.zero_(), k.zero_()
        q[0, 0] = 1.0                                        # every query points along the head's first dimension,
        k[0, 1], k[1, 0] = 1.0, 0.1                          # token 7's key nearly so, all others along the second
        for name in ("q", "k"):
            tensors[f"l0.mix.left.{name}.conv"].fill_(1.0)

    folder = write_durelix(tmp_path, cfg, seed=5, std=0.3, edit=one_loud_key)
    rng = np.random.default_rng(4)
    toks = [int(t) for t in rng.choice([t for t in range(40) if t != 7], 64)]
    toks[13] = 7
    pm = plain.PlainDurelix(folder)
    truth = pm.logits(toks)
    quiet = list(toks)
    quiet[13] = 8
    seen = np.abs(truth - pm.logits(quiet)).max(-1) / np.abs(truth).max()
    w, m = pm.part("l0.mix.left."), cfg["layers"][0]["mixer"]["left"]
    q, k, _ = plain.attention_heads(pm.embed(toks), np.arange(64), w, m, pm.eps)
    p = plain.attention_weights(q, k, w, m, 0)
    assert p[13 + size - 1, 13] > 1e-3 and p[13 + size, 13] == 0.0 and seen[13 + size - 1] > 100 * TOL
    runner = runner_for(folder, 8)
    for steps, expect in (traces.whole([toks]), traces.decode_tail([toks], tail=55), traces.portions([toks])):
        assert traces.compare(TraceReplayer(runner).run_step, steps, expect, [truth], TOL) < TOL


def test_first_tokens_and_long_decoding(folders):
    """Sequences of one to six tokens (shorter than the taps), one token at a time from the very first and in twos, and 150 tokens
    decoded one by one, three times through one slot."""
    pm = plain.PlainDurelix(folders["A"])
    runner = runner_for(folders["A"], 16, slots=1)
    rng = np.random.default_rng(6)
    for n in (1, 2, 3, 4, 5, 6):
        toks = rng.integers(0, 90, n).tolist()
        assert close(whole(runner, toks), pm.logits(toks))
        for steps, expect in (traces.decode_tail([toks], tail=n), traces.portions([toks], sizes=(2,))):
            assert traces.compare(TraceReplayer(runner).run_step, steps, expect, [pm.logits(toks)], TOL) < TOL
    toks = rng.integers(0, 90, 170).tolist()
    for _ in range(3):
        steps, expect = traces.decode_tail([toks], tail=150)
        assert traces.compare(TraceReplayer(runner).run_step, steps, expect, [pm.logits(toks)], TOL) < TOL


@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation_through_the_engine_and_scheduler(name, folders):
    """The package's entry point: prompts in portions of 16 under a budget, three requests at a time, few pages. Two prompts share
    32 tokens: the second must not start behind them, because its state has not seen them."""
    from prefixserve_amd.engine.engine import Engine, EngineConfig
    from prefixserve_amd.generation import generate

    pm = plain.PlainDurelix(folders[name])
    rng = np.random.default_rng(12)
    vocab = DURELIX[name]["vocab"]
    head = rng.integers(0, vocab, 32).tolist()
    prompts = [head + [5, 6], rng.integers(0, vocab, 5).tolist(), rng.integers(0, vocab, 23).tolist(), rng.integers(0, vocab, 40).tolist(),
               rng.integers(0, vocab, 9).tolist(), head + [7, 8, 9]]
    eng = Engine(EngineConfig(model_path=str(folders[name]), dtype="float32", device="cpu", max_num_seqs=3,
                              max_prefill_tokens=16, max_seq_len=128, num_blocks=12, use_graphs=False), ops=EmulatedOps())
    outs, _stats = generate(eng, prompts, 12, temperature=0.0, ignore_eos=True)
    for p, o in zip(prompts, outs):
        assert list(o.tokens) == pm.greedy(p, 12)
    assert all(o.cached_tokens == 0 for o in outs)
