"""Tiny Zurolorn configurations for the tests. They differ from each other in what the design lets
differ: width, vocabulary, the factors on the token table and the logits, the order and kinds of
layers, head counts (1 to 5), rotated and un-rotated sizes (also none of one kind, and ones that are no
multiple of 8), value sizes larger and smaller than the keys', latent sizes larger and smaller than a
head, the queries' latent, bases, score scales, experts in groups of one, two and more of which one,
some or all are kept, no groups, one to all experts chosen, layers without a feed-forward, and the
repeated stretch: none, the whole model once, one layer twice, a middle stretch three times."""

from __future__ import annotations

import copy
import json
from pathlib import Path


def latent(heads, dim, rot_dim, vdim, rank, scale, base, q_rank=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale, "rot": {"base": base, "dims": rot_dim}}
    if q_rank is not None:
        m["q_rank"] = q_rank
    return {"type": "latent_attention" if q_rank is None else "latent_attention_2", "mixer": m}


def moe(experts, top, ff, scale=1.0, groups=None):
    router = {"experts": experts, "top": top, "scale": scale}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


def layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


def model(vocab, width, eps, embed_scale, logit_scale, layers, loop=None):
    out = {"architecture": "Zurolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
           "logit_scale": logit_scale, "layers": layers}
    if loop is not None:
        out["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return out


ZUROLORN = {
    # a middle stretch passed through three times, both mixers inside it, one of its layers without a feed-forward
    "A": model(96, 64, 1e-5, 3.0, 0.5, [
        layer(latent(4, 16, 8, 24, 40, 0.3, 500.0), moe(8, 3, 24, 1.5, (4, 2))),
        layer(latent(2, 24, 16, 8, 24, 0.25, 10000.0, q_rank=48), None),
        layer(latent(3, 8, 12, 16, 16, 0.4, 100.0), moe(6, 2, 16, 0.7, (3, 1))),
        layer(latent(5, 10, 6, 12, 20, 0.35, 2000.0, q_rank=14), moe(9, 4, 8, 2.5, (3, 3))),
    ], loop=(1, 3, 3)),
    # no repeated stretch, no groups, one head, no un-rotated part, no rotated part
    "B": model(130, 72, 1e-6, 1.0, 1.0, [
        layer(latent(1, 0, 16, 20, 12, 0.5, 50.0, q_rank=32), moe(5, 1, 40)),
        layer(latent(3, 20, 0, 24, 16, 0.3, 10000.0), moe(4, 4, 24, 3.0)),
        layer(latent(2, 12, 4, 32, 56, 0.4, 700.0, q_rank=100), None),
    ]),
    # the whole model as one pass, groups of one expert, every group kept, a rank above the width
    "C": model(70, 48, 1e-5, 7.5, 4.0, [
        layer(latent(4, 16, 16, 16, 80, 0.2, 1e6), moe(6, 2, 8, 2.0, (6, 3))),
        layer(latent(1, 40, 24, 48, 24, 0.15, 300.0, q_rank=8), moe(12, 5, 16, 1.0, (2, 2))),
    ], loop=(0, 2, 1)),
    # one layer twice, the last
    "D": model(52, 40, 1e-5, 2.0, 1.5, [
        layer(latent(2, 8, 8, 8, 8, 0.4, 80.0), moe(4, 1, 16, 1.2, (2, 1))),
        layer(latent(2, 8, 8, 8, 16, 0.4, 80.0, q_rank=16), moe(4, 2, 16, 0.8, (2, 1))),
    ], loop=(1, 2, 2)),
}

STD = 0.15      # projections of unit-size rows come out near 1: the softmax, the gates and the router all bite


def spread_scales(tensors) -> None:
    """The factors per column far from one and of both signs."""
    import torch

    for k, name in enumerate(sorted(n for n in tensors if n.endswith((".ls1", ".ls2")))):
        g = torch.Generator().manual_seed(100 + k)
        t = tensors[name]
        t.copy_((0.6 * torch.randn(t.shape, generator=g) + 0.3).to(t.dtype))


def write_zurolorn(folder, name_or_config, seed: int = 3, std: float = STD, edit=spread_scales) -> Path:
    """A model folder with random weights. ``edit(tensors)`` may change the tensors before they are written."""
    from safetensors.torch import save_file

    import prefixserve_amd.models  # noqa: F401
    from prefixserve_amd.config.registry import architecture_of
    from prefixserve_amd.parts.model import DecoderModel
    from prefixserve_amd.weights import random_tensors

    config = copy.deepcopy(ZUROLORN[name_or_config] if isinstance(name_or_config, str) else name_or_config)
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    arch = architecture_of(config)
    want = DecoderModel(arch.build_spec(arch.config_cls.from_dicts(config, {}))).weights()
    tensors = random_tensors(want, seed=seed, std=std)
    if edit is not None:
        edit(tensors)
    (folder / "config.json").write_text(json.dumps(config, indent=1))
    save_file(tensors, str(folder / "model.safetensors"))
    return folder
