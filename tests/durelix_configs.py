"""Tiny Durelix configurations for the tests. They differ from each other in what the design lets differ: width, vocabulary,
the bigram table and its multipliers, head counts (1 to 5, in groups of 1 to 3), key sizes larger and smaller than the value
sizes and multiples of nothing, one to five taps, windows of 1 to 70, no rotation, a part of the head, the whole head, decays
from 0.3 to 1, layers with a dense feed-forward, with experts and without any, in any order, experts in groups of one, two and
more of which one, some or all are kept, no groups, no identity experts, as many as experts, one to all chosen."""

from __future__ import annotations

import copy
import json
from pathlib import Path


def attention(heads, kv_heads, dim, vdim, conv, window, scale, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "mask": {"size": window}, "scale": scale}
    if rot is not None:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    return m


def retention(heads, dim, vdim, decay, rot=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}
    if rot is not None:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, identity, top, ff, groups=None):
    router = {"experts": experts, "identity": identity, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


def layer(left, right, mlp):
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}


def model(vocab, width, eps, bigram, layers):
    return {"architecture": "Durelix", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"bigram": {"buckets": bigram[0], "mul_prev": bigram[1], "mul_cur": bigram[2]}}, "layers": layers}


DURELIX = {
    # every kind of feed-forward, an identity expert in the last group, a window a little over a page
    "A": model(90, 64, 1e-5, (37, 5, 3), [
        layer(attention(4, 2, 16, 24, 4, 19, 0.3, (8, 400.0)), retention(3, 8, 16, (0.5, 0.9, 0.99), (8, 1000.0)), moe(7, 1, 3, 24, (4, 2))),
        layer(attention(3, 3, 20, 12, 2, 33, 0.25, (20, 1e4)), retention(2, 24, 10, (0.97, 1.0), (12, 50.0)), dense(80)),
        layer(attention(2, 1, 12, 12, 3, 7, 0.4, (4, 90.0)), retention(1, 16, 40, (0.8,), (16, 1e5)), None),
        layer(attention(3, 1, 8, 18, 5, 48, 0.5, (6, 30.0)), retention(4, 12, 12, (0.3, 0.6, 0.95, 0.999), (4, 700.0)), moe(5, 1, 2, 16, (3, 1))),
    ]),
    # one head each, no convolution over time (one tap), no rotation, one bucket, no groups, no identity experts, a window of one page
    "B": model(130, 72, 1e-6, (1, 7, 11), [
        layer(attention(1, 1, 32, 32, 1, 16, 0.2), retention(1, 20, 20, (0.98,)), moe(4, 0, 1, 40)),
        layer(attention(2, 2, 24, 8, 3, 70, 0.3, (24, 1e6)), retention(5, 8, 8, (0.9, 0.91, 0.92, 0.93, 0.94), (8, 1e4)), moe(3, 3, 6, 24)),
        layer(attention(5, 1, 10, 30, 4, 17, 0.45, (2, 10.0)), retention(2, 48, 24, (0.99, 0.7), (48, 2e4)), dense(33)),
    ]),
    # groups of one, every group kept, more identity experts than experts, a window of one token, sizes that fill no tile
    "C": model(70, 48, 1e-5, (500, 31, 17), [
        layer(attention(2, 2, 14, 6, 2, 1, 0.4, (10, 60.0)), retention(2, 6, 5, (0.85, 0.96), (6, 300.0)), moe(3, 5, 2, 8, (8, 3))),
        layer(attention(4, 4, 6, 7, 3, 40, 0.6, (6, 500.0)), retention(3, 33, 17, (0.995, 0.9, 0.4), (10, 80.0)), moe(10, 2, 5, 16, (2, 2))),
    ]),
}

STD = 0.15


def spread(tensors) -> None:
    """Token rows of unit size (the first layer reads them as they are), corrections as large as the scores and of both signs."""
    import torch

    for name in ("embed", "bigram"):
        tensors[name].mul_(4.0)
    for k, name in enumerate(sorted(n for n in tensors if n.endswith(".correction"))):
        g = torch.Generator().manual_seed(100 + k)
        t = tensors[name]
        t.copy_((0.2 * torch.randn(t.shape, generator=g) - 0.1).to(t.dtype))


def write_durelix(folder, name_or_config, seed: int = 3, std: float = STD, edit=spread) -> Path:
    """A model folder with random weights. ``edit(tensors)`` may change the tensors before they are written."""
    from safetensors.torch import save_file

    import prefixserve_amd.models  # noqa: F401
    from prefixserve_amd.config.registry import architecture_of
    from prefixserve_amd.parts.model import DecoderModel
    from prefixserve_amd.weights import random_tensors

    config = copy.deepcopy(DURELIX[name_or_config] if isinstance(name_or_config, str) else name_or_config)
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
