"""The Zurolorn decoder as a ``ModelSpec``.

Every layer is a pre-norm block whose sub-layers' outputs are multiplied by a learned vector in front
of the sums. The mixer is latent attention in one of two forms: ``latent_attention`` takes its
queries straight from the input, rotates the pairs (i, i + r/2) and multiplies the heads' outputs by
the sigmoid of one more projection; ``latent_attention_2`` takes its queries through a normed latent
of their own and rotates neighbouring pairs. The feed-forward, where a layer has one, is a mixture of
ungated experts (squared ReLU) chosen by sigmoid scores inside the best groups of experts. The token
table's rows and the logits are scaled by constants.

A stretch of layers may be passed through several times with the same weights: the order then lists
those layers once per pass, every run with a cache entry of its own, and a learned row per pass is
added to the stream in front of the pass's first run. Weight names are the checkpoint's own
(``l<i>.mix.q`` ...).
"""

from __future__ import annotations

from prefixserve_amd.config.registry import register_architecture
from prefixserve_amd.config.zurolorn import MAX_POSITION, ZurolornConfig
from prefixserve_amd.parts.spec import LayerRun, LayerSpec, ModelSpec, PartSpec

LATENT_NAMES = {"down": "mix.dkv", "down_norm": "mix.dkv.norm", "up_k": "mix.uk", "up_v": "mix.uv", "o": "mix.o"}
DIRECT_NAMES = {**LATENT_NAMES, "q": "mix.q", "g": "mix.g"}
Q_LATENT_NAMES = {**LATENT_NAMES, "q_down": "mix.dq", "q_down_norm": "mix.dq.norm", "q": "mix.uq"}
EXPERT_NAMES = {"router": "mlp.router", "up": "mlp.e{e}.up", "down": "mlp.e{e}.down"}


def build_zurolorn_spec(cfg: ZurolornConfig) -> ModelSpec:
    positions: dict[str, PartSpec] = {}
    by_params: dict[tuple, str] = {}
    layers, ignored = [], []
    for i, layer in enumerate(cfg.layers):
        m, name = layer.mixer, None
        if m.rot_dim:
            name = by_params.setdefault((m.rot_dim, m.rot_base), f"rot{len(by_params)}")     # equal rotations share one table
            positions[name] = PartSpec("yarn", {"head_dim": m.rot_dim, "rotary_dim": m.rot_dim, "base": m.rot_base, "scaling": None})
        mixer = PartSpec("latent_attention", {
            "num_heads": m.heads, "head_dim": m.dim, "rot_dim": m.rot_dim, "value_dim": m.vdim, "rank": m.kv_rank,
            "q_rank": m.q_rank, "norm_eps": cfg.norm_eps, "position": name, "scale": m.scale,
            **({"names": DIRECT_NAMES, "pairs": "halves", "gate": True} if layer.type == "latent_attention"
               else {"names": Q_LATENT_NAMES, "pairs": "neighbours"}),
        })
        ff = ff_norm = None
        scales = {"mixer_scale": "ls1"}
        if layer.mlp is not None:
            f = layer.mlp
            ff = PartSpec("routed_experts", {
                "num_experts": f.experts, "top_k": f.top, "intermediate_size": f.ff, "names": EXPERT_NAMES,
                "expert": "squared_relu", "score": "sigmoid", "weight_on": "output", "weight_scale": f.scale,
                "groups": None if f.groups is None else {"count": f.groups, "keep": f.keep},
            })
            ff_norm = PartSpec("rmsnorm", {"eps": cfg.norm_eps, "name": "norm2"})
            scales["feed_forward_scale"] = "ls2"
        else:
            ignored += [f"l{i}.norm2", f"l{i}.ls2"]       # nothing reads them in a layer without a feed-forward
        layers.append(LayerSpec(
            prefix=f"l{i}.", mixer=mixer, feed_forward=ff, mixer_norm=PartSpec("rmsnorm", {"eps": cfg.norm_eps, "name": "norm1"}),
            feed_forward_norm=ff_norm, block="prenorm", block_params=scales,
        ))

    # The order: layers in front of the repeated stretch, the stretch once per pass, the rest.
    n, loop = len(cfg.layers), cfg.loop
    transforms: dict[str, PartSpec] = {}
    sequence = [(i, 0, False) for i in range(n)]
    if loop is not None:
        transforms["pass"] = PartSpec("pass_step", {"passes": loop.times, "name": "loop.step"})
        sequence = [(i, 0, False) for i in range(loop.start)]
        for p in range(loop.times):
            sequence += [(i, p, i == loop.start) for i in range(loop.start, loop.stop)]
        sequence += [(i, 0, False) for i in range(loop.stop, n)]
    order = tuple(LayerRun(i, entry, True, before=("pass",) if opens else (), pass_index=p)
                  for entry, (i, p, opens) in enumerate(sequence))
    return ModelSpec(
        vocab_size=cfg.vocab_size, hidden_size=cfg.hidden_size, embedding="embed", layers=tuple(layers), order=order,
        final_norm=PartSpec("rmsnorm", {"eps": cfg.norm_eps, "name": "final.norm"}), final_norm_prefix="", head="head",
        positions=positions, max_position=MAX_POSITION, stop_token_ids=cfg.stop_token_ids, ignored_weights=tuple(ignored),
        embedding_transforms=(PartSpec("scale", {"factor": cfg.embedding_scale}),),
        logit_transforms=(PartSpec("scale", {"factor": cfg.logit_scale}),), stream_transforms=transforms,
    )


register_architecture("Zurolorn", ZurolornConfig, build_zurolorn_spec)
