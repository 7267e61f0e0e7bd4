"""The Durelix decoder as a ``ModelSpec``.

The token table's rows get a row of a bigram table added (``bigram_embedding``: hashed from the token and the one in front of
it). Every layer normalizes each sub-layer's output before it is added and nothing in front (block "output_norm"). The
mixer is two side by side on the same input (``parallel_mixers``, each output normalized over the width, half their sum):
attention in a sliding window with short convolutions on q, k and v, a weighted norm per head in front of a rotation of
neighbouring pairs, a sink per head and a gate on the output (``paged_attention``), beside retention (``retention``). The
feed-forward, where a layer has one, is down(relu(up x)^2) or a mixture of SiLU-gated experts and identity experts, scored by a
softmax over all of them and chosen by score plus correction inside the best groups. The output matrix is the token table.
Weight names are the checkpoint's own (``l<i>.mix.left.q`` ...).
"""

from __future__ import annotations

from prefixserve_amd.config.durelix import MAX_POSITION, DenseFeedForward, DurelixConfig, Rotary
from prefixserve_amd.config.registry import register_architecture
from prefixserve_amd.parts.attention import slot_size
from prefixserve_amd.parts.retention import padded
from prefixserve_amd.parts.spec import LayerRun, LayerSpec, ModelSpec, PartSpec

ATTENTION_NAMES = {"q": "mix.left.q", "k": "mix.left.k", "v": "mix.left.v", "o": "mix.left.o", "q_norm": "mix.left.q.norm",
                   "k_norm": "mix.left.k.norm", "q_conv": "mix.left.q.conv", "k_conv": "mix.left.k.conv",
                   "v_conv": "mix.left.v.conv", "sink": "mix.left.sink", "gate": "mix.left.g"}
RETENTION_NAMES = {"q": "mix.right.q", "k": "mix.right.k", "v": "mix.right.v", "gate": "mix.right.g", "o": "mix.right.o"}
DENSE_NAMES = {"up": "mlp.up", "down": "mlp.down"}
EXPERT_NAMES = {"router": "mlp.router", "correction": "mlp.correction", "gate": "mlp.e{e}.gate", "up": "mlp.e{e}.up",
                "down": "mlp.e{e}.down"}
# Fixed by the design, not by a file: half the sum of the two mixers' normalized outputs.
MIXER_SHARE = 0.5


def _norm(eps: float, name: str) -> PartSpec:
    return PartSpec("rmsnorm", {"eps": eps, "name": name})


def build_durelix_spec(cfg: DurelixConfig) -> ModelSpec:
    layers, ignored = [], []
    positions: dict[str, PartSpec] = {}
    by_params: dict[tuple, str] = {}

    def rotation(rot: Rotary | None, head_dim: int) -> str:
        """The encoding for heads of ``head_dim`` slots; equal rotations share one table."""
        dims, base = (rot.dims, rot.base) if rot is not None else (0, 1.0)
        name = by_params.setdefault((head_dim, dims, base), f"rot{len(by_params)}")
        positions[name] = PartSpec("rope", {"head_dim": head_dim, "theta": base, "rotary_dim": dims})
        return name

    for i, layer in enumerate(cfg.layers):
        a, r = layer.mixer.left, layer.mixer.right
        left = PartSpec("paged_attention", {
            "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim, "value_dim": a.vdim, "names": ATTENTION_NAMES,
            "scale": a.scale, "window": a.window, "qk_norm_eps": cfg.norm_eps, "qk_norm_weights": True, "norm_first": True,
            "pairs": "neighbours", "conv_taps": a.conv, "sink": True, "out_gate": True, "exact_weights": True,
            "position": rotation(a.rot, slot_size(a.dim, a.vdim)),
        })
        right = PartSpec("retention", {
            "num_heads": r.heads, "head_dim": r.dim, "value_dim": r.vdim, "decays": r.decay, "names": RETENTION_NAMES,
            "norm_eps": cfg.norm_eps, "position": rotation(r.rot, padded(r.dim)),
        })
        mixer = PartSpec("parallel_mixers", {
            "left": left, "right": right,
            "out_norms": {"left": "mix.left.out", "right": "mix.right.out", "eps": cfg.norm_eps, "scale": MIXER_SHARE},
        })
        ff = ff_norm = None
        if layer.mlp is not None:
            f = layer.mlp
            if isinstance(f, DenseFeedForward):
                ff = PartSpec("dense_mlp", {"intermediate_size": f.ff, "names": DENSE_NAMES, "activation": "squared_relu"})
            else:
                ff = PartSpec("routed_experts", {
                    "num_experts": f.experts, "top_k": f.top, "intermediate_size": f.ff, "names": EXPERT_NAMES, "limit": None,
                    "gate_alpha": 1.0, "up_shift": 0.0, "score": "softmax", "weight_on": "output", "choice_bias": True,
                    "identity": f.identity, "group_score": "max",
                    "groups": None if f.groups is None else {"count": f.groups, "keep": f.keep},
                })
            ff_norm = _norm(cfg.norm_eps, "norm2")
        else:
            ignored.append(f"l{i}.norm2")             # nothing reads it in a layer without a feed-forward
        layers.append(LayerSpec(prefix=f"l{i}.", mixer=mixer, feed_forward=ff, mixer_norm=_norm(cfg.norm_eps, "norm1"),
                                feed_forward_norm=ff_norm, block="output_norm"))
    b = cfg.bigram
    return ModelSpec(
        vocab_size=cfg.vocab_size, hidden_size=cfg.hidden_size, embedding="embed", layers=tuple(layers),
        order=tuple(LayerRun(i, i, True) for i in range(len(layers))), final_norm=_norm(cfg.norm_eps, "final.norm"),
        final_norm_prefix="", head=None, positions=positions, max_position=MAX_POSITION, stop_token_ids=cfg.stop_token_ids,
        ignored_weights=tuple(ignored),
        embedding_transforms=(PartSpec("bigram_embedding", {"buckets": b.buckets, "mul_prev": b.mul_prev, "mul_cur": b.mul_cur,
                                                            "name": "bigram"}),),
    )


register_architecture("Durelix", DurelixConfig, build_durelix_spec)
