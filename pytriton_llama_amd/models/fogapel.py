"""``Fogapel``: layers given as a list, each with one of two mixers (grouped-query attention inside chunks
of the positions, its projections behind short convolutions, queries and keys turned in pairs and
normed behind the rotation, capped scores and one added to the softmax's denominator; the time mixer of
RWKV) and, beside it on the same normed input, a dense clamped feed-forward, routed experts with a shared
one, or none. Both results are scaled entry by entry and added to a float32 stream that starts from the
scaled embedding; the head matrix is its own. The model is a list of layer specs over the engine's parts;
tensor names are the checkpoint's own ("l<i>.mix.q", "l<i>.mix.q.conv", "l<i>.mix.mu.r", "l<i>.mlp.e0.gate",
"l<i>.norm1", "l<i>.ls1", ...).
"""
from __future__ import annotations

from ..config.fogapel_config import FogapelConfig
from ..config.registry import register_model
from ..parts.base import build_part
from .causal_lm import CausalLM, LayerCall

# role of a part inside a block -> what follows "l<i>." in its tensors' names
FOGAPEL_BLOCK_PREFIXES = {"norm1": "norm1", "mixer": "mix.", "feed_forward": "mlp.", "scales": ""}


def _norm(cfg: FogapelConfig):
    return build_part("norm", "rmsnorm", size=cfg.hidden_size, eps=cfg.norm_eps, weight_name="")


def _mixer(cfg: FogapelConfig, layer):
    W, eps, m = cfg.hidden_size, cfg.norm_eps, layer.mixer
    if layer.kind == "wkv":
        return build_part("mixer", "time_mixer", hidden_size=W, num_heads=m.heads, dim=m.dim, eps=eps, rank=m.rank)
    return build_part("mixer", "normed_attention", hidden_size=W, num_heads=m.heads, num_kv_heads=m.kv_heads,
                      dim=m.dim, vdim=m.vdim, scale=m.scale, eps=eps, qk_norm="rotated", maps=1, bias=True,
                      rot_dims=m.rot_dims, rot_base=m.rot_base, rot_layout="pairs", taps=m.conv, softcap=m.softcap,
                      sink=0.0, chunk=m.chunk)


def _feed_forward(cfg: FogapelConfig, mlp):
    if mlp is None:
        return None
    W = cfg.hidden_size
    if mlp.kind == "dense":
        return build_part("feed_forward", "gated_mlp", hidden_size=W, intermediate_size=mlp.ff, activation="clamped",
                          limit=mlp.limit)
    shared = None
    if mlp.shared_ff:
        shared = build_part("feed_forward", "gated_mlp", hidden_size=W, intermediate_size=mlp.shared_ff,
                            activation="silu")
    return build_part("feed_forward", "routed_experts", hidden_size=W, intermediate_size=mlp.ff,
                      num_experts=mlp.experts, top=mlp.top, activation="silu", weight_on_input=False,
                      renormalize=True, score="softmax", router_bias_name="router.b", shared=shared,
                      shared_gate=False)


def build_fogapel(cfg: FogapelConfig) -> CausalLM:
    W = cfg.hidden_size
    embedding = build_part("embedding", "token_embedding", vocab_size=cfg.vocab_size, hidden_size=W,
                           weight_name="embed", float32_stream=True, scale=cfg.embedding_scale)
    blocks, cache_layers, schedule, ranked = [], [], [], []

    def keep(spec):
        cache_layers.append(spec)
        return len(cache_layers) - 1

    for i, layer in enumerate(cfg.layers):
        mixer = _mixer(cfg, layer)
        blocks.append(build_part("block", "parallel_residual", hidden_size=W, mixer=mixer, norm=_norm(cfg),
                                 feed_forward=_feed_forward(cfg, layer.mlp)))
        spec = mixer.cache_spec()
        schedule.append(LayerCall(i, tuple(keep(s) for s in spec) if isinstance(spec, tuple) else keep(spec), True))
        if layer.kind == "wkv":
            ranked.append((f"l{i}.mix.", mixer))
    final_norm = _norm(cfg)
    head = build_part("head", "linear_head", vocab_size=cfg.vocab_size, hidden_size=W, weight_name="head")
    prefixes = [("", embedding)]
    for i, b in enumerate(blocks):
        for role, part in b.children().items():
            prefixes.append((f"l{i}.{FOGAPEL_BLOCK_PREFIXES[role]}", part))
    prefixes += [("final.norm", final_norm), ("", head)]
    # (a layer without a feed-forward has nothing for a second scale to be on)
    unused = [f"l{i}.ls2" for i, layer in enumerate(cfg.layers) if layer.mlp is None]
    model = CausalLM(cfg, embedding, blocks, final_norm, head, cache_layers, schedule, prefixes, unused)

    def ranks_from_the_file(names, shape_of):
        """The rank of the decays' projection is not in config.json: the tensors' shapes say."""
        for prefix, mixer in ranked:
            if prefix + mixer.names["w1"] in names:
                mixer.rank_from(prefix, shape_of)
    model.before_load = ranks_from_the_file
    return model


register_model("Fogapel", FogapelConfig, build_fogapel)
