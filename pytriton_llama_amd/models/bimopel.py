"""``Bimopel``: layers given as a list, each with one of two mixers (Mamba-2; softmax attention inside
chunks of the positions beside gated linear attention, both results normed and averaged) and a dense
GELU-gated feed-forward or none, an RMS norm behind every residual sum on a float32 stream whose old
value is scaled first, sinusoidal positions added to the scaled embedding, a head matrix of its own
and capped logits. The model is a list of layer specs over the engine's parts; tensor names are the
checkpoint's own ("l<i>.mix.in", "l<i>.mix.left.q", "l<i>.mix.right.out", "l<i>.norm1", ...).
"""
from __future__ import annotations

from ..config.bimopel_config import BimopelConfig
from ..config.registry import register_model
from ..parts.base import build_part
from .causal_lm import CausalLM, LayerCall

# role of a part inside a block -> what follows "l<i>." in its tensors' names
BIMOPEL_BLOCK_PREFIXES = {"norm1": "norm1", "norm2": "norm2", "mixer": "mix.", "feed_forward": "mlp."}
POSITION_BASE = 10000.0        # of the sinusoidal positions


def _norm(cfg: BimopelConfig, name: str = ""):
    return build_part("norm", "rmsnorm", size=cfg.hidden_size, eps=cfg.norm_eps, weight_name=name)


def _mixer(cfg: BimopelConfig, layer):
    W, eps, m = cfg.hidden_size, cfg.norm_eps, layer.mixer
    if layer.kind == "mamba2":
        return build_part("mixer", "mamba2", hidden_size=W, num_heads=m.heads, vdim=m.vdim, state=m.state,
                          groups=m.groups, taps=m.conv, norm_groups=m.norm_groups, eps=eps)
    l, r = m.left, m.right
    left = build_part("mixer", "normed_attention", hidden_size=W, num_heads=l.heads, num_kv_heads=l.kv_heads,
                      dim=l.dim, vdim=l.vdim, scale=l.scale, eps=eps, qk_norm="whole", maps=1, bias=True,
                      o_bias=False, head_gated=True, sink=0.0, chunk=l.chunk)
    right = build_part("mixer", "gated_linear_attention", hidden_size=W, num_heads=r.heads, dim=r.dim, vdim=r.vdim,
                       tau=r.tau, eps=eps, rank=r.rank)
    return build_part("mixer", "parallel", left=left, right=right, left_scale=0.5, right_scale=0.5,
                      left_norm=_norm(cfg, "out"), right_norm=_norm(cfg, "out"))


def build_bimopel(cfg: BimopelConfig) -> CausalLM:
    W = cfg.hidden_size
    embedding = build_part("embedding", "token_embedding", vocab_size=cfg.vocab_size, hidden_size=W,
                           weight_name="embed", float32_stream=True, scale=cfg.embedding_scale,
                           sinusoidal=POSITION_BASE)
    blocks, cache_layers, schedule, ranked = [], [], [], []

    def keep(spec):
        cache_layers.append(spec)
        return len(cache_layers) - 1

    for i, layer in enumerate(cfg.layers):
        mixer = _mixer(cfg, layer)
        ffn = None
        if layer.ff:
            ffn = build_part("feed_forward", "swiglu", hidden_size=W, intermediate_size=layer.ff, gate_name="gate",
                             up_name="up", down_name="down", activation="gelu_tanh")
        blocks.append(build_part("block", "post_norm", mixer=mixer, mixer_norm=_norm(cfg), feed_forward=ffn,
                                 ffn_norm=_norm(cfg) if ffn is not None else None, alpha=cfg.postln_alpha))
        spec = mixer.cache_spec()
        schedule.append(LayerCall(i, tuple(keep(s) for s in spec) if isinstance(spec, tuple) else keep(spec), True))
        if layer.kind == "parallel":
            ranked.append((f"l{i}.mix.right.", mixer.right))
    blocks[-1].last = True                  # (the run order is the order of the layers)
    final_norm = _norm(cfg)
    head = build_part("head", "linear_head", vocab_size=cfg.vocab_size, hidden_size=W, weight_name="head",
                      softcap=cfg.logit_softcap)
    prefixes = [("", embedding)]
    for i, b in enumerate(blocks):
        for role, part in b.children().items():
            prefixes.append((f"l{i}.{BIMOPEL_BLOCK_PREFIXES[role]}", part))
    prefixes += [("final.norm", final_norm), ("", head)]
    model = CausalLM(cfg, embedding, blocks, final_norm, head, cache_layers, schedule, prefixes)

    def ranks_from_the_file(names, shape_of):
        """The rank of the decays' projection is not in config.json: the tensors' shapes say."""
        for prefix, mixer in ranked:
            if prefix + mixer.names["a1"] in names:
                mixer.rank_from(prefix, shape_of)
    model.before_load = ranks_from_the_file
    return model


register_model("Bimopel", BimopelConfig, build_bimopel)
