"""Tesopel as a plan of parts.

A decoder whose layers have no norm in front of a sublayer and an RMS norm behind it: x += norm1(mixer(x)), then (if
the layer has a feed-forward) x += norm2(ff(x)); the sublayers read the stream itself.  The file picks each layer's
mixer: latent attention inside a sliding window, without positions, over one cached compressed vector a token, which
a later layer may read again with its own matrices; the matrix memory of an mLSTM; or retention (both as Lefisun
has them).  The feed-forward is gated by a swish of slope 1.702 whose inputs are held under a limit, the up
projection raised by one.  The head is the embedding table behind the model's norm, and the logits are multiplied by
a factor.  Tensor names: `embed`, `final.norm`, and per layer i `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.*`,
`l<i>.mlp.{gate,up,down}`.
"""
from __future__ import annotations

from wllm_amd.architectures.lefisun import exponential_memory, retention_memory
from wllm_amd.architectures.tesopel_config import TesopelConfig
from wllm_amd.config.registry import register_architecture
from wllm_amd.parts.specs import (
    BlockSpec,
    EmbeddingSpec,
    GatedMLPSpec,
    HeadSpec,
    LatentAttentionSpec,
    ModelPlan,
    NormSpec,
    ScheduleEntry,
)

# the design names no longest sequence: a request is as long as the cache lets it be
NO_POSITION_LIMIT = 1 << 30
GATE_SLOPE = 1.702          # of the swish in the feed-forward
UP_SHIFT = 1.0              # what the feed-forward's up projection is raised by


def tesopel_plan(cfg: TesopelConfig) -> ModelPlan:
    def norm(name: str) -> NormSpec:
        return NormSpec(size=cfg.width, eps=cfg.norm_eps, weight=name, kind="rms")

    # the windows of all layers that read one cache: its pages go back by the widest, or not at all if one has none
    windows = {}
    for i, layer in enumerate(cfg.layers):
        if layer.type == "latent_attention":
            windows.setdefault(i if layer.mixer.kv_from is None else layer.mixer.kv_from, []).append(layer.mixer.window)
    layers = []
    for i, layer in enumerate(cfg.layers):
        m, q = layer.mixer, f"l{i}."
        p = q + "mix."
        if layer.type == "latent_attention":
            owns = m.kv_from is None
            of_cache = windows[i if owns else m.kv_from]
            mixer = LatentAttentionSpec(
                hidden_size=cfg.width, num_heads=m.heads, head_dim=m.dim, value_dim=m.vdim, kv_rank=m.kv_rank,
                scale=m.scale, norm_eps=cfg.norm_eps, q_weight=p + "q", dkv_weight=p + "dkv" if owns else "",
                dkv_norm_weight=p + "dkv.norm" if owns else "", uk_weight=p + "uk", uv_weight=p + "uv", o_weight=p + "o",
                window=m.window, release_window=None if None in of_cache else max(of_cache), owns_cache=owns,
                weights_in_float32=True)
        elif layer.type == "mlstm":
            mixer = exponential_memory(cfg.width, cfg.norm_eps, m, p)
        else:
            mixer = retention_memory(cfg.width, cfg.norm_eps, m, p)
        ff = None
        if layer.mlp is not None:
            ff = GatedMLPSpec(hidden_size=cfg.width, intermediate_size=layer.mlp.ff, activation="clamped_swish",
                              gate_limit=layer.mlp.limit, gate_slope=GATE_SLOPE, up_shift=UP_SHIFT, gate_weight=q + "mlp.gate",
                              up_weight=q + "mlp.up", down_weight=q + "mlp.down")
        layers.append(BlockSpec(
            arrangement="post_norm", mixer=mixer, feed_forward=ff, mixer_norm=None, feed_forward_norm=None,
            mixer_post_norm=norm(q + "norm1"), feed_forward_post_norm=norm(q + "norm2") if ff is not None else None))
    return ModelPlan(
        embedding=EmbeddingSpec(vocab_size=cfg.vocab, hidden_size=cfg.width, weight="embed"),
        layers=tuple(layers),
        # a layer that expands another layer's compressed vectors: its run reads the cache of that layer's run
        schedule=tuple(ScheduleEntry(layer=i, reads_cache_of=getattr(layer.mixer, "kv_from", None))
                       for i, layer in enumerate(cfg.layers)),
        final_norm=norm("final.norm"),
        head=HeadSpec(vocab_size=cfg.vocab, hidden_size=cfg.width, logit_scale=cfg.logit_scale),
        max_positions=NO_POSITION_LIMIT,
        # a layer without a feed-forward does not need its second norm; a file may still carry it
        ignored_tensor_suffixes=tuple(f"l{i}.norm2" for i, layer in enumerate(cfg.layers) if layer.mlp is None))


register_architecture("Tesopel", TesopelConfig.from_dict, tesopel_plan)
