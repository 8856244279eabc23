"""Modasun as a plan of parts.

A decoder whose layers norm the sum of the weighed stream and a sublayer's result: x = norm1(alpha x + mixer(x)), then
(if the layer has a feed-forward) x = norm2(alpha x + ff(x)); the sublayers read the stream itself, and the norms are RMS
norms whose weight is stored around zero.  The file picks each layer's mixer: causal attention without rotation, with
unit queries and keys and a temperature on the queries that grows with the position; or a gated delta rule with a decay
a head and key channel.  The feed-forward is a squared relu without a gate, or a mixture of silu-gated experts chosen
by sigmoid scores and a correction among the best groups, with an expert behind a gate of its own that every token
uses.  A layer may run another layer's weights once more, with a cache or state of its own.  The head is the embedding
table (without the embedding's factor) behind the model's norm.  Tensor names: `embed`, `final.norm`, and per layer i
with weights of its own `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.*`, and `l<i>.mlp.{up,down}` or `l<i>.mlp.{router,
correction, e<j>.{gate,up,down}, shared.{gate,up,down,sg}}`.
"""
from __future__ import annotations

from wllm_amd.architectures.modasun_config import ModasunConfig
from wllm_amd.config.registry import register_architecture
from wllm_amd.parts.specs import (
    AttentionSpec,
    BlockSpec,
    DeltaRuleSpec,
    EmbeddingSpec,
    GatedMLPSpec,
    HeadSpec,
    MixtureOfExpertsSpec,
    MLPSpec,
    ModelPlan,
    NormSpec,
    PositionSpec,
    ScheduleEntry,
)

# the design names no longest sequence: a request is as long as the cache lets it be
NO_POSITION_LIMIT = 1 << 30
UNIT_EPS = 1e-6             # what the squares' sum of a delta rule's query or key is raised by
ROUTER_EPS = 1e-20          # what the sum of the chosen experts' scores is raised by


def modasun_plan(cfg: ModasunConfig) -> ModelPlan:
    def norm(name: str) -> NormSpec:
        return NormSpec(size=cfg.width, eps=cfg.norm_eps, weight=name, weight_offset=1.0, kind="rms")

    layers, index_of, ignored = [], {}, []
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is not None:
            continue
        m, q = layer.mixer, f"l{i}."
        p = q + "mix."
        if layer.type == "attention":
            mixer = AttentionSpec(
                hidden_size=cfg.width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim,
                scale=m.scale, position=PositionSpec(kind="none"), q_weight=p + "q", k_weight=p + "k", v_weight=p + "v",
                o_weight=p + "o", qk_norm_eps=cfg.norm_eps, q_temperature=m.q_temp, weights_in_float32=True)
        else:
            mixer = DeltaRuleSpec(
                hidden_size=cfg.width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim,
                conv_taps=m.taps, q_scale=m.dim ** -0.5, unit_eps=UNIT_EPS, norm_eps=cfg.norm_eps, decay_rank=m.dim,
                gate_rank=m.dim, q_weight=p + "q", k_weight=p + "k", v_weight=p + "v", q_conv_weight=p + "q.conv",
                k_conv_weight=p + "k.conv", v_conv_weight=p + "v.conv", b_weight=p + "b", a1_weight=p + "a1",
                a2_weight=p + "a2", a_log=p + "A_log", dt_bias=p + "dt_bias", g1_weight=p + "g1", g2_weight=p + "g2",
                norm_weight=p + "norm", o_weight=p + "o")
        ff = None
        if layer.mlp is None:
            ignored.append(q + "norm2")
        elif layer.mlp.kind == "dense":
            ff = MLPSpec(hidden_size=cfg.width, intermediate_size=layer.mlp.ff, activation="squared_relu",
                         up_weight=q + "mlp.up", down_weight=q + "mlp.down")
        else:
            e, s = layer.mlp, q + "mlp.shared."
            shared = None
            if e.shared_ff is not None:
                shared = GatedMLPSpec(hidden_size=cfg.width, intermediate_size=e.shared_ff, activation="silu",
                                      gate_weight=s + "gate", up_weight=s + "up", down_weight=s + "down")
            ff = MixtureOfExpertsSpec(
                hidden_size=cfg.width, intermediate_size=e.ff, num_experts=e.experts, top=e.top, num_groups=e.groups,
                keep_groups=e.keep, weight_eps=ROUTER_EPS, activation="silu", router_weight=q + "mlp.router",
                expert_prefix=q + "mlp.e", scoring="sigmoid", correction_weight=q + "mlp.correction", group_best=2,
                shared=shared, shared_gate_weight=s + "sg" if shared is not None else None)
        index_of[i] = len(layers)
        layers.append(BlockSpec(
            arrangement="norm_of_sum", mixer=mixer, feed_forward=ff, mixer_norm=None, feed_forward_norm=None,
            mixer_post_norm=norm(q + "norm1"), feed_forward_post_norm=norm(q + "norm2") if ff is not None else None,
            stream_weight=cfg.alpha))
    return ModelPlan(
        embedding=EmbeddingSpec(vocab_size=cfg.vocab, hidden_size=cfg.width, weight="embed", scale=cfg.embedding_scale),
        layers=tuple(layers),
        # a layer that uses another's weights is one more run of that layer, with a cache or state of its own
        schedule=tuple(ScheduleEntry(layer=index_of[i if layer.weights_of is None else layer.weights_of])
                       for i, layer in enumerate(cfg.layers)),
        final_norm=norm("final.norm"), head=HeadSpec(vocab_size=cfg.vocab, hidden_size=cfg.width),
        max_positions=NO_POSITION_LIMIT,
        # a layer without a feed-forward does not need its second norm; a file may still carry it
        ignored_tensor_suffixes=tuple(ignored))


register_architecture("Modasun", ModasunConfig.from_dict, modasun_plan)
