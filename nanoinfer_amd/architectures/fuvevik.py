"""``Fuvevik``: its configuration keys, its model as a list of parts, its tensor names.

A decoder whose tokens have several float32 streams: a sublayer reads the norm of a weighted sum of the streams, and its
output goes to all of them with a weight each while a small matrix mixes the old streams into the new ones; the streams
start as the embedding's row plus a sinusoid of the position and are summed at the end.  The mixer is causal softmax
attention (grouped heads, a norm a head on queries and keys, no rotation, a query factor that grows with the position, a
sink in the softmax's denominator, a gate a channel), whose keys and values a later layer may read again (``kv_from``).
The feed-forward is dense with squared ReLU, or routed experts with capped hidden units beside experts that give their
input back, chosen by the softmax over all of them plus a correction, weighed by the chosen ones' shares over their sum,
plus one expert every token uses.  The logits read the embedding's table.
Tensor names: ``embed``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.hc1.*``, ``l<i>.hc2.*``,
``final.norm``.
"""
from __future__ import annotations

from typing import Optional

from ..config.fuvevik_config import DenseConfig, FuvevikConfig
from ..config.spec import BlockSpec, LayerRun, ModelSpec, PartSpec
from ..registry import Architecture, register_architecture
from ..weights.random_init import InitRule

POSITIONS = 1 << 24          # beyond it a float32 no longer holds every position
GLU_SLOPE = 1.702            # the slope inside the sigmoid of an expert's hidden units
SINUSOID_BASE = 10000.0


def _mixer(i: int, cfg: FuvevikConfig) -> PartSpec:
    m, pre = cfg.layers[i].mixer, f"l{i}.mix."
    names = {k: pre + k for k in ("q", "sink", "g", "o")}
    names["q_norm"] = pre + "q.norm"
    if m.kv_from is None:
        names.update(k=pre + "k", v=pre + "v", k_norm=pre + "k.norm")
    return PartSpec("sink_attention",
                    {"hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "key_dim": m.dim, "value_dim": m.vdim,
                     "scale": m.scale, "window": None, "cache_window": None, "eps": cfg.norm_eps, "position": None,
                     "shares_kv": m.kv_from is not None, "gate": "channel", "temp_coef": None if m.q_temp is None else m.q_temp[0],
                     "temp_every": None if m.q_temp is None else m.q_temp[1]}, names)


def _feed_forward(i: int, cfg: FuvevikConfig) -> Optional[PartSpec]:
    mlp = cfg.layers[i].mlp
    if mlp is None:
        return None
    d, pre = cfg.width, f"l{i}.mlp."
    if isinstance(mlp, DenseConfig):
        return PartSpec("relu2_mlp", {"hidden_size": d, "intermediate_size": mlp.ff}, {"up": pre + "up", "down": pre + "down"})
    names = {"router": pre + "router", "correction": pre + "correction"}
    for e in range(mlp.experts):
        names.update({f"gate{e}": f"{pre}e{e}.gate", f"up{e}": f"{pre}e{e}.up", f"down{e}": f"{pre}e{e}.down"})
    shared = None
    if mlp.shared is not None:
        shared = PartSpec("capped_glu", {"hidden_size": d, "intermediate_size": mlp.shared[0], "limit": mlp.shared[1], "slope": GLU_SLOPE},
                          {k: f"{pre}shared.{k}" for k in ("gate", "up", "down")})
    return PartSpec("routed_experts", {"hidden_size": d, "expert_size": mlp.ff, "experts": mlp.experts, "identity": mlp.identity,
                                       "top": mlp.top, "activation": "capped_glu", "limit": mlp.limit, "slope": GLU_SLOPE,
                                       "mix": "softmax_share", "shared": shared}, names)


def build_spec(cfg: FuvevikConfig) -> ModelSpec:
    d = cfg.width

    def norm(name: str) -> PartSpec:
        return PartSpec("rmsnorm_one_plus", {"size": d, "eps": cfg.norm_eps}, {"weight": name})

    def link(name: str) -> PartSpec:
        return PartSpec("static", {"streams": cfg.streams}, {k: f"{name}.{k}" for k in ("in", "out", "mix")})

    blocks, order = [], []
    for i, layer in enumerate(cfg.layers):
        parts = {"mixer_link": link(f"l{i}.hc1"), "mixer_norm": norm(f"l{i}.norm1"), "mixer": _mixer(i, cfg)}
        ff = _feed_forward(i, cfg)
        if ff is not None:
            parts.update(ffn_link=link(f"l{i}.hc2"), ffn_norm=norm(f"l{i}.norm2"), ffn=ff)
        blocks.append(BlockSpec(kind="linked_streams", parts=parts, params={"streams": cfg.streams}))
        # a layer that reads another's keys and values runs on that layer's cache and writes nothing there
        source = layer.mixer.kv_from
        order.append(LayerRun(block=i, cache=i if source is None else source, writes_cache=source is None))
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=d, max_positions=POSITIONS,
        embedding=PartSpec("scaled_table", {"vocab_size": cfg.vocab, "hidden_size": d, "scale": 1.0, "max_positions": POSITIONS,
                                            "sinusoid_base": SINUSOID_BASE}, {"weight": "embed"}),
        blocks=blocks, order=order, final_norm=norm("final.norm"),
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": d}, {"weight": "embed"}),
        # a layer without a feed-forward has no use for its second norm and link
        ignorable_suffixes=(".norm2", ".hc2.in", ".hc2.out", ".hc2.mix"),
    )


FUVEVIK = register_architecture(Architecture(
    name="Fuvevik",
    config_from_dict=FuvevikConfig.from_dict,
    build_spec=build_spec,
    init=InitRule(matrix_std=0.05, vector_mean=0.0, vector_std=0.1,
                  overrides=((".q.norm", 1.0, 0.05), (".k.norm", 1.0, 0.05), (".sink", 0.0, 1.0), (".correction", 0.0, 0.05),
                             (".mlp.router", 0.0, 0.3), (".in", 0.5, 0.3), (".out", 0.8, 0.3), ("hc1.mix", 0.3, 0.25), ("hc2.mix", 0.3, 0.25),
                             ("embed", 0.0, 0.5), (".mix.g", 0.0, 0.1))),
))
