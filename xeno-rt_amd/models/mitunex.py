"""Mitunex: a decoder whose sublayers read the residual stream itself and are normed on their way back onto it, described in parts.

Embedding plus a learnt vector per position, RMS-normed; then the layers that config.json lists. A layer is
x += norm1(mixer(x)), x += norm2(feed_forward(x)) with RMS norms. The mixer:
  latent_attention  softmax attention under a sliding window whose keys and values are made from a cached latent; queries
                    straight from the layer's input, a part of every query and one shared key part turned by rotary positions
                    in pairs of neighbours, every head's output times the sigmoid of a number of its own (parts/latent.py)
The feed-forward is a plain one with the tanh form of gelu (`dense`), a mixture of experts chosen by sigmoid scores that multiply
what the chosen experts read, beside a shared expert with a gate of its own (`moe`), or absent. A layer with `weights_of`
runs another layer's weights once more, with a cache entry of its own. Final norm, output head, a factor on the logits
and a tanh cap.
Tensor names: `embed`, `pos`, `embed.norm`, `l<i>.norm1|norm2`, `l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`, `head`.
"""
from __future__ import annotations

from ..config import register_architecture
from ..config.mitunex import MitunexConfig
from ..parts import DenseMLP, ExpertsMLP, LatentAttention, OutputHead, PositionedEmbedding, PostNormBlock, RMSNorm
from .decoder import LayerCall, ModelSpec


def _mixer(m: dict, p: str, c: MitunexConfig) -> LatentAttention:
    mask, rot = m.get("mask"), m["rot"]
    return LatentAttention(p, c.width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], None, m["scale"], c.norm_eps, rot["dims"],
                           rot["base"], sink=None, window=None if mask is None else mask["size"], output_gate="g")


def _feed_forward(mlp, p: str, c: MitunexConfig):
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return DenseMLP(p, c.width, mlp["ff"], "gelu_tanh")
    router, shared = mlp["router"], mlp.get("shared")
    return ExpertsMLP(p, c.width, mlp["expert"]["ff"], router["experts"], router["top"], normalized=False, weigh_input=True,
                      shared=None if shared is None else shared["ff"])


def build_mitunex(config: MitunexConfig) -> ModelSpec:
    c = config
    layers, place = [], {}            # place: a layer of config.json that has weights -> its place in `layers`
    for index, layer in enumerate(c.layers):
        if c.weights_of(index) != index:
            continue
        p = f"l{index}."
        feed_forward = _feed_forward(layer["mlp"], p + "mlp.", c)
        place[index] = len(layers)
        layers.append(PostNormBlock(_mixer(layer["mixer"], p + "mix.", c), RMSNorm(p, c.width, c.norm_eps, name=p + "norm1"), feed_forward,
                                    None if feed_forward is None else RMSNorm(p, c.width, c.norm_eps, name=p + "norm2"),
                                    unread=[] if feed_forward is not None else [p + "norm2"]))
    schedule = [LayerCall(place[c.weights_of(index)]) for index in range(len(c.layers))]
    return ModelSpec(config=c, embedding=PositionedEmbedding("", c.vocab, c.width, c.max_positions, name="embed", positions_name="pos",
                                                             norm=("embed.norm", c.norm_eps)),
                     layers=layers, schedule=schedule, final_norm=RMSNorm("", c.width, c.norm_eps, name="final.norm"),
                     head=OutputHead("", c.vocab, c.width, name="head", softcap=c.logit_softcap, scale=c.logit_scale))


register_architecture("Mitunex", MitunexConfig, build_mitunex)
