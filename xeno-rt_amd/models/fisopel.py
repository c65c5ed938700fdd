"""Fisopel: a decoder of layers whose mixer and experts stand side by side, each behind a norm of its own, described in parts.

Embedding times a constant; then the layers that config.json lists, of which a run may be gone through several times in a row. A layer
is x += mixer(norm1(x)) + feed_forward(norm2(x)) with RMS norms, both of the same x. Before every pass of the layers that are gone
through several times, the stream is made anew from what it holds and from the embedding's rows by one matrix
(parts/block.py: PassEntry); each pass has cache entries of its own. The mixers:
  latent_attention  softmax attention whose keys and values are made from a cached latent; queries straight from the layer's input, a
                    part of every query and one shared key part turned by rotary positions in pairs of halves, with frequencies
                    stretched for long contexts; every output of every head times the sigmoid of a number of its own (parts/latent.py)
  attention         grouped softmax attention without positions: RMS norms of the heads of q and k, a tanh cap on the scores, a learnt
                    sink per head, and a window that keeps a sequence's first tokens in sight (parts/attention.py)
The feed-forward is a mixture of experts weighed by a softmax over the chosen ones' logits, beside a shared expert that every token
uses as it is, or absent. Final norm, then the embedding table as the output head, without the constant.
Tensor names: `embed`, `loop.in`, `l<i>.norm1|norm2`, `l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`.
"""
from __future__ import annotations

from ..config import register_architecture
from ..config.fisopel import FisopelConfig
from ..parts import Attention, Embedding, ExpertsMLP, LatentAttention, OutputHead, PairRotation, ParallelBlock, PassEntry, RMSNorm
from .decoder import LayerCall, ModelSpec


def _mixer(kind: str, m: dict, p: str, c: FisopelConfig):
    if kind == "latent_attention":
        rot = m["rot"]
        position = PairRotation(rot["dims"], rot["base"], neighbours=False, scaling=rot.get("scaling"))
        return LatentAttention(p, c.width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], None, m["scale"], c.norm_eps, rot["dims"],
                               rot["base"], sink=None, output_gate="g", gate_per="output", position=position)
    mask = m.get("mask")
    return Attention(p, c.width, m["heads"], m["kv_heads"], m["dim"], qk_norm=True, qk_norm_eps=c.norm_eps, scale=m["scale"], value_dim=m["vdim"],
                     sink="sink", softcap=m.get("softcap"), window=None if mask is None else mask["size"],
                     keep_first=0 if mask is None else mask.get("keep_first", 0),
                     names={"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"})


def _feed_forward(mlp, p: str, c: FisopelConfig):
    if mlp is None:
        return None
    router, shared = mlp["router"], mlp.get("shared")
    return ExpertsMLP(p, c.width, mlp["expert"]["ff"], router["experts"], router["top"], scores="softmax",
                      shared=None if shared is None else shared["ff"], shared_gate=None)


def build_fisopel(config: FisopelConfig) -> ModelSpec:
    c = config
    layers = []
    for index, layer in enumerate(c.layers):
        p = f"l{index}."
        feed_forward = _feed_forward(layer["mlp"], p + "mlp.", c)
        layers.append(ParallelBlock(RMSNorm(p, c.width, c.norm_eps, name=p + "norm1"), _mixer(layer["type"], layer["mixer"], p + "mix.", c), feed_forward,
                                    feed_forward_norm=None if feed_forward is None else RMSNorm(p, c.width, c.norm_eps, name=p + "norm2"),
                                    unread=[] if feed_forward is not None else [p + "norm2"]))
    embedding = Embedding("", c.vocab, c.width, name="embed", scale=c.embedding_scale)
    return ModelSpec(config=c, embedding=embedding, layers=layers, schedule=[LayerCall(layer, enters=enters) for layer, enters in c.order()],
                     final_norm=RMSNorm("", c.width, c.norm_eps, name="final.norm"), head=OutputHead("", c.vocab, c.width, tied_to=embedding),
                     entry=None if c.loop is None else PassEntry("loop.in", c.width))


register_architecture("Fisopel", FisopelConfig, build_fisopel)
