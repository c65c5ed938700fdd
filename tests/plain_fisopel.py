"""The Fisopel decoder in plain, slow arithmetic: float64, whole sequences, no cache, no batch, one function per mechanism.

It shares no code with the package. `tensors` maps checkpoint names to torch tensors, `config` is config.json as a dict.
x is the residual stream [tokens, width], h what a sublayer reads, t a token's index in its sequence (its position).
"""
from __future__ import annotations

import json
import math
import os
import struct

import torch

F = torch.float64


def silu(z):
    return z * torch.sigmoid(z)


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w.to(F)


# ---- what enters the stream, what enters it again, what leaves it ---------------------------------------------------------

def embedding(ids, table, scale):
    return table[torch.as_tensor(ids, dtype=torch.long)].to(F) * scale


def enter_pass(x, first, w):
    """The stream before a pass of the layers that run several times: a matrix on [what the stream holds | what it began with]."""
    return torch.cat([x, first], dim=-1) @ w.to(F).T


def output_logits(x, gain, table, eps):
    return rms_norm(x, gain, eps) @ table.to(F).T


# ---- rotation of halves, with frequencies stretched for contexts beyond the trained one --------------------------------------

def frequencies(dims, base, scaling):
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return plain, 1.0
    def pair_with(turns):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(pair_with(scaling["fast"])), 0)
    hi = min(math.ceil(pair_with(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        share = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(share * f / scaling["factor"] + (1.0 - share) * f)
    return out, 1.0 + 0.1 * math.log(scaling["factor"])


def turn_halves(part, rot):
    """part [tokens, ..., r]: of its first rot.dims numbers, number i and number i + dims / 2 turn together by position * frequency i."""
    dims = rot["dims"]
    table, magnitude = frequencies(dims, rot["base"], rot.get("scaling"))
    out = part.clone()
    for t in range(part.shape[0]):
        for i, f in enumerate(table):
            cos, sin = magnitude * math.cos(t * f), magnitude * math.sin(t * f)
            u, v = part[t, ..., i], part[t, ..., i + dims // 2]
            out[t, ..., i] = u * cos - v * sin
            out[t, ..., i + dims // 2] = v * cos + u * sin
    return out


# ---- which keys a query sees ---------------------------------------------------------------------------------------------------

def seen(tokens, size=None, keep_first=0):
    """[queries, keys]: keys at or before the query that are fewer than `size` tokens behind it, or among the sequence's first
    `keep_first` (size None: all of them)."""
    i, j = torch.arange(tokens)[:, None], torch.arange(tokens)[None, :]
    causal = j <= i
    return causal if size is None else causal & ((i - j < size) | (j < keep_first))


# ---- attention through a latent --------------------------------------------------------------------------------------------------

def latent_rows(h, p, m, eps):
    """What a token leaves for later ones: the normed latent, and the key part that all heads share, turned."""
    down = h @ p["dkv"].to(F).T
    latent = rms_norm(down[:, :m["kv_rank"]], p["dkv.norm"], eps)
    return latent, turn_halves(down[:, m["kv_rank"]:], m["rot"])


def latent_attention(h, p, m, eps):
    heads, d, r, e = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    tokens = h.shape[0]
    q = (h @ p["q"].to(F).T).reshape(tokens, heads, d + r)
    q_plain, q_turned = q[..., :d], turn_halves(q[..., d:], m["rot"])
    latent, k_turned = latent_rows(h, p, m, eps)
    k_plain = (latent @ p["uk"].to(F).T).reshape(tokens, heads, d)
    v = (latent @ p["uv"].to(F).T).reshape(tokens, heads, e)
    scores = (torch.einsum("ihd,jhd->hij", q_plain, k_plain) + torch.einsum("ihr,jr->hij", q_turned, k_turned)) * m["scale"]
    weights = torch.softmax(scores.masked_fill(~seen(tokens), -math.inf), dim=-1)
    o = torch.einsum("hij,jhe->ihe", weights, v).reshape(tokens, heads * e)
    return (o * torch.sigmoid(h @ p["g"].to(F).T)) @ p["o"].to(F).T


# ---- attention under a window that keeps a sequence's first tokens ---------------------------------------------------------------

def cap(scores, limit):
    return scores if limit is None else limit * torch.tanh(scores / limit)


def weights_with_sink(scores, mask, sink):
    """softmax over the keys that are seen, whose denominator also holds exp(sink of the head); scores [heads, queries, keys]."""
    scores = scores.masked_fill(~mask, -math.inf)
    if sink is None:
        return torch.softmax(scores, dim=-1)
    extra = sink.to(F)[:, None, None].expand(scores.shape[0], scores.shape[1], 1)
    return torch.softmax(torch.cat([scores, extra], dim=-1), dim=-1)[..., :-1]


def attention(h, p, m, eps):
    heads, groups, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    tokens = h.shape[0]
    q = rms_norm((h @ p["q"].to(F).T).reshape(tokens, heads, d), p["q.norm"], eps)
    k = rms_norm((h @ p["k"].to(F).T).reshape(tokens, groups, d), p["k.norm"], eps)
    v = (h @ p["v"].to(F).T).reshape(tokens, groups, e)
    k, v = (t.repeat_interleave(heads // groups, dim=1) for t in (k, v))
    scores = cap(torch.einsum("ihd,jhd->hij", q, k) * m["scale"], m.get("softcap"))
    mask = m.get("mask") or {}
    weights = weights_with_sink(scores, seen(tokens, mask.get("size"), mask.get("keep_first") or 0), p.get("sink"))
    return torch.einsum("hij,jhe->ihe", weights, v).reshape(tokens, heads * e) @ p["o"].to(F).T


MIXERS = {"latent_attention": latent_attention, "attention": attention}


# ---- experts -----------------------------------------------------------------------------------------------------------------------

def expert(h, gate, up, down):
    return (silu(h @ gate.to(F).T) * (h @ up.to(F).T)) @ down.to(F).T


def choose(z, top):
    """(chosen experts, their weights) of one token from its router logits: a softmax over the largest of them alone."""
    chosen = sorted(range(len(z)), key=lambda e: (-float(z[e]), e))[:top]
    largest = max(float(z[e]) for e in chosen)
    powers = [math.exp(float(z[e]) - largest) for e in chosen]
    return chosen, [p / sum(powers) for p in powers]


def experts(h, p, mlp):
    z = h @ p["router"].to(F).T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(*choose(z[t], mlp["router"]["top"])):
            out[t] += w * expert(h[t:t + 1], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])[0]
    if mlp.get("shared") is not None:
        out = out + expert(h, p["shared.gate"], p["shared.up"], p["shared.down"])
    return out


# ---- the model -----------------------------------------------------------------------------------------------------------------------

def part(tensors, prefix):
    return {name[len(prefix):]: t for name, t in tensors.items() if name.startswith(prefix)}


def add_layer(x, tensors, index, layer, eps):
    """x after one layer: both sublayers read the same stream, each through a norm of its own."""
    p = f"l{index}."
    y = MIXERS[layer["type"]](rms_norm(x, tensors[p + "norm1"], eps), part(tensors, p + "mix."), layer["mixer"], eps)
    if layer.get("mlp") is not None:
        y = y + experts(rms_norm(x, tensors[p + "norm2"], eps), part(tensors, p + "mlp."), layer["mlp"])
    return x + y


def order(config):
    """The layers in the order in which they run, as (layer, whether a pass begins before it)."""
    count, loop = len(config["layers"]), config.get("loop")
    if loop is None:
        return [(i, False) for i in range(count)]
    begin, end = loop["start"], loop["stop"]
    once = [(i, i == begin) for i in range(begin, end)]
    return [(i, False) for i in range(begin)] + once * loop["times"] + [(i, False) for i in range(end, count)]


def residual_after_layers(config, tensors, ids):
    eps = config["norm"]["eps"]
    first = x = embedding(ids, tensors["embed"], config["embedding"]["scale"])
    out = []
    for index, begins in order(config):
        if begins:
            x = enter_pass(x, first, tensors["loop.in"])
        x = add_layer(x, tensors, index, config["layers"][index], eps)
        out.append(x)
    return out


def logits(config, tensors, ids):
    """float64 [tokens, vocab] for one whole sequence."""
    x = residual_after_layers(config, tensors, ids)[-1]
    return output_logits(x, tensors["final.norm"], tensors["embed"], config["norm"]["eps"])


def load_folder(folder):
    """(config, tensors) of a model folder, read without the package."""
    with open(os.path.join(folder, "config.json")) as handle:
        config = json.load(handle)
    with open(os.path.join(folder, "model.safetensors"), "rb") as handle:
        size = struct.unpack("<Q", handle.read(8))[0]
        header = json.loads(handle.read(size))
        data = handle.read()
    kinds = {"BF16": torch.bfloat16, "F32": torch.float32, "I32": torch.int32}
    tensors = {}
    for name, entry in header.items():
        if name != "__metadata__":
            begin, end = entry["data_offsets"]
            tensors[name] = torch.frombuffer(bytearray(data[begin:end]), dtype=kinds[entry["dtype"]]).reshape(entry["shape"])
    return config, tensors


class PlainModel:
    def __init__(self, folder):
        self.config, self.tensors = load_folder(folder)

    def logits(self, ids):
        with torch.no_grad():
            return logits(self.config, self.tensors, list(ids)).to(torch.float32)


def generate_greedy(model, prompt, count):
    ids, out = list(prompt), []
    for _ in range(count):
        token = int(model.logits(ids)[-1].argmax())
        out.append(token)
        ids.append(token)
    return out
