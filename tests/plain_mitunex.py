"""The Mitunex decoder in plain, slow arithmetic: float64, whole sequences, no cache, no batch, one function per mechanism.

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


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w.to(F)


# ---- what enters the stream, and what leaves it --------------------------------------------------------------------------

def embedding(ids, table, positions, gain, eps):
    """A token's row plus its position's row, normed together."""
    ids = torch.as_tensor(ids, dtype=torch.long)
    return rms_norm(table[ids].to(F) + positions[:len(ids)].to(F), gain, eps)


def output_logits(x, gain, head, eps, scale, cap):
    z = rms_norm(x, gain, eps) @ head.to(F).T * scale
    return cap * torch.tanh(z / cap)


# ---- attention through a latent, under a window ---------------------------------------------------------------------------

def turn_neighbours(part, dims, base):
    """part [tokens, ..., r]: its first `dims` numbers in pairs (2i, 2i + 1) turned by position * base^(-2i / dims)."""
    out = part.clone()
    for t in range(part.shape[0]):
        for i in range(dims // 2):
            a = t * base ** (-2.0 * i / dims)
            u, v = part[t, ..., 2 * i], part[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = u * math.cos(a) - v * math.sin(a)
            out[t, ..., 2 * i + 1] = v * math.cos(a) + u * math.sin(a)
    return out


def window_mask(tokens, size):
    """[queries, keys]: what a query sees are the `size` newest tokens up to its own, its own among them (size None: all of them)."""
    behind = torch.arange(tokens)[:, None] - torch.arange(tokens)[None, :]
    seen = behind >= 0
    return seen if size is None else seen & (behind < size)


def latent_rows(h, p, m, eps):
    """What a token leaves for later ones: the normed latent, and the key part that all heads share, turned."""
    down = h @ p["dkv"].to(F).T
    latent = rms_norm(down[:, :m["kv_rank"]], p["dkv.norm"], eps)
    return latent, turn_neighbours(down[:, m["kv_rank"]:], m["rot"]["dims"], m["rot"]["base"])


def head_gate(h, gate):
    return torch.sigmoid(h @ gate.to(F).T)


def latent_attention(h, p, m, eps):
    heads, d, r, e = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    tokens = h.shape[0]
    q = (h @ p["q"].to(F).T).reshape(tokens, heads, d + r)
    q_plain, q_turned = q[..., :d], turn_neighbours(q[..., d:], m["rot"]["dims"], m["rot"]["base"])
    latent, k_turned = latent_rows(h, p, m, eps)
    k_plain = (latent @ p["uk"].to(F).T).reshape(tokens, heads, d)
    v = (latent @ p["uv"].to(F).T).reshape(tokens, heads, e)
    scores = (torch.einsum("ihd,jhd->hij", q_plain, k_plain) + torch.einsum("ihr,jr->hij", q_turned, k_turned)) * m["scale"]
    scores = scores.masked_fill(~window_mask(tokens, (m.get("mask") or {}).get("size")), -math.inf)
    o = torch.einsum("hij,jhe->ihe", torch.softmax(scores, dim=-1), v)
    o = o * head_gate(h, p["g"])[..., None]
    return o.reshape(tokens, heads * e) @ p["o"].to(F).T


# ---- feed-forwards ------------------------------------------------------------------------------------------------------------

def dense(h, p):
    return gelu_tanh(h @ p["up"].to(F).T) @ p["down"].to(F).T


def expert(h, gate, up, down):
    return (silu(h @ gate.to(F).T) * (h @ up.to(F).T)) @ down.to(F).T


def choose(z, top):
    """(chosen experts, their weights) of one token from its router logits: the largest sigmoids, as they are."""
    s = torch.sigmoid(z)
    chosen = sorted(range(len(s)), key=lambda e: (-float(s[e]), e))[:top]
    return chosen, [float(s[e]) for e in chosen]


def experts(h, p, mlp):
    """A chosen expert reads the token's row times the router's weight; a shared expert reads the row itself."""
    z = h @ p["router"].to(F).T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(*choose(z[t], mlp["router"]["top"])):
            out[t] += expert(w * h[t:t + 1], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])[0]
    if mlp.get("shared") is not None:
        out = out + torch.sigmoid(h @ p["shared.sg"].to(F).T) * expert(h, p["shared.gate"], p["shared.up"], p["shared.down"])
    return out


# ---- the model -----------------------------------------------------------------------------------------------------------------

def owner(layers, index):
    """The layer whose tensors layer `index` runs on."""
    while layers[index].get("weights_of") is not None:
        index = layers[index]["weights_of"]
    return index


def part(tensors, prefix):
    return {name[len(prefix):]: t for name, t in tensors.items() if name.startswith(prefix)}


def add_layer(x, tensors, index, layer, eps):
    """x after one layer: each sublayer reads the stream itself, and its output is normed on the way onto it."""
    p = f"l{index}."
    x = x + rms_norm(latent_attention(x, part(tensors, p + "mix."), layer["mixer"], eps), tensors[p + "norm1"], eps)
    mlp = layer.get("mlp")
    if mlp is None:
        return x
    q = part(tensors, p + "mlp.")
    y = dense(x, q) if mlp["kind"] == "dense" else experts(x, q, mlp)
    return x + rms_norm(y, tensors[p + "norm2"], eps)


def residual_after_layers(config, tensors, ids):
    eps = config["norm"]["eps"]
    x = embedding(ids, tensors["embed"], tensors["pos"], tensors["embed.norm"], eps)
    out = []
    for index, layer in enumerate(config["layers"]):
        x = add_layer(x, tensors, owner(config["layers"], index), layer, eps)
        out.append(x)
    return out


def logits(config, tensors, ids):
    """float64 [tokens, vocab] for one whole sequence."""
    x = residual_after_layers(config, tensors, ids)[-1]
    return output_logits(x, tensors["final.norm"], tensors["head"], config["norm"]["eps"], config["logit_scale"], config["logit_softcap"])


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
