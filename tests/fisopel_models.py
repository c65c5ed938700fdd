"""Small Fisopel configurations for the tests, and model folders with random weights for them.

The configurations differ from each other in every size and option: windows of one token, smaller than a cache block, one token wider
than it, several blocks wide and none; none, one and several first tokens kept, less than a cache block and more than one, fewer and
more than the window holds; scores capped hard, loosely and not at all; one head, heads with a key/value head each, several on one; values
wider and narrower than keys; latents narrower and wider than a head; sizes in whole tiles of the matrix cores and multiples of
nothing; rotations with frequencies stretched and plain; experts of which one, some and all are chosen, with a shared expert narrower
or wider than they are and without one, and layers without experts; passes from the first layer on, from a later one, over all layers,
one, two and three of them, and none at all.
"""
import os

import torch


def _attention(heads, kv_heads, dim, vdim, scale, mlp, size=None, keep_first=0, softcap=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        mixer["mask"] = {"size": size, "keep_first": keep_first}
    if softcap is not None:
        mixer["softcap"] = softcap
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def _latent(heads, dim, rot_dim, vdim, kv_rank, scale, base, mlp, scaling=None):
    rot = {"dims": rot_dim, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "rot": rot},
            "mlp": mlp}


def _moe(ff, experts, top, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return mlp


def _model(vocab, width, eps, scale, layers, loop=None):
    raw = {"architecture": "Fisopel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}
    if loop is not None:
        raw["loop"] = dict(zip(("start", "stop", "times"), loop))
    return raw


MIXED = _model(101, 48, 1e-5, 2.5, [
    _latent(3, 16, 8, 12, 24, 0.3, 1000.0, _moe(24, 6, 2, 40), scaling=(4.0, 64, 8.0, 0.5)),
    _attention(4, 2, 20, 28, 0.4, _moe(16, 5, 3), size=24, keep_first=3, softcap=2.0),
    _attention(6, 3, 12, 12, 0.5, None, size=65, keep_first=70, softcap=8.0),
    _latent(1, 20, 12, 28, 40, 0.2, 50.0, _moe(20, 4, 1, 12)),
], loop=(1, 3, 2))

# sizes in whole tiles: the matrix-core kernels in bfloat16, sorted picks for steps of many tokens
TILES = _model(130, 64, 1e-6, 0.5, [
    _attention(8, 2, 64, 96, 0.3, _moe(64, 4, 1, 128), size=40, keep_first=5, softcap=3.0),
    _latent(5, 24, 32, 48, 96, 0.2, 5000.0, _moe(128, 6, 3, 64), scaling=(8.0, 32, 4.0, 1.0)),
    _attention(20, 1, 32, 32, 0.5, _moe(64, 8, 2), size=33, keep_first=34),
    _attention(3, 3, 128, 64, 0.2, _moe(64, 3, 2, 192), softcap=5.0),
], loop=(0, 1, 3))

# edges: a window of one token, everything chosen, a loop over all layers that is gone through once, nothing capped, a scale of one
EDGES = _model(64, 32, 1e-3, 1.0, [
    _attention(2, 1, 8, 4, 1.0, _moe(12, 3, 3, 8), size=1, keep_first=1),
    _latent(6, 8, 2, 4, 40, 0.5, 10.0, None, scaling=(1.0, 16, 2.0, 2.0)),
    _attention(5, 5, 16, 24, 0.3, _moe(16, 5, 1), size=64, keep_first=64, softcap=0.5),
], loop=(0, 3, 1))

# sizes that are multiples of nothing, and no passes
ODD = _model(33, 50, 1e-4, 7.0, [
    _attention(3, 1, 5, 3, 0.6, _moe(9, 3, 2, 5), size=13, keep_first=2, softcap=4.0),
    _latent(2, 7, 6, 11, 9, 0.4, 30.0, _moe(21, 7, 2, 3)),
    _attention(2, 2, 9, 17, 0.3, _moe(11, 2, 1)),
])

CONFIGS = {"mixed": MIXED, "tiles": TILES, "edges": EDGES, "odd": ODD}


def make_fisopel_folder(raw_config, folder, seed, std=0.12, router_std=0.3):
    """A model folder for `raw_config` with the library's random weights, where the small tensors are then given values that make
    them matter: gains away from one, sinks of either sign, a router and gates whose numbers differ, and a matrix before the passes
    that keeps about as much as it is given."""
    from xeno_rt_amd.config import parse_config
    from xeno_rt_amd.weights import SafetensorsFile, write_random_model, write_safetensors

    folder = str(folder)
    write_random_model(parse_config(raw_config), folder, seed=seed, std=std)
    path = os.path.join(folder, "model.safetensors")
    with SafetensorsFile(path) as file:
        tensors = {name: file.read(name) for name in file.names()}
    generator = torch.Generator().manual_seed(seed + 1)
    for name, tensor in tensors.items():
        last = name.split(".")[-1]
        if last in ("norm1", "norm2", "norm"):
            mean, deviation = 1.0, 0.3
        elif last == "sink":
            mean, deviation = 0.5, 1.0
        elif last in ("router", "g"):
            mean, deviation = 0.0, router_std
        elif name == "loop.in":
            mean, deviation = 0.0, (1.5 / tensor.shape[1]) ** 0.5
        elif name == "embed":
            mean, deviation = 0.0, 0.3
        else:
            continue
        tensors[name] = (mean + deviation * torch.randn(tensor.shape, generator=generator)).to(tensor.dtype)
    write_safetensors(path, tensors)
    return folder
