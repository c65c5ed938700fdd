"""Small Mitunex configurations for the tests, and model folders with random weights for them.

The configurations differ from each other in every size and option: windows smaller than a cache block, one token wider than it,
several blocks wide, of a single token, and none; one head and more heads than a matrix-core tile has columns; values wider and
narrower than keys; latents narrower and wider than a head, in whole tiles and not; turned parts of two to thirty-two dims; plain
feed-forwards, experts of which one, some and all are chosen, with a shared expert narrower or wider than they are and without one,
and layers without a feed-forward; layers that run an earlier layer's weights once or several times, a later layer's, and those of a
layer that runs another's.
"""
import os

import torch


def _layer(heads, dim, rot_dim, vdim, kv_rank, scale, base, window, mlp, weights_of=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "rot": {"dims": rot_dim, "base": base}}
    if window is not None:
        mixer["mask"] = {"size": window}
    layer = {"type": "latent_attention", "mixer": mixer, "mlp": mlp}
    if weights_of is not None:
        layer["weights_of"] = weights_of
    return layer


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return mlp


def _again(layers, index):
    return dict(layers[index], weights_of=index)


def _model(vocab, width, max_positions, eps, scale, cap, layers):
    return {"architecture": "Mitunex", "vocab": vocab, "width": width, "max_positions": max_positions, "norm": {"eps": eps},
            "logit_scale": scale, "logit_softcap": cap, "layers": layers}


_mixed = [_layer(3, 16, 8, 12, 24, 0.3, 1000.0, 24, _dense(72)), _layer(2, 20, 4, 28, 40, 0.25, 50.0, 65, _moe(24, 6, 2, 40))]
MIXED = _model(101, 48, 700, 1e-5, 1.5, 12.0, _mixed + [_again(_mixed, 1), _layer(1, 12, 6, 8, 16, 0.4, 10.0, 7, None), _again(_mixed, 0)])

# sizes in whole tiles: the matrix-core kernels in bfloat16, sorted picks for steps of many tokens
_tiles = [_layer(5, 24, 32, 48, 96, 0.2, 5000.0, 100, _moe(64, 4, 1, 128)), _layer(18, 16, 64, 16, 64, 0.15, 200.0, 33, _dense(96)),
          _layer(4, 40, 32, 24, 160, 0.2, 1e5, None, _moe(128, 6, 3))]
TILES = _model(130, 64, 512, 1e-6, 0.5, 40.0, [_tiles[0], _tiles[1], _again(_tiles, 0), _tiles[2]])
TILES["layers"][2]["weights_of"] = 0

# edges: a window of one token, all experts chosen, a scale of one, a layer that runs a later layer's weights, and one that runs that one's
_edges = [_layer(6, 8, 2, 4, 40, 0.5, 10.0, 1, _moe(12, 3, 3, 8)), _layer(2, 32, 16, 36, 20, 0.2, 3000.0, 64, _moe(16, 5, 1))]
EDGES = _model(64, 32, 400, 1e-3, 1.0, 5.0, [dict(_edges[1], weights_of=2), _edges[0], _edges[1], dict(_edges[1], weights_of=0)])

# sizes that are multiples of nothing
ODD = _model(33, 50, 300, 1e-4, 3.0, 7.5, [_layer(3, 5, 2, 3, 7, 0.3, 100.0, 13, _moe(9, 3, 2, 5)), _layer(1, 7, 4, 11, 9, 0.4, 30.0, 90, _dense(21))])

CONFIGS = {"mixed": MIXED, "tiles": TILES, "edges": EDGES, "odd": ODD}


def make_mitunex_folder(raw_config, folder, seed, std=0.12, router_std=0.15):
    """A model folder for `raw_config` with the library's random weights, where the small tensors are then given values that make
    them matter: gains away from one, a router and gates whose numbers differ, positions as large as the tokens' rows."""
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
        elif last in ("router", "g", "sg"):
            mean, deviation = 0.0, router_std
        else:
            continue
        tensors[name] = (mean + deviation * torch.randn(tensor.shape, generator=generator)).to(tensor.dtype)
    write_safetensors(path, tensors)
    return folder
