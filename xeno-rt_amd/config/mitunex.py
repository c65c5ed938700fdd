"""Configuration of the Mitunex decoder: layers of windowed attention through a latent, each before a feed-forward, a mixture of
experts or nothing, some of which run another layer's weights.

config.json names the design under `architecture`; every entry of its `layers` has a `type` (`latent_attention`), the mixer's
sizes under `mixer` (`heads`, `dim`, `rot_dim`, `vdim`, `kv_rank`, `scale`, `rot.dims|base`, `mask.size`: the window, which may be
absent for none), and `mlp`: `kind` "dense" with `ff`, `kind` "moe" with `expert.ff`, `router.experts|top` and `shared.ff` (absent: no
shared expert), or null. An entry with `weights_of`: j has the same sizes as layer j and runs on its tensors. Beside the layers:
`vocab`, `width`, `max_positions` (rows of the table of positions), `norm.eps`, `logit_scale`, `logit_softcap`.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Optional, Tuple

from . import ConfigError, _positive_int, _require
from .sozopel import _number, _sizes

MIXER_TYPES = ("latent_attention",)
MLP_KINDS = ("dense", "moe")


def _part(raw: dict, key: str, where: str) -> dict:
    value = raw.get(key)
    if not isinstance(value, dict):
        raise ConfigError(f"config.json: {where}: '{key}' must be an object, found {value!r}")
    return value


def _check_mixer(mixer: dict, where: str) -> None:
    _sizes(mixer, ("heads", "dim", "rot_dim", "vdim", "kv_rank"), where)
    _number(mixer, "scale", where)
    rot = _part(mixer, "rot", where)
    _sizes(rot, ("dims",), where + ".rot")
    if rot["dims"] % 2 != 0 or rot["dims"] > mixer["rot_dim"]:
        raise ConfigError(f"config.json: {where}.rot: {rot['dims']} dims turn in pairs inside a part of {mixer['rot_dim']}")
    if _number(rot, "base", where + ".rot") <= 0:
        raise ConfigError(f"config.json: {where}.rot: 'base' must be positive")
    if mixer.get("mask") is not None:
        _sizes(_part(mixer, "mask", where), ("size",), where + ".mask")


def _check_mlp(mlp: dict, where: str) -> None:
    if not isinstance(mlp, dict) or mlp.get("kind") not in MLP_KINDS:
        raise ConfigError(f"config.json: {where}: 'kind' must be one of {MLP_KINDS}")
    if mlp["kind"] == "dense":
        _sizes(mlp, ("ff",), where)
        return
    _sizes(_part(mlp, "expert", where), ("ff",), where + ".expert")
    router = _part(mlp, "router", where)
    _sizes(router, ("experts", "top"), where + ".router")
    if router["top"] > router["experts"]:
        raise ConfigError(f"config.json: {where}.router: {router['top']} of {router['experts']} experts chosen")
    if mlp.get("shared") is not None:
        _sizes(_part(mlp, "shared", where), ("ff",), where + ".shared")


@dataclass(frozen=True)
class MitunexConfig:
    architecture: str
    vocab: int
    width: int
    max_positions: int
    norm_eps: float
    logit_scale: float
    logit_softcap: float
    layers: Tuple[dict, ...]                    # as config.json lists them: {"type", "mixer", "mlp"} and, for a layer that runs another's, "weights_of"
    eos_token_ids: Tuple[int, ...] = ()
    bos_token_id: Optional[int] = None

    # what the rest of the library asks of any configuration
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def max_position_embeddings(self) -> int:
        return self.max_positions

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def weights_of(self, index: int) -> int:
        """The layer whose tensors layer `index` runs on: itself, or the one it names, or the one that names."""
        while self.layers[index].get("weights_of") is not None:
            index = self.layers[index]["weights_of"]
        return index

    @classmethod
    def from_dict(cls, raw: dict) -> "MitunexConfig":
        layers = _require(raw, "layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        kept = []
        for index, layer in enumerate(layers):
            where = f"layers[{index}]"
            if not isinstance(layer, dict) or layer.get("type") not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where}: 'type' must be one of {MIXER_TYPES}")
            _check_mixer(_part(layer, "mixer", where), where + ".mixer")
            mlp = layer.get("mlp")
            if mlp is not None:
                _check_mlp(mlp, where + ".mlp")
            entry = {"type": layer["type"], "mixer": layer["mixer"], "mlp": mlp}
            if layer.get("weights_of") is not None:
                entry["weights_of"] = layer["weights_of"]
            kept.append(copy.deepcopy(entry))
        for index, layer in enumerate(kept):
            source, hops = layer.get("weights_of"), 0
            while source is not None:
                if isinstance(source, bool) or not isinstance(source, int) or not 0 <= source < len(kept) or hops > len(kept):
                    raise ConfigError(f"config.json: layers[{index}]: 'weights_of' must lead to a layer with weights of its own, found {layer['weights_of']!r}")
                if any(kept[source][key] != layer[key] for key in ("type", "mixer", "mlp")):
                    raise ConfigError(f"config.json: layers[{index}]: layer {source}, whose weights it runs on, has other sizes")
                source, hops = kept[source].get("weights_of"), hops + 1
        norm = _part(raw, "norm", "the configuration")
        softcap = _number(raw, "logit_softcap", "the configuration")
        if softcap <= 0:
            raise ConfigError("config.json: 'logit_softcap' must be positive")
        eos = raw.get("eos_token_id")
        eos = () if eos is None else tuple(eos) if isinstance(eos, list) else (eos,)
        return cls(architecture=str(raw.get("architecture") or raw["architectures"][0]), vocab=_positive_int(raw, "vocab"),
                   width=_positive_int(raw, "width"), max_positions=_positive_int(raw, "max_positions"), norm_eps=_number(norm, "eps", "norm"),
                   logit_scale=_number(raw, "logit_scale", "the configuration"), logit_softcap=softcap, layers=tuple(kept),
                   eos_token_ids=tuple(int(e) for e in eos), bos_token_id=raw.get("bos_token_id"))

    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "max_positions": self.max_positions,
               "norm": {"eps": self.norm_eps}, "logit_scale": self.logit_scale, "logit_softcap": self.logit_softcap,
               "layers": copy.deepcopy(list(self.layers))}
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        if self.bos_token_id is not None:
            out["bos_token_id"] = self.bos_token_id
        return out

    def __hash__(self):
        return hash((self.architecture, self.vocab, self.width, self.max_positions, len(self.layers)))
