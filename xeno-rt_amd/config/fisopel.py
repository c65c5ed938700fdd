"""Configuration of the Fisopel decoder: layers of two kinds of attention, each beside a mixture of experts, some of which run several
times in a row.

config.json names the design under `architecture` and lists the layers; each entry gives `type` (the mixer: `latent_attention`,
attention whose keys and values are made from a cached latent, or `attention`, grouped attention with head norms, a cap on the scores, a
learnt sink and a window that keeps a sequence's first tokens in sight), the mixer's sizes under `mixer` (`heads`, `dim`, `vdim`,
`scale`; latent: `rot_dim`, `kv_rank`, `rot.dims|base|scaling`, the latter `factor|original|fast|slow` or absent; the other:
`kv_heads`, `softcap`, `mask.size|keep_first`, the last two absent for none), and `mlp`: `kind` "moe" with `expert.ff`,
`router.experts|top` and `shared.ff` (absent: no shared expert), or null. Beside the layers: `vocab`, `width`, `norm.eps`,
`embedding.scale`, and `loop` (`start`, `stop`, `times`: layers start .. stop - 1 run that many times in a row; absent or null: every
layer once).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import List, Optional, Tuple

from . import ConfigError, _positive_int, _require
from .mitunex import _part
from .sozopel import _number, _sizes

MIXER_TYPES = ("latent_attention", "attention")


def _check_mixer(kind: str, mixer: dict, where: str) -> None:
    _number(mixer, "scale", where)
    if kind == "attention":
        _sizes(mixer, ("heads", "kv_heads", "dim", "vdim"), where)
        if mixer["heads"] % mixer["kv_heads"] != 0:
            raise ConfigError(f"config.json: {where}: {mixer['heads']} heads cannot share {mixer['kv_heads']} key/value heads")
        if mixer.get("softcap") is not None and _number(mixer, "softcap", where) <= 0:
            raise ConfigError(f"config.json: {where}: 'softcap' must be positive")
        if mixer.get("mask") is not None:
            mask = _part(mixer, "mask", where)
            _sizes(mask, ("size",), where + ".mask")
            kept = mask.get("keep_first", 0)
            if isinstance(kept, bool) or not isinstance(kept, int) or kept < 0:
                raise ConfigError(f"config.json: {where}.mask: 'keep_first' must be an integer from 0 up, found {kept!r}")
        return
    _sizes(mixer, ("heads", "dim", "rot_dim", "vdim", "kv_rank"), where)
    rot = _part(mixer, "rot", where)
    _sizes(rot, ("dims",), where + ".rot")
    if rot["dims"] % 2 != 0 or rot["dims"] > mixer["rot_dim"]:
        raise ConfigError(f"config.json: {where}.rot: {rot['dims']} dims turn in pairs inside a part of {mixer['rot_dim']}")
    if _number(rot, "base", where + ".rot") <= 0:
        raise ConfigError(f"config.json: {where}.rot: 'base' must be positive")
    if rot.get("scaling") is not None:
        scaling = _part(rot, "scaling", where + ".rot")
        for key in ("factor", "original", "fast", "slow"):
            if _number(scaling, key, where + ".rot.scaling") <= 0:
                raise ConfigError(f"config.json: {where}.rot.scaling: '{key}' must be positive")
        if rot["base"] == 1:
            raise ConfigError(f"config.json: {where}.rot: frequencies that are all one cannot be stretched by how often they turn")


def _check_mlp(mlp, where: str) -> None:
    if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
        raise ConfigError(f"config.json: {where}: 'kind' must be 'moe'")
    _sizes(_part(mlp, "expert", where), ("ff",), where + ".expert")
    router = _part(mlp, "router", where)
    _sizes(router, ("experts", "top"), where + ".router")
    if router["top"] > router["experts"]:
        raise ConfigError(f"config.json: {where}.router: {router['top']} of {router['experts']} experts chosen")
    if mlp.get("shared") is not None:
        _sizes(_part(mlp, "shared", where), ("ff",), where + ".shared")


@dataclass(frozen=True)
class FisopelConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[dict, ...]                    # as config.json lists them: {"type", "mixer", "mlp"}
    loop: Optional[Tuple[int, int, int]] = None     # (start, stop, times), or None
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
    def max_position_embeddings(self):
        return None                             # nothing in the design ends at a position

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def order(self) -> List[Tuple[int, bool]]:
        """The layers in the order in which they run, each with whether a pass of the loop begins before it."""
        count = len(self.layers)
        start, stop, times = (0, 0, 0) if self.loop is None else self.loop
        return ([(i, False) for i in range(start)] + [(i, i == start) for i in range(start, stop)] * times
                + [(i, False) for i in range(stop, count)])

    @classmethod
    def from_dict(cls, raw: dict) -> "FisopelConfig":
        layers = _require(raw, "layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        kept = []
        for index, layer in enumerate(layers):
            where = f"layers[{index}]"
            if not isinstance(layer, dict) or layer.get("type") not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where}: 'type' must be one of {MIXER_TYPES}")
            _check_mixer(layer["type"], _part(layer, "mixer", where), where + ".mixer")
            if layer.get("mlp") is not None:
                _check_mlp(layer["mlp"], where + ".mlp")
            kept.append(copy.deepcopy({"type": layer["type"], "mixer": layer["mixer"], "mlp": layer.get("mlp")}))
        loop = raw.get("loop")
        if loop is not None:
            loop = _part(raw, "loop", "the configuration")
            if any(isinstance(loop.get(key), bool) or not isinstance(loop.get(key), int) for key in ("start", "stop", "times")):
                raise ConfigError("config.json: loop: 'start', 'stop' and 'times' must be integers")
            if not 0 <= loop["start"] < loop["stop"] <= len(kept) or loop["times"] < 1:
                raise ConfigError(f"config.json: loop: layers {loop['start']} to {loop['stop']} of {len(kept)}, {loop['times']} times")
            loop = (loop["start"], loop["stop"], loop["times"])
        norm = _part(raw, "norm", "the configuration")
        embedding = raw.get("embedding") or {}
        if not isinstance(embedding, dict):
            raise ConfigError("config.json: 'embedding' must be an object")
        eos = raw.get("eos_token_id")
        eos = () if eos is None else tuple(eos) if isinstance(eos, list) else (eos,)
        return cls(architecture=str(raw.get("architecture") or raw["architectures"][0]), vocab=_positive_int(raw, "vocab"),
                   width=_positive_int(raw, "width"), norm_eps=_number(norm, "eps", "norm"),
                   embedding_scale=_number(embedding, "scale", "embedding") if "scale" in embedding else 1.0, layers=tuple(kept), loop=loop,
                   eos_token_ids=tuple(int(e) for e in eos), bos_token_id=raw.get("bos_token_id"))

    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "embedding": {"scale": self.embedding_scale}, "layers": copy.deepcopy(list(self.layers))}
        if self.loop is not None:
            out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        if self.bos_token_id is not None:
            out["bos_token_id"] = self.bos_token_id
        return out

    def __hash__(self):
        return hash((self.architecture, self.vocab, self.width, len(self.layers), self.loop))
