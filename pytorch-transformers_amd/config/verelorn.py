"""Typed configuration of the Verelorn design: a decoder with several residual streams whose layers are listed one by one in
``config.json``, each with the kind of its token mixer (``attention``: grouped heads whose values are their keys, a
learned number per head in the softmax's sum, an output gate; ``channel_delta``: the gated delta rule with a decay per key
channel; ``latent_attention``: attention over cached latents, its own or an earlier layer's, queries through a latent),
that mixer's sizes and constants, and its feed-forward (dense with a tanh-GELU gate, or none).

Keys of ``config.json``: ``architecture`` ("Verelorn"), ``vocab``, ``width``, ``streams``, ``norm`` (``{"eps"}``), ``canon``
(``{"taps"}``: the inputs of the convolution in front of every mixer), ``layers`` (a list of ``{"type", "mixer": {...},
"mlp": {"kind": "dense", "ff"} or null}``).

Mixer ``attention``: ``heads``, ``kv_heads``, ``dim``, ``vdim`` (equal to ``dim``), ``scale``, ``rot``.  Mixer
``latent_attention``: ``heads``, ``dim``, ``rot_dim``, ``vdim``, ``kv_rank``, ``q_rank``, ``scale``, ``rot``, ``kv_from`` (the
layer whose latents it reads; absent: its own).  Mixer ``channel_delta``: ``heads``, ``kv_heads``, ``dim``, ``vdim``,
``conv`` (taps), and optionally ``a_rank`` and ``g_rank``, the inner sizes of the decays' and the output gate's products,
which otherwise follow from the weight file's tensors (``vdim`` where there is none).  ``rot``: ``{"base", "dims",
"scaling": {"factor", "low", "high", "original"} or absent}``; absent: no rotation.
"""
from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Dict, List

from .base import ConfigError, ModelConfig
from .bimepel import _number, _positive_int

MIXER_SIZES = {
    "attention": ("heads", "kv_heads", "dim", "vdim"),
    "channel_delta": ("heads", "kv_heads", "dim", "vdim", "conv"),
    "latent_attention": ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"),
}
INNER_RANKS = {"a_rank": "a1", "g_rank": "g1"}  # key -> the tensor whose rows it counts


def _check_rot(where: str, rot, most: int, what: str) -> None:
    if not isinstance(rot, dict) or "base" not in rot or "dims" not in rot:
        raise ConfigError(f"{where}.rot must give 'base' and 'dims'")
    _positive_int(f"{where}.rot", rot, "dims")
    if _number(f"{where}.rot", rot, "base") <= 0:
        raise ConfigError(f"{where}.rot: 'base' must be positive")
    if rot["dims"] % 2 or rot["dims"] > most:
        raise ConfigError(f"{where}.rot.dims ({rot['dims']}) must be even and at most {what} ({most})")
    sc = rot.get("scaling")
    if sc is not None:
        for k in ("factor", "low", "high", "original"):
            if _number(f"{where}.rot.scaling", sc, k) <= 0:
                raise ConfigError(f"{where}.rot.scaling: {k!r} must be positive")
        if sc["high"] <= sc["low"]:
            raise ConfigError(f"{where}.rot.scaling: 'high' ({sc['high']}) must be above 'low' ({sc['low']})")


@dataclasses.dataclass
class VerelornConfig(ModelConfig):
    model_type: ClassVar[str] = "verelorn"

    architecture: str = "Verelorn"
    vocab: int = 512
    width: int = 256
    streams: int = 2
    layers: List[Dict[str, Any]] = dataclasses.field(default_factory=list)
    norm: Dict[str, Any] = dataclasses.field(default_factory=lambda: {"eps": 1e-6})
    canon: Dict[str, Any] = dataclasses.field(default_factory=lambda: {"taps": 4})
    tie_word_embeddings: bool = False
    initializer_range: float = 0.05

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])

    @property
    def taps(self) -> int:
        return int(self.canon["taps"])

    def inner_rank(self, layer: int, key: str) -> int:
        m = self.layers[layer]["mixer"]
        return int(m.get(key) or m["vdim"])

    def sizes_from_weights(self, shapes) -> None:
        if not any(l["type"] == "channel_delta" and l["mixer"].get(k) is None for l in self.layers for k in INNER_RANKS):
            return
        held = shapes()
        layers = [dict(l, mixer=dict(l["mixer"])) for l in self.layers]  # (entries of the list may be one object)
        for i, layer in enumerate(layers):
            if layer["type"] != "channel_delta":
                continue
            for key, tensor in INNER_RANKS.items():
                shape = held.get(f"l{i}.mix.{tensor}")
                if layer["mixer"].get(key) is None and shape is not None and len(shape) == 2:
                    layer["mixer"][key] = int(shape[0])
        self.layers = layers

    def validate(self) -> None:
        me = dataclasses.asdict(self)
        for key in ("vocab", "width", "streams"):
            _positive_int("config", me, key)
        if not isinstance(self.norm, dict) or "eps" not in self.norm:
            raise ConfigError("config: 'norm' must be an object with the key 'eps'")
        _positive_int("config.canon", self.canon, "taps")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("config: 'layers' must list at least one layer")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            kind = layer.get("type") if isinstance(layer, dict) else None
            if kind not in MIXER_SIZES:
                raise ConfigError(f"{where}: type {kind!r} is not built; built: {', '.join(sorted(MIXER_SIZES))}")
            mixer = layer.get("mixer")
            if not isinstance(mixer, dict):
                raise ConfigError(f"{where}: 'mixer' must hold the mixer's sizes")
            missing = [k for k in MIXER_SIZES[kind] if k not in mixer]
            if missing:
                raise ConfigError(f"{where} ({kind}): the mixer lacks {', '.join(missing)}")
            for k in MIXER_SIZES[kind]:
                _positive_int(f"{where}.mixer", mixer, k)
            if "kv_heads" in MIXER_SIZES[kind] and mixer["heads"] % mixer["kv_heads"]:
                raise ConfigError(f"{where}: {mixer['heads']} heads are no multiple of {mixer['kv_heads']} kv heads")
            if kind == "channel_delta":
                for k in INNER_RANKS:
                    if mixer.get(k) is not None:
                        _positive_int(f"{where}.mixer", mixer, k)
            else:
                if "scale" not in mixer:
                    raise ConfigError(f"{where} ({kind}): the mixer lacks scale")
                _number(f"{where}.mixer", mixer, "scale")
                turned, what = (mixer["rot_dim"], "rot_dim") if kind == "latent_attention" else (mixer["dim"], "dim")
                if mixer.get("rot") is not None:
                    _check_rot(f"{where}.mixer", mixer["rot"], turned, what)
            if kind == "attention" and mixer["vdim"] != mixer["dim"]:
                raise ConfigError(f"{where}: values that are the keys have the keys' size: vdim {mixer['vdim']}, dim {mixer['dim']}")
            if kind == "latent_attention" and mixer.get("kv_from") is not None:
                self._check_kv_from(i, where, mixer)
            mlp = layer.get("mlp")
            if mlp is None:
                continue
            if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
                raise ConfigError(f"{where}.mlp: kind {mlp.get('kind') if isinstance(mlp, dict) else mlp!r} is not built; "
                                  "built: dense, or null for no feed-forward")
            _positive_int(f"{where}.mlp", mlp, "ff")

    def _check_kv_from(self, i: int, where: str, mixer: dict) -> None:
        j = mixer["kv_from"]
        if isinstance(j, bool) or not isinstance(j, int) or not (0 <= j < i):
            raise ConfigError(f"{where}.mixer.kv_from: {j!r} is no earlier layer")
        other = self.layers[j]
        if other["type"] != "latent_attention" or other["mixer"].get("kv_from") is not None:
            raise ConfigError(f"{where}.mixer.kv_from: layer {j} has no latents of its own")
        for k in ("kv_rank", "rot_dim", "rot"):
            if mixer.get(k) != other["mixer"].get(k):
                raise ConfigError(f"{where}.mixer.kv_from: {k} is {mixer.get(k)} here and {other['mixer'].get(k)} in layer {j}")
