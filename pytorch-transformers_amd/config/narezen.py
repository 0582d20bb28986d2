"""Typed configuration of the Narezen design: a decoder whose layers are listed one by one in ``config.json``, each with the kind
of its token mixer (``parallel``: attention whose values are its keys beside linear attention with a decay per key channel;
``parallel_2``: rotated attention beside retention; ``rglru``: a real-gated linear recurrent unit), that mixer's sizes and
constants, and its feed-forward (routed experts with a shared one, or none).

Keys of ``config.json``: ``architecture`` ("Narezen"), ``vocab``, ``width``, ``embedding`` (``{"scale"}``), ``norm`` (``{"eps"}``),
``logit_softcap`` (absent or null: none), ``layers`` (a list of ``{"type", "mixer": {...}, "mlp": {...} or null}``).

Mixers ``parallel`` and ``parallel_2``: ``left``, ``right``, ``left_scale``, ``right_scale``.  ``left``: ``heads``, ``kv_heads``, ``dim``,
``vdim`` (in ``parallel`` equal to ``dim``), ``scale``, in ``parallel_2`` also ``rot``.  ``right``: ``heads``, ``dim``, ``vdim``, and in
``parallel`` ``tau`` and optionally ``a_rank``, the inner size of the decays' product, which otherwise follows from the weight
file's tensors (``dim`` where there is none), in ``parallel_2`` ``decay`` (one a head) and ``rot``.  Mixer ``rglru``: ``width``,
``blocks``, ``conv`` (taps).  ``rot``: ``{"base", "dims"}``; absent: no rotation.  ``mlp``: ``{"kind": "moe", "expert": {"ff"},
"router": {"experts", "top"}, "shared": {"ff"} or absent}``.
"""
from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Dict, List

from .base import ConfigError, ModelConfig
from .bimepel import _number, _positive_int

LEFT_SIZES = ("heads", "kv_heads", "dim", "vdim")
RIGHT_SIZES = ("heads", "dim", "vdim")
KINDS = ("parallel", "parallel_2", "rglru")


def _check_rot(where: str, rot, dim: int) -> None:
    if rot is None:
        return
    if not isinstance(rot, dict) or "base" not in rot or "dims" not in rot:
        raise ConfigError(f"{where}.rot must give 'base' and 'dims'")
    _positive_int(f"{where}.rot", rot, "dims")
    if _number(f"{where}.rot", rot, "base") <= 0:
        raise ConfigError(f"{where}.rot: 'base' must be positive")
    if rot["dims"] % 2 or rot["dims"] > dim:
        raise ConfigError(f"{where}.rot.dims ({rot['dims']}) must be even and at most dim ({dim})")


@dataclasses.dataclass
class NarezenConfig(ModelConfig):
    model_type: ClassVar[str] = "narezen"

    architecture: str = "Narezen"
    vocab: int = 512
    width: int = 256
    layers: List[Dict[str, Any]] = dataclasses.field(default_factory=list)
    embedding: Dict[str, Any] = dataclasses.field(default_factory=lambda: {"scale": 1.0})
    norm: Dict[str, Any] = dataclasses.field(default_factory=lambda: {"eps": 1e-6})
    logit_softcap: Any = None
    tie_word_embeddings: bool = False
    initializer_range: float = 0.05

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])

    @property
    def softcap(self) -> float:
        return float(self.logit_softcap or 0.0)

    def decay_rank(self, layer: int) -> int:
        """The inner size of the product that makes a ``parallel`` layer's decays."""
        r = self.layers[layer]["mixer"]["right"]
        return int(r.get("a_rank") or r["dim"])

    def sizes_from_weights(self, shapes) -> None:
        open_layers = [i for i, l in enumerate(self.layers) if l["type"] == "parallel" and l["mixer"]["right"].get("a_rank") is None]
        if not open_layers:
            return
        held = shapes()
        layers = list(self.layers)
        for i in open_layers:  # (entries of the list may be one object)
            shape = held.get(f"l{i}.mix.right.a1")
            if shape is not None and len(shape) == 2:
                mixer = layers[i]["mixer"]
                layers[i] = dict(layers[i], mixer=dict(mixer, right=dict(mixer["right"], a_rank=int(shape[0]))))
        self.layers = layers

    def validate(self) -> None:
        me = dataclasses.asdict(self)
        for key in ("vocab", "width"):
            _positive_int("config", me, key)
        if not isinstance(self.norm, dict) or "eps" not in self.norm:
            raise ConfigError("config: 'norm' must be an object with the key 'eps'")
        _number("config.embedding", self.embedding, "scale")
        if self.logit_softcap is not None and _number("config", me, "logit_softcap") < 0:
            raise ConfigError("config: 'logit_softcap' must be positive, or 0 or absent for none")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("config: 'layers' must list at least one layer")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            kind = layer.get("type") if isinstance(layer, dict) else None
            if kind not in KINDS:
                raise ConfigError(f"{where}: type {kind!r} is not built; built: {', '.join(KINDS)}")
            mixer = layer.get("mixer")
            if not isinstance(mixer, dict):
                raise ConfigError(f"{where}: 'mixer' must hold the mixer's sizes")
            if kind == "rglru":
                for k in ("width", "blocks", "conv"):
                    _positive_int(f"{where}.mixer", mixer, k)
                if mixer["width"] % mixer["blocks"]:
                    raise ConfigError(f"{where}: {mixer['width']} channels do not split into {mixer['blocks']} equal blocks")
            else:
                self._check_halves(where, kind, mixer)
            self._check_mlp(where, layer.get("mlp"))

    def _check_halves(self, where: str, kind: str, mixer: dict) -> None:
        for k in ("left", "right"):
            if not isinstance(mixer.get(k), dict):
                raise ConfigError(f"{where}.mixer lacks {k!r}")
            _number(f"{where}.mixer", mixer, f"{k}_scale")
        left, right = mixer["left"], mixer["right"]
        for k in LEFT_SIZES:
            _positive_int(f"{where}.mixer.left", left, k)
        _number(f"{where}.mixer.left", left, "scale")
        if left["heads"] % left["kv_heads"]:
            raise ConfigError(f"{where}: {left['heads']} heads are no multiple of {left['kv_heads']} kv heads")
        for k in RIGHT_SIZES:
            _positive_int(f"{where}.mixer.right", right, k)
        if kind == "parallel":
            if left["vdim"] != left["dim"]:
                raise ConfigError(f"{where}: values that are the keys have the keys' size: vdim {left['vdim']}, dim {left['dim']}")
            if _number(f"{where}.mixer.right", right, "tau") <= 0:
                raise ConfigError(f"{where}.mixer.right: 'tau' must be positive")
            if right.get("a_rank") is not None:
                _positive_int(f"{where}.mixer.right", right, "a_rank")
        else:
            _check_rot(f"{where}.mixer.left", left.get("rot"), left["dim"])
            _check_rot(f"{where}.mixer.right", right.get("rot"), right["dim"])
            decay = right.get("decay")
            if not isinstance(decay, list) or len(decay) != right["heads"]:
                raise ConfigError(f"{where}.mixer.right.decay must list one decay for each of the {right['heads']} heads")

    @staticmethod
    def _check_mlp(where: str, mlp) -> None:
        if mlp is None:
            return
        if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
            raise ConfigError(f"{where}.mlp: kind {mlp.get('kind') if isinstance(mlp, dict) else mlp!r} is not built; "
                              "built: moe, or null for no feed-forward")
        _positive_int(f"{where}.mlp.expert", mlp.get("expert"), "ff")
        for k in ("experts", "top"):
            _positive_int(f"{where}.mlp.router", mlp.get("router"), k)
        if mlp["router"]["top"] > mlp["router"]["experts"]:
            raise ConfigError(f"{where}.mlp.router: top {mlp['router']['top']} of {mlp['router']['experts']} experts")
        if mlp.get("shared") is not None:
            _positive_int(f"{where}.mlp.shared", mlp["shared"], "ff")
