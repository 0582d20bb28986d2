"""The Narezen design as a list of parts: the builder registered for ``model_type: narezen`` (a ``config.json`` that says
``"architecture": "Narezen"``).

A layer is a ``SandwichBlock`` of RMS norms over a 32-bit stream.  The mixer is two mixers side by side (``SideBySideMixer``) --
attention whose values are its keys, with normed heads, no rotation and a learned sink per head, beside linear attention with
a decay per head and key channel; or rotated attention with one added to the softmax's sum, beside retention (linear attention
with rotated queries and keys and a constant decay per head) -- or a real-gated linear recurrent unit.  The feed-forward is
routed experts whose unnormalised sigmoid scores multiply the experts' inputs, plus a shared expert; or absent.  The embedding
is scaled; the head is a matrix of its own on the final norm, its logits capped by a tanh.

Tensor names: ``embed``, ``final.norm``, ``head``, and per layer i ``l<i>.norm1``, ``l<i>.norm1b``, ``l<i>.norm2``, ``l<i>.norm2b``,
``l<i>.mix.<name>`` (``l<i>.mix.left.<name>``, ``l<i>.mix.right.<name>``), ``l<i>.mlp.<name>``.

Storage per sequence: attention halves with equal kv heads and page head size share a page pool; linear halves of one state
shape share a state table, as do recurrent units of one shape.
"""
from __future__ import annotations

from typing import Dict, List, Tuple

from ..config.narezen import NarezenConfig
from ..config.registry import register
from ..parts import (Embedding, GatedAttentionMixer, LinearStateMixer, NoPositions, OutputHead, RealGatedMixer, RMSNorm, RotaryPositions,
                     RoutedFeedForward, SandwichBlock, SideBySideMixer)
from .spec import CACHE_FULL, CACHE_STATE, CacheGroupSpec, LayerCall, ModelSpec


def _norm(name: str, cfg: NarezenConfig) -> RMSNorm:
    return RMSNorm(name, cfg.width, cfg.eps)


def _positions(rot, head_dim: int):
    if not rot:
        return NoPositions()
    # (a head of an odd size is rotated in its even first part)
    return RotaryPositions(head_dim + head_dim % 2, float(rot["base"]), rotary_dim=int(rot["dims"]))


def _mixer(cfg: NarezenConfig, i: int):
    layer, prefix = cfg.layers[i], f"l{i}.mix"
    m, kind = layer["mixer"], layer["type"]
    if kind == "rglru":
        return RealGatedMixer(prefix, cfg.width, m["width"], m["blocks"], m["conv"])
    l, r = m["left"], m["right"]
    if kind == "parallel":
        left = GatedAttentionMixer(f"{prefix}.left", cfg.width, l["heads"], l["kv_heads"], l["dim"], l["vdim"], float(l["scale"]), cfg.eps,
                                   NoPositions(), qk_norm="plain", v_norm=False, gate=False, v_from_k=True, sink=True)
        right = LinearStateMixer(f"{prefix}.right", cfg.width, r["heads"], r["dim"], r["vdim"], cfg.eps, NoPositions(),
                                 q_scale=r["dim"] ** -0.5, tau=float(r["tau"]), decay_rank=cfg.decay_rank(i))
    else:
        left = GatedAttentionMixer(f"{prefix}.left", cfg.width, l["heads"], l["kv_heads"], l["dim"], l["vdim"], float(l["scale"]), cfg.eps,
                                   _positions(l.get("rot"), l["dim"]), qk_norm=False, v_norm=False, gate=False, sink="one")
        right = LinearStateMixer(f"{prefix}.right", cfg.width, r["heads"], r["dim"], r["vdim"], cfg.eps, _positions(r.get("rot"), r["dim"]),
                                 k_scale=r["dim"] ** -0.5, decay=r["decay"], gain=False)
    return SideBySideMixer(prefix, left, right, float(m["left_scale"]), float(m["right_scale"]))


def _feed_forward(cfg: NarezenConfig, prefix: str, mlp: dict) -> RoutedFeedForward:
    r, shared = mlp["router"], mlp.get("shared")
    return RoutedFeedForward(prefix, cfg.width, mlp["expert"]["ff"], r["experts"], r["top"], score="sigmoid", normalise=False, act="silu",
                             shared_ff=int(shared["ff"]) if shared else 0, weight_input=True)


def build_narezen(cfg: NarezenConfig) -> ModelSpec:
    H = cfg.width
    blocks, order = [], []
    groups: Dict[Tuple, List] = {}  # what a layer keeps -> [name, layers so far]

    def storage(key: Tuple) -> Tuple[str, int]:
        g = groups.setdefault(key, [f"{key[0]}{len(groups)}", 0])
        g[1] += 1
        return g[0], g[1] - 1

    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        mixer = _mixer(cfg, i)
        ffn = norm2 = norm2b = None
        if layer.get("mlp") is not None:
            ffn, norm2, norm2b = _feed_forward(cfg, f"{p}.mlp", layer["mlp"]), _norm(f"{p}.norm2", cfg), _norm(f"{p}.norm2b", cfg)
        blocks.append(SandwichBlock(mixer, ffn, _norm(f"{p}.norm1", cfg), _norm(f"{p}.norm1b", cfg), norm2, norm2b))
        if isinstance(mixer, SideBySideMixer):
            group, at = storage(("kv", mixer.left.kv_heads, mixer.left.frame))
            order.append(LayerCall(i, group, at, more=(("right",) + storage(("linear", mixer.right.state_shape, 0)),)))
        else:
            order.append(LayerCall(i, *storage(("rglru", mixer.state_shape, 0))))
    cache_groups = []
    for (kind, size, frame), (name, count) in groups.items():
        if kind == "kv":
            cache_groups.append(CacheGroupSpec(name, CACHE_FULL, count, size, frame))
        else:
            cache_groups.append(CacheGroupSpec(name, CACHE_STATE, count, state_shape=size))
    return ModelSpec(
        config=cfg,
        embedding=Embedding("embed", cfg.vocab, H, weight_name="embed", scale=float(cfg.embedding["scale"])),
        blocks=blocks,
        order=order,
        final_norm=_norm("final.norm", cfg),
        head=OutputHead("head", cfg.vocab, H, None, weight_name="head", softcap=cfg.softcap),
        cache_groups=cache_groups,
    )


register("narezen", NarezenConfig, build_narezen, exist_ok=True, aliases=("Narezen",))
