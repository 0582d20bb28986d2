"""The Verelorn design as a list of parts: the builder registered for ``model_type: verelorn`` (a ``config.json`` that
says ``"architecture": "Verelorn"``).

A layer is a ``HyperBlock``: several residual streams in 32-bit, an RMS norm with a gain stored around zero in front of
each sublayer, and a causal convolution that adds to what the mixer reads.  The mixer is attention whose values are its
keys (biases on queries and keys, a rotation with stretched low frequencies, a learned number per head in the softmax's
sum, an output gate), the gated delta rule with a decay per key channel, or latent attention with queries through a latent
of their own, over its own cached latents or an earlier layer's.  The feed-forward is dense with a tanh-GELU gate, or
absent.  The embedding is normed; the head is a matrix of its own on the final norm of the streams' sum.

Tensor names: ``embed``, ``embed.norm``, ``final.norm``, ``head``, and per layer i ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.hc1.*``, ``l<i>.hc2.*``, ``l<i>.canon1``, ``l<i>.mix.<name>``, ``l<i>.mlp.<name>``.

Storage per sequence: latent layers with equal cache rows share a page pool without values (a layer that reads another's
latents names that layer's part of it); attention layers with equal kv heads and page head size share a page pool with
values; delta-rule layers of one shape share a state table; the convolutions' last inputs of all layers are one more.
"""
from __future__ import annotations

from typing import Dict, List, Tuple

from ..config.registry import register
from ..config.verelorn import VerelornConfig
from ..parts import (ChannelDeltaMixer, Embedding, GatedAttentionMixer, GatedFeedForward, HyperBlock, LatentAttentionMixer,
                     NoPositions, OutputHead, RMSNorm, RotaryPositions)
from ..parts.positions import llama3_frequencies
from .spec import CACHE_FULL, CACHE_STATE, CacheGroupSpec, LayerCall, ModelSpec


def _norm(name: str, cfg: VerelornConfig) -> RMSNorm:
    return RMSNorm(name, cfg.width, cfg.eps, offset=1.0)


def _positions(rot, head_dim: int, pairing: str):
    if not rot:
        return NoPositions()
    dims, base, sc = int(rot["dims"]), float(rot["base"]), rot.get("scaling")
    table = None
    if sc:
        table = llama3_frequencies(dims, base, float(sc["factor"]), float(sc["low"]), float(sc["high"]), sc["original"], precise=True)
    return RotaryPositions(head_dim, base, inv_freq=table, rotary_dim=dims, pairing=pairing)


def _mixer(cfg: VerelornConfig, i: int):
    layer, prefix = cfg.layers[i], f"l{i}.mix"
    m, kind = layer["mixer"], layer["type"]
    if kind == "attention":
        return GatedAttentionMixer(prefix, cfg.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]), cfg.eps,
                                   _positions(m.get("rot"), m["dim"], "half"), qk_norm=False, v_norm=False, gate=True, bias="qk",
                                   v_from_k=True, sink=True)
    if kind == "channel_delta":
        return ChannelDeltaMixer(prefix, cfg.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"],
                                 cfg.inner_rank(i, "a_rank"), cfg.inner_rank(i, "g_rank"), cfg.eps)
    return LatentAttentionMixer(prefix, cfg.width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], float(m["scale"]),
                                cfg.eps, _positions(m.get("rot"), m["rot_dim"], "interleaved"), q_rank=m["q_rank"],
                                reads_other=m.get("kv_from") is not None)


def build_verelorn(cfg: VerelornConfig) -> ModelSpec:
    H = cfg.width
    blocks, order = [], []
    groups: Dict[Tuple, List] = {}  # what a layer keeps -> [name, layers so far]
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        mixer = _mixer(cfg, i)
        ffn = norm2 = None
        if layer.get("mlp") is not None:
            ffn, norm2 = GatedFeedForward(f"{p}.mlp", H, layer["mlp"]["ff"], "gelu_tanh"), _norm(f"{p}.norm2", cfg)
        blocks.append(HyperBlock(p, mixer, ffn, _norm(f"{p}.norm1", cfg), norm2, cfg.streams, H, cfg.taps, f"{p}.canon1"))
        more = (("conv", "canon", i),) if cfg.taps > 1 else ()
        source = layer["mixer"].get("kv_from") if layer["type"] == "latent_attention" else None
        if source is not None:  # another layer's cache rows, as that layer has written them
            order.append(LayerCall(i, order[source].cache_group, order[source].cache_layer, write_cache=False, more=more))
            continue
        if isinstance(mixer, LatentAttentionMixer):
            key = ("latent", 1, mixer.cache_row)
        elif isinstance(mixer, GatedAttentionMixer):
            key = ("kv", mixer.kv_heads, mixer.frame)
        else:
            key = ("delta", mixer.state_shape, 0)
        g = groups.setdefault(key, [f"{key[0]}{len(groups)}", 0])
        order.append(LayerCall(i, g[0], g[1], more=more))
        g[1] += 1
    cache_groups = [CacheGroupSpec("canon", CACHE_STATE, len(order), state_shape=((cfg.taps - 1) * H,))] if cfg.taps > 1 else []
    for (kind, heads, size), (name, count) in groups.items():
        if kind == "delta":
            cache_groups.append(CacheGroupSpec(name, CACHE_STATE, count, state_shape=heads))
        else:
            cache_groups.append(CacheGroupSpec(name, CACHE_FULL, count, heads, size, values=kind == "kv"))
    return ModelSpec(
        config=cfg,
        embedding=Embedding("embed", cfg.vocab, H, weight_name="embed", norm=_norm("embed.norm", cfg)),
        blocks=blocks,
        order=order,
        final_norm=_norm("final.norm", cfg),
        head=OutputHead("head", cfg.vocab, H, None, weight_name="head"),
        cache_groups=cache_groups,
    )


register("verelorn", VerelornConfig, build_verelorn, exist_ok=True, aliases=("Verelorn",))
