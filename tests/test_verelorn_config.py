"""The Verelorn design's configuration, tensor names, sizes read from the weight file and cache groups (no GPU)."""
import copy

import pytest
import torch

import plain_verelorn as P
from pytorch_transformers_amd.config import AutoConfig, ConfigError


def _rot(dims, scaling=False):
    r = {"base": 10000.0, "dims": dims}
    if scaling:
        r["scaling"] = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}
    return r


def _layer(kind, m, mlp={"kind": "dense", "ff": 32}):
    return {"type": kind, "mixer": m, "mlp": mlp}


def _attn(mlp={"kind": "dense", "ff": 32}, **over):
    return _layer("attention", dict({"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 24, "scale": 0.2, "rot": _rot(16, True)}, **over), mlp)


def _latent(mlp=None, **over):
    return _layer("latent_attention", dict({"heads": 3, "dim": 24, "rot_dim": 8, "vdim": 20, "kv_rank": 40, "q_rank": 28, "scale": 0.2,
                                            "rot": _rot(8)}, **over), mlp)


def _delta(mlp=None, **over):
    return _layer("channel_delta", dict({"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 20, "conv": 3}, **over), mlp)


def _cfg(layers, **more):
    return dict({"architecture": "Verelorn", "vocab": 50, "width": 32, "streams": 3, "norm": {"eps": 1e-5}, "canon": {"taps": 4},
                 "layers": layers}, **more)


def test_the_architecture_key_chooses_the_design():
    cfg = AutoConfig.from_dict(_cfg([_latent(), _attn(), _delta()]))
    assert type(cfg).__name__ == "VerelornConfig" and cfg.model_type == "verelorn" and cfg.vocab_size == 50
    assert cfg.eps == 1e-5 and cfg.taps == 4 and cfg.streams == 3
    again = AutoConfig.from_dict(cfg.to_dict())
    assert again.layers == cfg.layers and again.canon == cfg.canon


@pytest.mark.parametrize("layers,more,word", [
    ([dict(_attn(), type="conv")], {}, "type"),
    ([_attn(kv_heads=3)], {}, "multiple"),
    ([_delta(kv_heads=3)], {}, "multiple"),
    ([_attn(vdim=20)], {}, "vdim"),
    ([_attn(rot=_rot(26))], {}, "dims"),
    ([_attn(rot=_rot(7))], {}, "dims"),
    ([_attn(rot=dict(_rot(8), scaling={"factor": 4.0, "low": 1.0, "high": 4.0}))], {}, "original"),
    ([_attn(rot=dict(_rot(8), scaling={"factor": 4.0, "low": 4.0, "high": 4.0, "original": 64}))], {}, "high"),
    ([_latent(rot=_rot(10))], {}, "dims"),
    ([_latent(q_rank=0)], {}, "q_rank"),
    ([_delta(conv=0)], {}, "conv"),
    ([_delta(a_rank=-1)], {}, "a_rank"),
    ([_layer("latent_attention", {"heads": 2})], {}, "lacks"),
    ([_attn(mlp={"kind": "glu", "ff": 8})], {}, "kind"),
    ([_latent(kv_from=0)], {}, "kv_from"),
    ([_latent(), _latent(kv_from=1)], {}, "kv_from"),
    ([_latent(), _latent(kv_from=True)], {}, "kv_from"),
    ([_attn(), _latent(kv_from=0)], {}, "latents of its own"),
    ([_latent(), _latent(kv_from=0), _latent(kv_from=1)], {}, "latents of its own"),
    ([_latent(), _latent(kv_from=0, kv_rank=32)], {}, "kv_rank"),
    ([_latent(), _latent(kv_from=0, rot=_rot(4))], {}, "rot"),
    ([_attn()], {"norm": {}}, "eps"),
    ([_attn()], {"canon": {"taps": 0}}, "taps"),
    ([_attn()], {"streams": 0}, "streams"),
    ([], {}, "layers"),
])
def test_configurations_that_cannot_be_built_are_refused_by_name(layers, more, word):
    with pytest.raises(ConfigError, match=word):
        AutoConfig.from_dict(_cfg(layers, **more))


def _spec(cfg, shapes=None):
    from pytorch_transformers_amd.config.registry import lookup

    c = AutoConfig.from_dict(cfg)
    if shapes is not None:
        c.sizes_from_weights(lambda: shapes)
    spec = lookup(c.model_type)[1](c)
    spec.validate()
    return spec


def test_tensor_names_and_shapes():
    names = {s.name: tuple(s.shape) for s in _spec(_cfg([_latent(), _attn(), _delta(a_rank=5, g_rank=6), _latent({"kind": "dense", "ff": 16}, kv_from=0)])).tensor_specs()}
    want = {
        "embed": (50, 32), "embed.norm": (32,), "final.norm": (32,), "head": (50, 32),
        "l0.norm1": (32,), "l0.canon1": (32, 4), "l0.hc1.in": (3,), "l0.hc1.out": (3,), "l0.hc1.mix": (3, 3),
        "l0.mix.dq": (28, 32), "l0.mix.dq.norm": (28,), "l0.mix.uq": (96, 28), "l0.mix.dkv": (48, 32), "l0.mix.dkv.norm": (40,),
        "l0.mix.uk": (72, 40), "l0.mix.uv": (60, 40), "l0.mix.o": (32, 60),
        "l1.norm1": (32,), "l1.norm2": (32,), "l1.canon1": (32, 4), "l1.hc1.in": (3,), "l1.hc1.out": (3,), "l1.hc1.mix": (3, 3),
        "l1.hc2.in": (3,), "l1.hc2.out": (3,), "l1.hc2.mix": (3, 3),
        "l1.mix.q": (96, 32), "l1.mix.q.b": (96,), "l1.mix.k": (48, 32), "l1.mix.k.b": (48,), "l1.mix.sink": (4,), "l1.mix.g": (96, 32),
        "l1.mix.o": (32, 96), "l1.mlp.gate": (32, 32), "l1.mlp.up": (32, 32), "l1.mlp.down": (32, 32),
        "l2.norm1": (32,), "l2.canon1": (32, 4), "l2.hc1.in": (3,), "l2.hc1.out": (3,), "l2.hc1.mix": (3, 3),
        "l2.mix.q": (24, 32), "l2.mix.k": (24, 32), "l2.mix.v": (80, 32), "l2.mix.q.conv": (24, 3), "l2.mix.k.conv": (24, 3),
        "l2.mix.v.conv": (80, 3), "l2.mix.b": (4, 32), "l2.mix.A_log": (4,), "l2.mix.dt_bias": (48,), "l2.mix.a1": (5, 32),
        "l2.mix.a2": (48, 5), "l2.mix.g1": (6, 32), "l2.mix.g2": (80, 6), "l2.mix.norm": (20,), "l2.mix.o": (32, 80),
        "l3.norm1": (32,), "l3.norm2": (32,), "l3.canon1": (32, 4), "l3.hc1.in": (3,), "l3.hc1.out": (3,), "l3.hc1.mix": (3, 3),
        "l3.hc2.in": (3,), "l3.hc2.out": (3,), "l3.hc2.mix": (3, 3), "l3.mix.dq": (28, 32), "l3.mix.dq.norm": (28,), "l3.mix.uq": (96, 28),
        "l3.mix.uk": (72, 40), "l3.mix.uv": (60, 40), "l3.mix.o": (32, 60), "l3.mlp.gate": (16, 32), "l3.mlp.up": (16, 32), "l3.mlp.down": (32, 16),
    }
    assert names == want


def test_inner_ranks_follow_from_the_weight_file(tmp_path):
    """The sizes of the decays' and the output gate's inner vectors stand in no configuration: they are the tensors' rows.
    Layers that share one entry of the list may still differ."""
    from pytorch_transformers_amd.weights.loader import save_weights, tensor_shapes

    one = _delta()
    cfg = _cfg([one, one])
    given = {"l0.mix.a1": (9, 32), "l0.mix.g1": (4, 32), "l1.mix.a1": (3, 32), "l1.mix.g1": (11, 32)}
    save_weights(str(tmp_path), {n: torch.zeros(s) for n, s in given.items()})
    shapes = tensor_shapes(str(tmp_path))
    assert shapes == given
    names = {s.name: tuple(s.shape) for s in _spec(copy.deepcopy(cfg), shapes).tensor_specs()}
    for n, s in given.items():
        assert names[n] == s
    assert names["l0.mix.a2"] == (48, 9) and names["l1.mix.g2"] == (80, 11)
    assert {s.name: tuple(s.shape) for s in _spec(cfg).tensor_specs()}["l0.mix.a1"] == (20, 32)  # without a file: vdim


def test_cache_groups_by_what_a_layer_keeps():
    spec = _spec(_cfg([_latent(), _attn(), _latent(kv_from=0), _latent(rot_dim=6, rot=_rot(6)), _delta(), _latent(heads=7, q_rank=4), _delta(conv=2),
                       _latent(kv_from=5), _attn(kv_heads=4), _delta()]))
    kinds = [(g.kind, g.num_layers, g.kv_heads, g.head_dim, g.values, g.state_shape) for g in spec.cache_groups]
    state = lambda taps: (4 * 12 * 20 + (taps - 1) * (2 * 24 + 80),)
    assert kinds == [("state", 10, 0, 0, True, (3 * 32,)), ("full", 2, 1, 48, False, ()), ("full", 1, 2, 32, True, ()), ("full", 1, 1, 46, False, ()),
                     ("state", 2, 0, 0, True, state(3)), ("state", 1, 0, 0, True, state(2)), ("full", 1, 4, 32, True, ())]
    calls = [(c.cache_group, c.cache_layer, c.write_cache) for c in spec.order]
    assert calls[2] == (calls[0][0], calls[0][1], False) and calls[7] == (calls[5][0], calls[5][1], False) and calls[5][1] == 1
    assert all(c[2] for i, c in enumerate(calls) if i not in (2, 7))
    assert [c.also("conv") for c in spec.order] == [("canon", i) for i in range(10)]


def test_one_tap_keeps_no_inputs():
    spec = _spec(_cfg([_attn()], canon={"taps": 1}))
    assert [g.name for g in spec.cache_groups] == ["kv0"] and spec.order[0].more == ()


@pytest.mark.parametrize("rot", [_rot(16), _rot(16, True), _rot(64, True), dict(_rot(32), base=500000.0, scaling={"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}),
                                 dict(_rot(8), scaling={"factor": 3.0, "low": 0.5, "high": 40.0, "original": 100})])
def test_rotation_frequencies(rot):
    """Whole, stretched and blended frequencies against the plain formulas, to the last bit of 32-bit."""
    from pytorch_transformers_amd.engine.verelorn import _positions

    r = _positions(rot, 64, "half").rotation()
    want = torch.tensor(P.rotary_frequencies(rot), dtype=torch.float64)
    assert r.rotary_dim == rot["dims"] and r.scale == 1.0 and r.pairing == "half"
    assert torch.allclose(r.inv_freq.double(), want, rtol=1e-7, atol=0)
