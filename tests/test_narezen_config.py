"""The Narezen design's configuration, tensor names, sizes read from the weight file and cache groups (no GPU)."""
import copy

import pytest
import torch

import plain_narezen as P
from pytorch_transformers_amd.config import AutoConfig, ConfigError


def _moe(**over):
    return dict({"kind": "moe", "expert": {"ff": 12}, "router": {"experts": 3, "top": 2}, "shared": {"ff": 20}}, **over)


def _tied(left=None, right=None, mlp=None, **over):
    m = {"left": dict({"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 24, "scale": 0.2}, **(left or {})), "left_scale": 0.5,
         "right": dict({"heads": 3, "dim": 10, "vdim": 14, "tau": 8.0}, **(right or {})), "right_scale": 0.7}
    return {"type": "parallel", "mixer": dict(m, **over), "mlp": mlp}


def _kept(left=None, right=None, mlp=None, **over):
    m = {"left": dict({"heads": 4, "kv_heads": 1, "dim": 24, "vdim": 20, "scale": 0.2, "rot": {"base": 10000.0, "dims": 8}}, **(left or {})),
         "left_scale": 1.0, "right": dict({"heads": 2, "dim": 12, "vdim": 16, "rot": {"base": 500.0, "dims": 12}, "decay": [0.9, 0.99]}, **(right or {})),
         "right_scale": 1.0}
    return {"type": "parallel_2", "mixer": dict(m, **over), "mlp": mlp}


def _unit(mlp=None, **over):
    return {"type": "rglru", "mixer": dict({"width": 36, "blocks": 3, "conv": 4}, **over), "mlp": mlp}


def _cfg(layers, **more):
    return dict({"architecture": "Narezen", "vocab": 50, "width": 32, "norm": {"eps": 1e-5}, "embedding": {"scale": 7.0}, "logit_softcap": 25.0,
                 "layers": layers}, **more)


def test_the_architecture_key_chooses_the_design():
    cfg = AutoConfig.from_dict(_cfg([_tied(), _unit(_moe()), _kept()]))
    assert type(cfg).__name__ == "NarezenConfig" and cfg.model_type == "narezen" and cfg.vocab_size == 50
    assert cfg.eps == 1e-5 and cfg.softcap == 25.0
    again = AutoConfig.from_dict(cfg.to_dict())
    assert again.layers == cfg.layers and again.embedding == cfg.embedding
    assert AutoConfig.from_dict(_cfg([_unit()], logit_softcap=None)).softcap == 0.0


@pytest.mark.parametrize("layers,more,word", [
    ([dict(_tied(), type="attention")], {}, "type"),
    ([_tied({"kv_heads": 3})], {}, "multiple"),
    ([_kept({"kv_heads": 3})], {}, "multiple"),
    ([_tied({"vdim": 20})], {}, "vdim"),
    ([_tied({"dim": 0, "vdim": 0})], {}, "dim"),
    ([_tied(right={"tau": 0})], {}, "tau"),
    ([_tied(right={"a_rank": -1})], {}, "a_rank"),
    ([_tied(left_scale="1")], {}, "left_scale"),
    ([_tied(right=None, right_scale=None)], {}, "right_scale"),
    ([dict(_tied(), mixer={"left": {}, "left_scale": 1.0})], {}, "right"),
    ([_kept({"rot": {"base": 10.0, "dims": 7}})], {}, "dims"),
    ([_kept({"rot": {"base": 10.0, "dims": 26}})], {}, "dims"),
    ([_kept(right={"rot": {"base": 10.0, "dims": 14}})], {}, "dims"),
    ([_kept(right={"rot": {"dims": 2}})], {}, "base"),
    ([_kept(right={"decay": [0.9]})], {}, "decay"),
    ([_kept(right={"decay": 0.9})], {}, "decay"),
    ([_unit(blocks=5)], {}, "blocks"),
    ([_unit(conv=0)], {}, "conv"),
    ([_unit({"kind": "dense", "ff": 8})], {}, "kind"),
    ([_unit(_moe(router={"experts": 2, "top": 3}))], {}, "top"),
    ([_unit(_moe(expert=None))], {}, "ff"),
    ([_unit(_moe(shared={"ff": 0}))], {}, "ff"),
    ([_unit()], {"norm": {}}, "eps"),
    ([_unit()], {"embedding": {}}, "scale"),
    ([_unit()], {"logit_softcap": -1.0}, "softcap"),
    ([_unit()], {"width": 0}, "width"),
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


def _names(spec):
    return {n: tuple(s) for t in spec.tensor_specs() for n, s in (t.pieces or ((t.name, t.shape),))}


def test_tensor_names_and_shapes():
    layers = [_tied(right={"a_rank": 5}), _kept(mlp=_moe(router={"experts": 2, "top": 1})), _unit(_moe(router={"experts": 1, "top": 1}, shared=None))]
    want = {
        "embed": (50, 32), "final.norm": (32,), "head": (50, 32), "l0.norm1": (32,), "l0.norm1b": (32,),
        "l0.mix.left.q": (96, 32), "l0.mix.left.k": (48, 32), "l0.mix.left.sink": (4,), "l0.mix.left.o": (32, 96),
        "l0.mix.right.q": (30, 32), "l0.mix.right.k": (30, 32), "l0.mix.right.v": (42, 32), "l0.mix.right.g": (42, 32), "l0.mix.right.o": (32, 42),
        "l0.mix.right.norm": (14,), "l0.mix.right.a1": (5, 32), "l0.mix.right.a2": (30, 5), "l0.mix.right.a2.b": (30,),
        "l1.norm1": (32,), "l1.norm1b": (32,), "l1.norm2": (32,), "l1.norm2b": (32,),
        "l1.mix.left.q": (96, 32), "l1.mix.left.k": (24, 32), "l1.mix.left.v": (20, 32), "l1.mix.left.o": (32, 80),
        "l1.mix.right.q": (24, 32), "l1.mix.right.k": (24, 32), "l1.mix.right.v": (32, 32), "l1.mix.right.g": (32, 32), "l1.mix.right.o": (32, 32),
        "l1.mlp.router": (2, 32), "l1.mlp.e0.gate": (12, 32), "l1.mlp.e0.up": (12, 32), "l1.mlp.e0.down": (32, 12), "l1.mlp.e1.gate": (12, 32),
        "l1.mlp.e1.up": (12, 32), "l1.mlp.e1.down": (32, 12), "l1.mlp.shared.gate": (20, 32), "l1.mlp.shared.up": (20, 32), "l1.mlp.shared.down": (32, 20),
        "l2.norm1": (32,), "l2.norm1b": (32,), "l2.norm2": (32,), "l2.norm2b": (32,),
        "l2.mix.y": (36, 32), "l2.mix.y.b": (36,), "l2.mix.x": (36, 32), "l2.mix.x.b": (36,), "l2.mix.conv": (36, 4), "l2.mix.conv.b": (36,),
        "l2.mix.ra": (3, 12, 12), "l2.mix.ra.b": (3, 12), "l2.mix.ri": (3, 12, 12), "l2.mix.ri.b": (3, 12), "l2.mix.lam": (36,), "l2.mix.o": (32, 36),
        "l2.mlp.router": (1, 32), "l2.mlp.e0.gate": (12, 32), "l2.mlp.e0.up": (12, 32), "l2.mlp.e0.down": (32, 12),
    }
    assert _names(_spec(_cfg(layers))) == want


def test_the_decays_inner_size_follows_from_the_weight_file(tmp_path):
    """Layers that share one entry of the list may still differ; a configuration that says the size does not ask."""
    from pytorch_transformers_amd.weights.loader import save_weights, tensor_shapes

    one = _tied()
    cfg = _cfg([one, one, _unit()])
    given = {"l0.mix.right.a1": (9, 32), "l1.mix.right.a1": (3, 32)}
    save_weights(str(tmp_path), {n: torch.zeros(s) for n, s in given.items()})
    shapes = tensor_shapes(str(tmp_path))
    assert shapes == given
    names = _names(_spec(copy.deepcopy(cfg), shapes))
    assert names["l0.mix.right.a1"] == (9, 32) and names["l0.mix.right.a2"] == (30, 9) and names["l1.mix.right.a2"] == (30, 3)
    assert _names(_spec(cfg))["l0.mix.right.a1"] == (10, 32)  # without a file: dim

    def asked():
        raise AssertionError("the files were asked for")

    AutoConfig.from_dict(_cfg([_tied(right={"a_rank": 4}), _kept()])).sizes_from_weights(asked)


def test_cache_groups_by_what_a_layer_keeps():
    spec = _spec(_cfg([_tied(), _unit(), _kept(), _tied(), _kept({"kv_heads": 2}), _unit(conv=2), _unit(), _tied({"dim": 40, "vdim": 40}, {"vdim": 16, "heads": 2, "dim": 12})]))
    kinds = [(g.kind, g.num_layers, g.kv_heads, g.head_dim, g.state_shape) for g in spec.cache_groups]
    assert kinds == [("full", 3, 2, 32, ()), ("state", 2, 0, 0, (3 * 10 * 14,)), ("state", 2, 0, 0, (36 * 5,)), ("full", 1, 1, 32, ()),
                     ("state", 3, 0, 0, (2 * 12 * 16,)), ("state", 1, 0, 0, (36 * 3,)), ("full", 1, 2, 48, ())]
    calls = [(c.cache_group, c.cache_layer) for c in spec.order]
    assert calls[0][0] == calls[3][0] == calls[4][0] and [calls[i][1] for i in (0, 3, 4)] == [0, 1, 2]
    assert [spec.order[i].also("right") for i in (0, 3)] == [(spec.cache_groups[1].name, 0), (spec.cache_groups[1].name, 1)]
    assert [spec.order[i].also("right")[1] for i in (2, 4, 7)] == [0, 1, 2]
    right = spec.order[3].on("right")
    assert (right.cache_group, right.cache_layer, right.more) == (spec.cache_groups[1].name, 1, ())


@pytest.mark.parametrize("rot", [{"base": 10000.0, "dims": 16}, {"base": 1e6, "dims": 64}, {"base": 100.0, "dims": 2}])
def test_rotation_frequencies(rot):
    """The builder's rotation against the plain formula: a unit vector's pair, turned by one position, shows each frequency."""
    from pytorch_transformers_amd.engine.narezen import _positions

    r = _positions(rot, 64).rotation()
    assert r.rotary_dim == rot["dims"] and r.scale == 1.0 and r.pairing == "half"
    v = torch.zeros(64, dtype=torch.float64)
    v[: rot["dims"] // 2] = 1.0
    turned = P.rotate(v, 1, rot)
    angles = torch.atan2(turned[rot["dims"] // 2: rot["dims"]], turned[: rot["dims"] // 2])
    assert torch.allclose(r.inv_freq.double(), angles, rtol=1e-7, atol=1e-12)


def test_sizes_that_no_kernel_takes_are_refused_before_a_weight_is_read():
    for layer, word in ((_unit(conv=17), "taps"), (_kept(right={"dim": 300, "rot": None}), "256"), (_kept(right={"vdim": 300}), "256"),
                        (_kept({"vdim": 300}), "256")):
        with pytest.raises(ValueError, match=word):
            _spec(_cfg([layer])).check_sizes()
