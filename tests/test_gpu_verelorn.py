"""The Verelorn design on the GPU against the plain implementation (``plain_verelorn``): every mechanism alone, then whole
models of several shapes through the step function, the cache, captured decode steps and ``generate``.

The tests make their own small configurations and weights.  Sizes are chosen so that nothing is equal that need not be, and
a far key, a page's edge, a head's own number, one stream or one tap shows in the result instead of drowning in averages.
"""
import json
import os

import pytest
import torch

import helpers
import plain_verelorn as P
from test_gpu_bimepel import _bf16, _close, _load_part, _rand, _run_in_cuts, assert_model_close, load, write_model

pytestmark = pytest.mark.gpu

DTYPES = [("float32", 3e-5), ("bfloat16", 4e-2)]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
REL_BF16_MODEL = 0.1


# ---- configurations ---------------------------------------------------------------------------------------------
def rot(dims, base=10000.0, scaling=False):
    r = {"base": base, "dims": dims}
    if scaling:
        r["scaling"] = {"factor": 8.0, "low": 1.0, "high": 5.0, "original": 96}
    return r


def attn(heads=6, kv=2, dim=24, scale=0.3, dims=16, base=5000.0, scaling=True, ff=56):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale}
    if dims:
        m["rot"] = rot(dims, base, scaling)
    return layer("attention", m, ff)


def latent(heads=3, dim=24, rot_dim=8, vdim=20, kv_rank=40, q_rank=28, scale=0.25, base=10000.0, dims=None, kv_from=None, ff=40):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
         "rot": rot(dims or rot_dim, base)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return layer("latent_attention", m, ff)


def delta(heads=4, kv=2, dim=12, vdim=20, conv=3, a_rank=7, g_rank=10, ff=None):
    return layer("channel_delta", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv, "a_rank": a_rank,
                                   "g_rank": g_rank}, ff)


def layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, vocab=131, width=48, eps=1e-5, streams=3, taps=3):
    return {"architecture": "Verelorn", "vocab": vocab, "width": width, "streams": streams, "layers": layers, "norm": {"eps": eps},
            "canon": {"taps": taps}}


CONFIGS = {
    # every mixer with and without a feed-forward, two latent shapes, layers that read an earlier layer's latents (one of
    # them twice read, with other heads and sizes of their own), two attention shapes, two delta-rule shapes
    "mixed": config([latent(), delta(), attn(), latent(2, 16, 8, 32, 40, 12, 0.3, kv_from=0), latent(2, 8, 6, 12, 24, 16, 0.4, 300.0, ff=None),
                     attn(4, 4, 40, 0.2, 0, ff=None), delta(3, 3, 8, 36, 5, 4, 4, ff=24), latent(5, 12, 8, 8, 40, 20, 0.2, kv_from=0, ff=None),
                     latent(1, 20, 6, 16, 24, 8, 0.3, 300.0, kv_from=4)]),
    # one stream, one tap, one head, inner ranks of one: the values that make indices and states vanish
    "ones": config([latent(1, 16, 2, 16, 16, 3, 1.0, ff=16), delta(1, 1, 1, 3, 1, 1, 1), attn(1, 1, 16, 1.0, 2, ff=1)], vocab=61, width=16,
                   streams=1, taps=1),
    # attention only, heads of sizes the matrix-core kernels are built for
    "attention": config([attn(8, 2, 32, 0.18, 32), attn(4, 4, 16, 0.25, 4, 100.0, False), attn(20, 1, 64, 0.12, 64)], vocab=97, width=64,
                        streams=4, taps=4),
    # delta rule only: no layer keeps keys and values
    "delta": config([delta(4, 1, 16, 16, 4, 8, 16, 32), delta(2, 2, 40, 72, 2, 5, 3)], vocab=77, width=40, streams=2, taps=2),
    # latent attention only, all later layers reading the first one's latents
    "latent": config([latent(4, 16, 16, 16, 32, 32, 0.3), latent(2, 40, 16, 12, 32, 8, 0.2, kv_from=0), latent(8, 8, 16, 64, 32, 24, 0.25, kv_from=0)],
                     vocab=83, width=56, streams=5, taps=6),
}


def _weight(n, shape, g, std=0.12):
    """A lively random weight by its name: gains, numbers per head and links between streams that differ."""
    t = torch.randn(shape, generator=g)
    last = n.rsplit(".", 1)[-1]
    if last in ("norm1", "norm2") or n in ("embed.norm", "final.norm"):
        return 0.3 * t  # (stored around zero)
    if last == "norm" or n.endswith(("dq.norm", "dkv.norm")):
        return 1.0 + 0.3 * t
    if last == "mix" and len(shape) == 2 and shape[0] == shape[1] and ".hc" in n:
        return 0.8 * torch.eye(shape[0]) + 0.15 * t
    if ".hc" in n:
        return 0.8 + 0.25 * t  # (links of one sign: streams that all but cancel would magnify every rounding)
    if last == "canon1" or last == "conv":
        return 0.3 * t
    if last == "sink":
        return 1.0 + t
    if last in ("A_log", "dt_bias"):
        return t - 1.0
    if n == "embed":
        return t
    if len(shape) == 1:
        return 0.4 * t
    return t * std * (48.0 / shape[-1]) ** 0.5


def make_weights(cfg, seed):
    """Random weights by the design's tensor names, rounded to bfloat16 (so that both compute types hold the same
    numbers), as float64."""
    from pytorch_transformers_amd.config import AutoConfig
    from pytorch_transformers_amd.config.registry import lookup

    c = AutoConfig.from_dict(cfg)
    g = torch.Generator().manual_seed(seed)
    return {s.name: _bf16(_weight(s.name, s.shape, g)) for s in lookup(c.model_type)[1](c).tensor_specs()}


def file_config(cfg):
    """The configuration as a file has it: the inner ranks of the delta rule follow from the tensors."""
    cfg = json.loads(json.dumps(cfg))
    for l in cfg["layers"]:
        l["mixer"].pop("a_rank", None)
        l["mixer"].pop("g_rank", None)
    return cfg


def save(folder, cfg, w):
    return write_model(folder, file_config(cfg), w)


def plain_all(cfg, w, reqs):
    return {rid: P.run_tokens(w, cfg, toks).float() for rid, toks in reqs.items()}


def _part_weights(part, seed, std=0.25):
    g = torch.Generator().manual_seed(seed)
    return {s.name: _bf16(_weight(s.name, s.shape, g, std)) for s in part.all_tensor_specs()}


# ---- the streams ---------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,rel", [("float32", 3e-6), ("bfloat16", 5e-3)])
@pytest.mark.parametrize("streams,width", [(1, 16), (2, 50), (3, 48), (4, 200), (5, 7), (6, 1100), (7, 64), (8, 4100)])
def test_streams_take_a_result_in_and_are_normed(dtype, rel, streams, width):
    """New streams, their weighted and plain sums and the norm; from equal streams (one vector) and unequal ones; with and
    without a result to take in; all tokens and chosen ones."""
    from pytorch_transformers_amd import ops

    dt, M, eps = TORCH[dtype], 7, 1e-4
    mix, into, out = _rand(streams, streams, seed=1), _rand(streams, seed=2), _rand(streams, seed=3)
    w = _rand(width, seed=4, scale=0.3)
    rows = torch.tensor([5, 0, 5], dtype=torch.int32)
    f = lambda t: t.float().cuda()
    for equal in (False, True):
        xs = _rand(M, width, seed=5, scale=2.0) if equal else _rand(M, streams, width, seed=5, scale=2.0)
        full = xs[:, None].expand(M, streams, width) if equal else xs
        for with_y in (False, True):
            y = _bf16(_rand(M, width, seed=6))
            new = torch.stack([P.hyper_update(full[m].double(), mix.double(), out.double(), y[m]) for m in range(M)]) if with_y else full.double()
            u = torch.stack([P.hyper_input(new[m], into.double()) for m in range(M)])
            kw = dict(y=y.to(dt).cuda(), mix=f(mix), out=f(out)) if with_y else {}
            h, n, uu, x2 = ops.hyper_norm(f(xs), streams, dt, weights=f(into), norm=(f(w), 1.0, eps), want_x=with_y, want_u=True,
                                          want_n=True, want_h=True, **kw)
            want = P.model_norm(u, w.double(), eps)
            _close(uu, u, 3e-6, "weighted sum")
            _close(n, want, 5e-6, "norm in 32-bit")
            _close(h, want, rel + 3e-6, "norm")
            assert h.dtype == dt and (x2 is None) == (not with_y)
            if with_y:
                _close(x2, new, 3e-6, "streams")
            h = ops.hyper_norm(f(xs), streams, dt, norm=(f(w), 1.0, eps), rows=rows.cuda(), want_h=True, **kw)[0]
            _close(h, P.model_norm(new.sum(1), w.double(), eps)[rows.long()], rel + 5e-6, "norm of the plain sum, chosen rows")


class _Echo:
    """A mixer that hands back what it reads."""

    def children(self):
        return ()

    def all_tensor_specs(self):
        return []

    def load_all(self, tensors):
        pass

    def forward(self, x, ctx, call, residual=None):
        return x.clone()


@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("streams,width,taps,ff", [(3, 24, 3, 40), (1, 16, 1, 0), (4, 50, 2, 24), (2, 264, 6, 0), (5, 40, 16, 8)])
def test_block_alone(dtype, rel, streams, width, taps, ff):
    """Streams, norms and the input convolution of a block around a mixer that echoes, in cuts down to one and two tokens,
    four sequences a step, on slots that were given back."""
    from pytorch_transformers_amd.engine.spec import CACHE_STATE, CacheGroupSpec, LayerCall
    from pytorch_transformers_amd.parts import GatedFeedForward, HyperBlock, RMSNorm

    dt, eps = TORCH[dtype], 1e-5
    ffn = GatedFeedForward("b.mlp", width, ff, "gelu_tanh") if ff else None
    block = HyperBlock("b", _Echo(), ffn, RMSNorm("b.norm1", width, eps, offset=1.0), RMSNorm("b.norm2", width, eps, offset=1.0) if ff else None,
                       streams, width, taps, "b.canon1")
    w = _part_weights(block, seed=streams * 10 + taps)
    _load_part(block, w, dt)
    groups = [CacheGroupSpec("canon", CACHE_STATE, 2, state_shape=(max(block.conv_state, 1),))]
    call = LayerCall(0, more=(("conv", "canon", 1),))
    cuts = [[80], [1] * 7 + [2, 71], [30, 2, 2, 46], [63, 1, 1, 15]]
    xs = [_bf16(_rand(80, width, seed=50 + i)) for i in range(4)]
    outs = _run_in_cuts(lambda x, ctx: block.forward(x, ctx, call).wide, groups, dt, xs, cuts, free_and_again=True)
    for i, x in enumerate(xs):
        kept, want = [], []
        for t in range(80):
            s = torch.stack([x[t]] * streams)
            h = P.model_norm(P.hyper_input(s, w["b.hc1.in"]), w["b.norm1"], eps)
            h = h + P.causal_conv(kept, h, w["b.canon1"])
            s = P.hyper_update(s, w["b.hc1.mix"], w["b.hc1.out"], h)
            if ff:
                h = P.model_norm(P.hyper_input(s, w["b.hc2.in"]), w["b.norm2"], eps)
                s = P.hyper_update(s, w["b.hc2.mix"], w["b.hc2.out"], P.dense_ff(w, "b.mlp", h))
            want.append(s.sum(0))
        _close(outs[i], torch.stack(want), rel, f"{streams} streams, {taps} taps, sequence {i}")


@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("ff,hidden,rows", [(56, 40, 7), (1, 8, 3), (300, 24, 40), (2048, 64, 300), (12, 8, 1)])
def test_feed_forward_with_a_tanh_gelu_gate(dtype, rel, ff, hidden, rows):
    from pytorch_transformers_amd.parts import GatedFeedForward

    dt = TORCH[dtype]
    part = GatedFeedForward("f", hidden, ff, "gelu_tanh")
    w = _part_weights(part, seed=ff)
    _load_part(part, w, dt)
    x = _bf16(_rand(rows, hidden, seed=1, scale=1.5))
    got = part.forward(x.to(dt).cuda(), None)
    _close(got, torch.stack([P.dense_ff(w, "f", x[i]) for i in range(rows)]), rel, f"feed-forward {ff}x{hidden}")


@pytest.mark.parametrize("dtype,rel", [("float32", 3e-6), ("bfloat16", 6e-3)])
def test_the_gate_over_its_whole_range(dtype, rel):
    """Both tails of the gate, where its exponential overflows and vanishes."""
    from pytorch_transformers_amd import ops

    z = _bf16(torch.cat([torch.linspace(-40, 40, 792), torch.tensor([0.0, -0.0, 300.0, -300.0, 1e4, -1e4, 1e-6, -1e-6])])).view(1, -1)
    both = torch.cat([z, torch.ones_like(z)], dim=1).to(TORCH[dtype]).cuda()
    got = ops.glu(both[:, :800], both[:, 800:], "gelu_tanh")
    want = P.gelu_tanh(z)
    assert torch.isfinite(got).all()
    err = (got.double().cpu() - want).abs()
    assert bool((err <= rel * want.abs() + 1e-6).all()), float(err.max())


@pytest.mark.parametrize("dtype,rel", [("float32", 3e-6), ("bfloat16", 3e-6)])
def test_the_embedding_is_normed_in_32_bit(dtype, rel):
    from pytorch_transformers_amd.parts import Embedding, RMSNorm

    dt = TORCH[dtype]
    part = Embedding("embed", 23, 56, weight_name="embed", norm=RMSNorm("embed.norm", 56, 1e-3, offset=1.0))
    w = _part_weights(part, seed=2)
    _load_part(part, w, dt)
    ids = torch.tensor([3, 22, 0, 3], dtype=torch.int32)
    got = part.forward(ids.cuda())
    assert got.dtype == torch.float32
    _close(got, P.model_norm(w["embed"][ids.long()], w["embed.norm"], 1e-3), rel, "normed embedding")


# ---- the mixers alone -----------------------------------------------------------------------------------------------------
def _mixer(m, kind, hidden, name="a", eps=1e-5):
    from pytorch_transformers_amd.engine.verelorn import _positions
    from pytorch_transformers_amd.parts import ChannelDeltaMixer, GatedAttentionMixer, LatentAttentionMixer

    if kind == "attention":
        return GatedAttentionMixer(name, hidden, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], eps,
                                   _positions(m.get("rot"), m["dim"], "half"), qk_norm=False, v_norm=False, gate=True, bias="qk",
                                   v_from_k=True, sink=True)
    if kind == "channel_delta":
        return ChannelDeltaMixer(name, hidden, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], m["a_rank"], m["g_rank"], eps)
    return LatentAttentionMixer(name, hidden, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["scale"], eps,
                                _positions(m.get("rot"), m["rot_dim"], "interleaved"), q_rank=m["q_rank"],
                                reads_other=m.get("kv_from") is not None)


def _group(mixer):
    from pytorch_transformers_amd.engine.spec import CACHE_FULL, CACHE_STATE, CacheGroupSpec

    if hasattr(mixer, "state_shape"):
        return CacheGroupSpec("kv", CACHE_STATE, 1, state_shape=mixer.state_shape)
    if hasattr(mixer, "cache_row"):
        return CacheGroupSpec("kv", CACHE_FULL, 1, 1, mixer.cache_row, values=False)
    return CacheGroupSpec("kv", CACHE_FULL, 1, mixer.kv_heads, mixer.frame)


def _plain_mixer(kind, w, m, x, eps=1e-5):
    kept, out = {}, []
    for pos in range(x.shape[0]):
        if kind == "attention":
            out.append(P.attention_token(w, "a", m, x[pos], kept, pos))
        elif kind == "channel_delta":
            out.append(P.channel_delta_token(w, "a", m, eps, x[pos], kept))
        else:
            out.append(P.latent_attention_token(w, "a", m, eps, x[pos], kept, pos))
    return torch.stack(out)


SHAPES = [attn(), attn(4, 1, 16, 0.2, 8, 100.0, False), attn(2, 2, 40, 0.15, 0), attn(5, 5, 8, 0.5, 8), attn(3, 1, 130, 0.1, 72),
          attn(20, 4, 16, 0.3, 2), attn(8, 2, 64, 0.2, 32), attn(1, 1, 24, 0.3, 24), attn(64, 1, 64, 0.15, 64), attn(3, 3, 200, 0.08, 16),
          latent(), latent(2, 16, 16, 32, 24, 56, 0.2, 300.0), latent(1, 16, 2, 16, 16, 16, 0.5), latent(5, 8, 4, 72, 130, 9, 0.3, dims=2),
          latent(16, 32, 32, 16, 64, 32, 0.15),
          delta(), delta(1, 1, 1, 3, 1, 1, 1), delta(6, 2, 33, 70, 4, 16, 8), delta(2, 1, 128, 128, 4, 24, 24), delta(3, 3, 16, 100, 2, 3, 5),
          delta(8, 8, 64, 16, 5, 8, 8), delta(2, 2, 200, 40, 16, 8, 40)]


@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("shape", SHAPES, ids=lambda s: s["type"][:3] + "-".join(str(v) for v in s["mixer"].values() if isinstance(v, int)))
def test_mixer_alone(dtype, rel, shape):
    """Whole, token by token, in portions down to two tokens and across page borders, four sequences a step, and once
    more on slots and pages that were given back."""
    from pytorch_transformers_amd.engine.spec import LayerCall

    m, hidden, dt = shape["mixer"], 32, TORCH[dtype]
    mixer = _mixer(m, shape["type"], hidden)
    w = _part_weights(mixer, seed=5)
    _load_part(mixer, w, dt)
    call = LayerCall(0, "kv", 0)
    cuts = [[150], [64, 1, 1, 62, 2, 20], [1] * 20 + [130], [63, 2, 85]]
    xs = [_bf16(_rand(150, hidden, seed=40 + i)) for i in range(4)]
    outs = _run_in_cuts(lambda x, ctx: mixer.forward(x, ctx, call), [_group(mixer)], dt, xs, cuts, free_and_again=True)
    for i in range(4):
        _close(outs[i], _plain_mixer(shape["type"], w, m, xs[i]), rel, f"{shape['type']} {m} sequence {i}")


@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("shape", [delta(), delta(6, 2, 33, 70, 4, 16, 8), delta(2, 1, 128, 128, 4, 24, 24), delta(1, 1, 16, 16, 2, 4, 4),
                                   delta(2, 2, 48, 24, 3, 8, 8), delta(1, 1, 160, 72, 4, 8, 8)],
                         ids=lambda s: "-".join(str(v) for v in s["mixer"].values()))
def test_delta_rule_over_prompts_cut_into_chunks(dtype, rel, shape):
    """Sequences long enough that the recurrence runs in chunks side by side, beside shorter ones and single tokens, with a
    state from before: the same as token by token.  Chunks end at 128 tokens: lengths just at, before and past them."""
    from pytorch_transformers_amd.engine.spec import LayerCall

    m, hidden, dt = shape["mixer"], 24, TORCH[dtype]
    mixer = _mixer(m, "channel_delta", hidden)
    w = _part_weights(mixer, seed=7)
    w["a.A_log"] = w["a.A_log"] - 3.0  # slow decays: what a chunk starts from reaches far into the next ones
    _load_part(mixer, w, dt)
    call = LayerCall(0, "kv", 0)
    cuts = [[700], [2, 257, 1, 440], [384, 1, 315], [1, 300, 399]]
    xs = [_bf16(_rand(700, hidden, seed=60 + i)) for i in range(4)]
    outs = _run_in_cuts(lambda x, ctx: mixer.forward(x, ctx, call), [_group(mixer)], dt, xs, cuts, free_and_again=True)
    for i in range(4):
        _close(outs[i], _plain_mixer("channel_delta", w, m, xs[i]), rel, f"{m} sequence {i}")


def test_the_delta_rule_overwrites_what_a_key_held():
    """A key that comes again: the second value replaces the first (read out alone), where a plain sum of outer products
    would hold both; and a channel with a fast decay forgets while the others keep."""
    from pytorch_transformers_amd import ops
    from pytorch_transformers_amd.cache.paged import PagedCache
    from pytorch_transformers_amd.engine.spec import CACHE_STATE, CacheGroupSpec
    from test_gpu_bimepel import _ctx

    N, V = 4, 3
    k = torch.zeros(5, N)
    k[0, 0] = k[1, 1] = k[2, 0] = k[3, 2] = k[4, 3] = 1.0
    q = torch.zeros(5, N)
    q[:, 0] = 1.0
    q[4, 0], q[4, 1] = 0.0, 1.0
    v = torch.arange(15.0).view(5, V) + 1
    g = torch.ones(5, N)
    g[3, 1] = 0.25  # the second key's channel, from the fourth token on
    qkv = torch.cat([q, k, v], dim=1)
    cache = PagedCache([CacheGroupSpec("s", CACHE_STATE, 1, state_shape=(N * V,))], 256, torch.float32, "cuda:0", max_slots=2)
    ctx, _ = _ctx(cache, [cache.alloc()], [5], torch.float32)
    o = ops.delta_scan(qkv.cuda(), g.cuda(), torch.ones(5, 1).cuda(), cache.state_layer("s", 0), ctx, 1, 1, N, V).cpu()
    want = torch.stack([v[0], v[0], v[2], v[2], 0.25 * v[1]])
    assert torch.allclose(o, want), o


@pytest.mark.parametrize("dtype,rel", DTYPES)
def test_layers_that_read_anothers_latents(dtype, rel):
    """Two layers with heads and sizes of their own over the rows a first layer wrote, in the step and from before."""
    from pytorch_transformers_amd.engine.spec import LayerCall

    hidden, dt, eps = 32, TORCH[dtype], 1e-5
    shapes = [latent(3, 24, 8, 20, 40, 28)["mixer"], latent(2, 8, 8, 12, 40, 12, 0.4, kv_from=0)["mixer"], latent(7, 16, 8, 8, 40, 5, 0.3, kv_from=0)["mixer"]]
    parts, w = [], {}
    for i, m in enumerate(shapes):
        part = _mixer(m, "latent_attention", hidden, name=f"a{i}")
        mine = _part_weights(part, seed=20 + i)
        assert (f"a{i}.dkv" in mine) == (i == 0) and (f"a{i}.dkv.norm" in mine) == (i == 0)
        _load_part(part, mine, dt)
        parts.append(part)
        w.update(mine)

    def step(x, ctx):
        ys = [p.forward(x, ctx, LayerCall(0, "kv", 0, write_cache=i == 0)) for i, p in enumerate(parts)]
        return torch.cat(ys, dim=1)

    xs = [_bf16(_rand(140, hidden, seed=70 + i)) for i in range(3)]
    outs = _run_in_cuts(step, [_group(parts[0])], dt, xs, [[140], [64, 1, 1, 62, 2, 10], [1] * 10 + [130]], free_and_again=True)
    for x, got in zip(xs, outs):
        kept, want = {}, []
        for pos in range(140):
            want.append(torch.cat([P.latent_attention_token(w, f"a{i}", m, eps, x[pos], kept, pos) for i, m in enumerate(shapes)]))
        want = torch.stack(want)
        for i in range(3):
            _close(got[:, i * hidden:(i + 1) * hidden], want[:, i * hidden:(i + 1) * hidden], rel, f"layer {i}")


# ---- the number that joins the weights' sum --------------------------------------------------------------------------------
def _pools(nkv, d, n_pages, seed, dt):
    k, v = _bf16(_rand(n_pages, nkv, 64, d, seed=seed)), _bf16(_rand(n_pages, nkv, d, 64, seed=seed + 1))
    return k, v, k.to(dt).cuda(), v.to(dt).cuda()


def _plain_attention(q, k, v, sink, scale, start):
    """q [new, nh, d] at positions start .. ; k [nkv, n, d], v [nkv, n, d]: softmax with e^sink in the sum."""
    new, nh, d = q.shape
    out = torch.zeros(new, nh, d, dtype=torch.float64)
    per = nh // k.shape[0]
    for t in range(new):
        for h in range(nh):
            s = k[h // per, :start + t + 1] @ q[t, h] * scale
            top = max(float(s.max()), float(sink[h]))
            e = torch.exp(s - top)
            out[t, h] = e @ v[h // per, :start + t + 1] / (e.sum() + torch.exp(sink[h] - top))
    return out


@pytest.mark.parametrize("nh,nkv,d", [(6, 2, 16), (8, 1, 64), (4, 4, 128), (64, 1, 64), (2, 1, 256), (40, 2, 32)])
@pytest.mark.parametrize("level", [-30.0, 0.0, 3.0, 60.0])
def test_sinks_in_every_attention_launch(nh, nkv, d, level):
    """Prompts (both workgroup shapes) and decode steps with one range of keys, several, waves that divide a range, and heads
    that share keys through LDS, against the plain softmax with a sink; sinks far below, among and far above the scores."""
    from pytorch_transformers_amd import ops

    sink = level + _rand(nh, seed=3).double()
    scale, lens = d ** -0.5, [200, 70]
    k, v, kp, vp = _pools(nkv, d, 8, 11, torch.bfloat16)
    table = torch.tensor([[3, 0, 5, 1], [7, 2, 0, 0]], dtype=torch.int32)
    row = lambda pool, s, axis: torch.cat([pool[int(p)].movedim(axis, 1) for p in table[s][:(lens[s] + 63) // 64]], dim=1)[:, :lens[s]]
    f = lambda t: t.float().cuda()
    i32 = lambda t: torch.tensor(t, dtype=torch.int32).cuda()
    for new in ([1, 1], [40, 70]):
        q = _bf16(_rand(sum(new), nh, d, seed=13))
        cu, start = [0, new[0], sum(new)], [n - m for n, m in zip(lens, new)]
        want = torch.cat([_plain_attention(q[cu[s]:cu[s + 1]], row(k, s, 1), row(v, s, 2), sink, scale, start[s]) for s in (0, 1)]).view(sum(new), -1)
        args = (q.to(torch.bfloat16).cuda(), kp, vp, table.cuda(), i32(cu), i32(start), None, scale)
        if new[0] == 1:
            ways = [dict(n_splits=1, split_size=256), dict(n_splits=2, split_size=128), dict(n_splits=4, split_size=64)]
            ways += [dict(n_splits=n, split_size=256 // n, decode_tiles=1, decode_waves=4) for n in (1, 2)
                     if ops.load_library().pta_attn_decode_waves_ok(d, 1, 4)]
            if ops.attn_decode_shared_ok(d, nh // nkv):
                ways += [dict(n_splits=n, split_size=256 // n, decode_waves=ops.SHARED_KEYS) for n in (1, 2)]
        else:
            ways = [dict(prompt_wide=False)] + ([dict(prompt_wide=True)] if d <= 64 else [])
        for how in ways:
            got = ops.attn_mfma(*args, max_new=max(new), sink=f(sink), **how)
            # (results far below a loud sink vanish: measured against the values' own size then)
            err = float((got.double().cpu() - want).abs().max())
            assert err <= 0.02 * max(float(want.abs().max()), 1e-3), f"{nh} heads of {d}, new {new}, {how}: {err}"
        seq = torch.tensor([0] * new[0] + [1] * new[1], dtype=torch.int32).cuda()
        pos = torch.tensor([start[s] + t for s in (0, 1) for t in range(new[s])], dtype=torch.int32).cuda()
        got = ops.attn_generic(f(q), f(k), f(v), table.cuda(), seq, pos, None, scale, sink=f(sink))
        err = float((got.double().cpu() - want).abs().max())
        assert err <= 3e-6 * max(float(want.abs().max()), 1e-3), f"32-bit kernel, new {new}: {err}"


def test_a_heads_own_sink_is_that_heads():
    """Two heads equal in everything but their sinks; swapping the sinks swaps their outputs, and the sink is not scaled."""
    from pytorch_transformers_amd.engine.spec import LayerCall

    m, hidden, dt = attn(2, 1, 16, 0.05, 8)["mixer"], 32, torch.float32
    outs = []
    for sinks in ([-6.0, 2.5], [2.5, -6.0]):
        mixer = _mixer(m, "attention", hidden)
        w = _part_weights(mixer, seed=9)
        for n in ("a.q", "a.q.b", "a.g"):
            w[n][16:] = w[n][:16]
        w["a.sink"] = _bf16(torch.tensor(sinks))
        _load_part(mixer, w, dt)
        x = _bf16(_rand(40, hidden, seed=1))
        got = _run_in_cuts(lambda t, ctx: mixer.forward(t, ctx, LayerCall(0, "kv", 0)), [_group(mixer)], dt, [x], [[30] + [1] * 10])[0]
        _close(got, _plain_mixer("attention", w, m, x), 3e-5, "two heads with sinks of their own")
        outs.append((got.double() @ torch.linalg.pinv(w["a.o"]).T).view(40, 2, 16))  # undo W_o: the heads side by side
    tol = 1e-4 * float(outs[0].abs().max())
    assert float((outs[0][:, 0] - outs[1][:, 1]).abs().max()) < tol
    assert float((outs[0][:, 0] - outs[0][:, 1]).abs().max()) > 100 * tol


# ---- far keys --------------------------------------------------------------------------------------------------------------
def _loud_weights(kind, mixer, m, hidden):
    """Weights under which a token whose first half of the input repeats an earlier token's gives that token's key a
    score that stands out."""
    w = _part_weights(mixer, seed=6, std=0.3)
    half = hidden // 2
    if kind == "attention":
        d = m["dim"]
        # half of a head's key reads the first half of the input and makes the score, the other half reads the rest
        w["a.k"][:d // 2, half:] = 0
        w["a.k"][d // 2:, :half] = 0
        q = w["a.k"].clone()
        q[d // 2:] = 0
        w["a.q"] = q.repeat(m["heads"], 1)
        for n in ("a.q.b", "a.k.b"):
            w[n] = torch.zeros_like(w[n])
        w["a.sink"] = torch.full((m["heads"],), 2.0, dtype=torch.float64)
    else:
        R, d, dr, H = m["kv_rank"], m["dim"], m["rot_dim"], m["heads"]
        w["a.dkv"][:R // 2, half:] = 0
        w["a.dkv"][R // 2:R, :half] = 0
        w["a.dkv"][R:] = 0
        w["a.dq"] = w["a.dkv"][:R].clone()
        w["a.dq"][R // 2:] = 0
        w["a.dq.norm"] = w["a.dkv.norm"] = torch.ones(R, dtype=torch.float64)
        w["a.uk"][:, R // 2:] = 0
        w["a.uv"][:, :R // 2] = 0
        uq = torch.zeros(H, d + dr, R, dtype=torch.float64)
        uq[:, :d] = w["a.uk"].view(H, d, R)
        w["a.uq"] = uq.view(H * (d + dr), R)
    return w


@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
@pytest.mark.parametrize("query,key", [(500, 0), (500, 1), (500, 63), (500, 64), (500, 137), (200, 199), (200, 201), (191, 127),
                                       (192, 128), (64, 63), (64, 65), (63, 0), (9, 8), (2, 0), (1, 0), (300, 302)])
def test_one_loud_key_is_seen_from_wherever_it_lies_behind(dtype, rel, kind, query, key):
    """One key far back among hundreds, at a page's first and last place, among a sequence's first tokens, right behind
    the query, and ahead of it (where it must not be seen): fed whole and with the query decoded alone.  The plain side
    checks that the loud key shows exactly where it is visible."""
    from pytorch_transformers_amd.engine.spec import LayerCall

    hidden, dt = 32, TORCH[dtype]
    shape = attn(2, 1, 24, 0.9, 0) if kind == "attention" else latent(2, 24, 8, 20, 32, 32, 0.6)
    m = shape["mixer"]
    mixer = _mixer(m, kind, hidden)
    w = _loud_weights(kind, mixer, m, hidden)
    n = max(query, key) + 2
    x = _bf16(_rand(n, hidden, seed=7))
    if kind == "attention":
        x[:, :16] = _bf16(0.3 * x[:, :16])
    _load_part(mixer, w, dt)
    loud = _bf16(_rand(16, seed=8) * 3.0)
    x[key, :16] = loud
    if kind == "attention":
        x[key, 16:] = _bf16(_rand(16, seed=9) * 6.0)
    x[query, :16] = loud
    want = _plain_mixer(kind, w, m, x)
    quiet = x.clone()
    quiet[key] = x[next(i for i in range(n) if i not in (key, query))]
    moved = float((_plain_mixer(kind, w, m, quiet)[query] - want[query]).abs().max()) > 0.1 * float(want[query].abs().max())
    assert moved == (key < query), "the test's loud key does not show where it should"
    call = LayerCall(0, "kv", 0)
    first = min(key, query)
    for cuts in ([n], [query, 1, n - query - 1], [first + 1, query - first - 1, 1, n - query - 1] if query - first > 1 else [1] * n):
        got = _run_in_cuts(lambda t, ctx: mixer.forward(t, ctx, call), [_group(mixer)], dt, [x], [[c for c in cuts if c]])[0]
        _close(got, want, rel, f"{kind}: query {query}, loud key {key}, cuts {cuts}")
        _close(got[query], want[query], 2 * rel, f"{kind}: query {query} alone")


# ---- whole models ------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,rel", [("float32", helpers.REL_F32), ("bfloat16", REL_BF16_MODEL)])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_schedules_give_the_plain_logits(tmp_path, name, dtype, rel):
    """Whole prompts, prompt then token by token, unequal batches decoded together, requests that join and leave with
    prompts in portions down to one token: all the plain logits, with slots and pages freed and used again."""
    from pytorch_transformers_amd.engine.replay import Replayer

    cfg = CONFIGS[name]
    w = make_weights(cfg, seed=11)
    model = load(save(tmp_path / name, cfg, w), dtype)
    reqs = helpers.make_requests(cfg["vocab"], [9, 70, 131, 1, 64, 65, 2, 300], seed=3)
    want = plain_all(cfg, w, reqs)
    rp = Replayer(model, 1024, max_slots=8)
    for label, records in (("whole", helpers.schedule_whole(reqs)), ("tail", helpers.schedule_tail(reqs, 40)),
                           ("batches", helpers.schedule_batches(reqs, 3)),
                           ("staggered", helpers.schedule_staggered(reqs, chunks=(None, 2, 19, 1))),
                           ("batches again", helpers.schedule_batches(reqs, 4, decode=(1, 30, 2, 5)))):
        got = helpers.run_schedule(rp, records)
        for rid in reqs:
            assert_model_close(got[rid], want[rid], rel, f"{name} {dtype} {label} {rid}")
        assert not rp.cache.live_slots()


def test_the_streams_sum_after_every_layer(tmp_path):
    """The sum of the 32-bit streams after every layer, last token of a prompt, against the plain model's."""
    cfg = CONFIGS["mixed"]
    w = make_weights(cfg, seed=17)
    model = load(save(tmp_path / "m", cfg, w), "float32")
    toks = helpers.make_requests(cfg["vocab"], [75], seed=2)["r0"]
    seen = {}
    model.layer_hook = lambda i, x: seen.__setitem__(i, x[-1].double().cpu())
    cache = model.new_cache(256)
    model.step(cache, [cache.alloc()], [toks], "last")
    seq, streams = P.Sequence(cfg), []
    for t in toks:
        streams = []
        P.step_token(w, cfg, seq, t, streams)
    assert len(seen) == len(streams) == len(cfg["layers"])
    for i, want in enumerate(streams):
        _close(seen[i], want, 2e-5, f"streams after layer {i}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_decode_steps_equal_direct_ones(tmp_path, dtype):
    """Decode steps replayed from a captured graph give the bits of the same steps launched one by one, with batches
    that are padded to the captured size."""
    from pytorch_transformers_amd.engine.replay import Replayer

    cfg = CONFIGS["mixed"]
    folder = save(tmp_path / "m", cfg, make_weights(cfg, seed=12))
    reqs = helpers.make_requests(cfg["vocab"], [9, 30, 70, 3, 41, 12, 25, 8, 19, 33, 50], seed=4)
    records = helpers.schedule_batches(reqs, 3, decode=(5, 2, 8)) + \
        [dict(r, step=r["step"] + 1000) for r in helpers.schedule_batches(reqs, 11, decode=(2, 9, 4))]
    outs = {}
    for graphs in (False, True):
        model = load(folder, dtype)
        assert model.use_graphs
        model.use_graphs = graphs
        rp = Replayer(model, 2048, max_slots=16)
        outs[graphs] = [rp.run(rec) for rec in records]
        torch.cuda.synchronize()
    for rec, a, b in zip(records, outs[False], outs[True]):
        assert (a is None) == (b is None)
        if a is not None:
            assert torch.equal(a, b), f"step {rec['step']}: a captured step differs from the same step launched directly"


@pytest.mark.parametrize("dtype,rel", [("float32", helpers.REL_F32), ("bfloat16", REL_BF16_MODEL)])
def test_long_decoding_and_a_loud_far_token(tmp_path, dtype, rel):
    """300 tokens decoded one by one after a short prompt, with a token near the start whose embedding points its own way:
    every layer keeps seeing it over hundreds of steps and several pages."""
    from pytorch_transformers_amd.engine.replay import Replayer

    cfg = CONFIGS["mixed"]
    w = make_weights(cfg, seed=13)
    w["embed"][7, :4] = _bf16(w["embed"][7, :4] * 8.0)
    model = load(save(tmp_path / "m", cfg, w), dtype)
    toks = [t if t != 7 else 8 for t in helpers.make_requests(cfg["vocab"], [330], seed=5)["r0"]]
    toks[2] = 7
    reqs = {"long": toks}
    want = plain_all(cfg, w, reqs)
    got = helpers.run_schedule(Replayer(model, 1024, max_slots=2), helpers.schedule_tail(reqs, 300))
    assert_model_close(got["long"], want["long"], rel, f"long decoding {dtype}")


def test_a_longer_prompt_through_all_mixers(tmp_path):
    """A prompt of several hundred tokens (the recurrence in chunks, a dozen pages) beside a short one, then decoded."""
    from pytorch_transformers_amd.engine.replay import Replayer

    cfg = CONFIGS["mixed"]
    w = make_weights(cfg, seed=18)
    folder = save(tmp_path / "m", cfg, w)
    reqs = helpers.make_requests(cfg["vocab"], [640, 33], seed=8)
    want = plain_all(cfg, w, reqs)
    for dtype, rel in (("float32", helpers.REL_F32), ("bfloat16", REL_BF16_MODEL)):
        got = helpers.run_schedule(Replayer(load(folder, dtype), 1024, max_slots=2), helpers.schedule_batches(reqs, 2, decode=(12, 5)))
        for rid in reqs:
            assert_model_close(got[rid], want[rid], rel, f"{dtype} {rid}")


def test_greedy_generation_follows_the_plain_model(tmp_path):
    cfg = CONFIGS["mixed"]
    w = make_weights(cfg, seed=14)
    model = load(save(tmp_path / "m", cfg, w), "float32")
    reqs = helpers.make_requests(cfg["vocab"], [5, 17, 2], seed=6)
    out = model.generate(list(reqs.values()), max_new_tokens=12, do_sample=False, eos_token_id=None)
    for seq, toks in zip(out, reqs.values()):
        assert list(seq) == list(toks) + P.greedy(w, cfg, list(toks), 12)


def test_random_weights_from_a_configuration_run(tmp_path):
    """The framework's own random-weights mode writes the design's tensor names, and what it writes loads and steps."""
    from safetensors import safe_open

    from pytorch_transformers_amd import AutoModelForCausalLM
    from pytorch_transformers_amd.config import AutoConfig
    from pytorch_transformers_amd.weights import write_random_model

    cfg = AutoConfig.from_dict(file_config(CONFIGS["mixed"]))
    folder = write_random_model(str(tmp_path / "r"), cfg, seed=1, std=0.1)
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as f:
        names = set(f.keys())
    assert {"embed", "embed.norm", "final.norm", "head", "l0.mix.dq", "l0.mix.dq.norm", "l0.mix.uq", "l0.mix.dkv", "l0.mix.dkv.norm",
            "l0.mix.uk", "l0.mix.uv", "l0.mix.o", "l0.mlp.gate", "l0.mlp.up", "l0.mlp.down", "l0.hc1.in", "l0.hc2.mix", "l0.canon1",
            "l1.mix.q.conv", "l1.mix.b", "l1.mix.A_log", "l1.mix.dt_bias", "l1.mix.a1", "l1.mix.a2", "l1.mix.g1", "l1.mix.g2",
            "l1.mix.norm", "l2.mix.q.b", "l2.mix.k.b", "l2.mix.sink", "l2.mix.g", "l3.mix.uk"} <= names
    assert not any(n.startswith(("l1.mlp", "l1.hc2", "l1.norm2", "l2.mix.v", "l3.mix.dkv")) or n.endswith((".weight", ".bias", "o.b")) for n in names)
    for dtype in ("bfloat16", "float32"):
        model = AutoModelForCausalLM.from_pretrained(folder, dtype=dtype)
        cache = model.new_cache(256)
        logits = model.step(cache, [cache.alloc()], [[1, 2, 3]], "all")
        assert logits.shape == (3, cfg.vocab) and torch.isfinite(logits).all()


def test_the_command_line_generates_from_a_model_folder(tmp_path, capsys):
    """``run_generation`` on a folder of this design: greedy tokens as the plain model chooses them."""
    from pytorch_transformers_amd import run_generation

    cfg = CONFIGS["delta"]
    w = make_weights(cfg, seed=15)
    folder = save(tmp_path / "m", cfg, w)
    rc = run_generation.main(["--model_name_or_path", folder, "--model_type", "verelorn", "--prompt_ids", "3,1,4,1,5",
                              "--length", "6", "--greedy", "--dtype", "float32"])
    assert rc == 0
    printed = [ln for ln in capsys.readouterr().out.splitlines() if ln and ln[0].isdigit()]
    assert [int(t) for t in printed[-1].split(",")] == [3, 1, 4, 1, 5] + P.greedy(w, cfg, [3, 1, 4, 1, 5], 6)


# ---- configurations drawn at random --------------------------------------------------------------------------------------
def draw_config(seed, large=False):
    import random

    r = random.Random(seed + (1000 if large else 0))
    sizes = (lambda small, big: r.choice(big if large else small))
    layers, sources = [], []
    for i in range(r.randint(2, 5)):
        ff = sizes([None, 8, 30, 64], [None, 192, 448])
        kind = r.choice(["attention", "latent", "latent", "delta"])
        if kind == "attention":
            kv, d = sizes([1, 2, 3], [1, 2, 4]), sizes([8, 12, 16, 40], [32, 48, 64, 128])
            layers.append(attn(kv * r.choice([1, 2, 4]), kv, d, r.choice([0.1, 0.2]), r.choice([0, 2, d // 2 // 2 * 2, d]),
                               r.choice([100.0, 10000.0, 500000.0]), r.random() < 0.5, ff))
        elif kind == "delta":
            G = r.choice([1, 2, 3])
            layers.append(delta(G * r.choice([1, 2, 3]), G, sizes([4, 12, 16, 40], [32, 64, 128]), sizes([5, 20, 48], [64, 96, 128]), r.choice([1, 2, 4, 5]),
                                sizes([1, 7, 16], [16, 24, 40]), sizes([1, 3, 16], [16, 20, 64]), ff))
        else:
            heads, dim, vdim, q_rank = sizes([1, 2, 3, 8], [4, 6, 12]), sizes([8, 12, 40], [32, 64, 128]), sizes([8, 20, 48], [32, 64, 128]), sizes([4, 12, 48], [64, 160])
            if sources and r.random() < 0.5:
                j = r.choice(sources)
                src = layers[j]["mixer"]
                layers.append(latent(heads, dim, src["rot_dim"], vdim, src["kv_rank"], q_rank, r.choice([0.1, 0.2]), src["rot"]["base"],
                                     src["rot"]["dims"], j, ff))
            else:
                dr = sizes([2, 4, 8, 16], [16, 32, 64])
                sources.append(i)
                layers.append(latent(heads, dim, dr, vdim, sizes([8, 24, 64], [64, 96, 256]), q_rank, r.choice([0.1, 0.2]), r.choice([100.0, 10000.0]),
                                     r.choice([2, dr]), None, ff))
    return config(layers, vocab=sizes([50, 101], [300, 513]), width=sizes([16, 24, 50, 72], [128, 192, 320]), eps=r.choice([1e-5, 1e-6, 1e-3]),
                  streams=r.randint(1, 5), taps=r.randint(1, 6))


@pytest.mark.parametrize("large,seed", [(False, s) for s in range(10)] + [(True, s) for s in range(6)])
def test_configurations_drawn_at_random(tmp_path, large, seed):
    from pytorch_transformers_amd.engine.replay import Replayer

    cfg = draw_config(seed, large)
    w = make_weights(cfg, seed=seed)
    reqs = helpers.make_requests(cfg["vocab"], [150, 9, 40, 70] if large else [70, 3, 130], seed=seed)
    want = plain_all(cfg, w, reqs)
    folder = save(tmp_path / "m", cfg, w)
    for dtype, rel in (("float32", helpers.REL_F32), ("bfloat16", REL_BF16_MODEL)):
        rp = Replayer(load(folder, dtype), 1024, max_slots=4)
        for label, records in (("whole", helpers.schedule_whole(reqs)), ("tail", helpers.schedule_tail(reqs, 20)),
                               ("batches", helpers.schedule_batches(reqs, 4, decode=(4, 1, 7)))):
            got = helpers.run_schedule(rp, records)
            for rid in reqs:
                assert_model_close(got[rid], want[rid], rel, f"{json.dumps(cfg)} {dtype} {label} {rid}")
