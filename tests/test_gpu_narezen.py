"""The Narezen design on the GPU against the plain implementation (``plain_narezen``): every mechanism alone, then whole models of
several shapes through the step function, the cache, captured decode steps and ``generate``.

The tests make their own small configurations and weights.  Sizes are chosen so that nothing is equal that need not be, and a
far key, a page's edge, a head's own sink, one tap or an expert's weight shows in the result instead of drowning in averages.
"""
import json
import os

import pytest
import torch

import helpers
import plain_narezen as P
from test_gpu_bimepel import _bf16, _close, _ctx, _load_part, _rand, _run_in_cuts, assert_model_close, load, write_model

pytestmark = pytest.mark.gpu

DTYPES = [("float32", 3e-5), ("bfloat16", 4e-2)]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
REL_BF16_MODEL = 0.1


# ---- configurations ---------------------------------------------------------------------------------------------
def moe(ff=24, experts=5, top=2, shared=40):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": {"ff": shared} if shared else None}


def rot(dims, base=10000.0):
    return {"base": base, "dims": dims} if dims else None


def tied(heads=6, kv=2, dim=24, scale=0.2, lheads=3, ldim=12, lvdim=20, tau=16.0, rank=7, scales=(0.6, 0.9), mlp=None):
    """Attention whose values are its keys, beside linear attention with a decay per key channel."""
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale}, "left_scale": scales[0],
        "right": {"heads": lheads, "dim": ldim, "vdim": lvdim, "tau": tau, "a_rank": rank}, "right_scale": scales[1]}}


def kept(heads=6, kv=2, dim=24, vdim=20, scale=0.25, dims=8, base=10000.0, lheads=3, ldim=12, lvdim=20, ldims=12, lbase=1e6,
         decay=(0.5, 0.9, 0.99), scales=(0.8, 1.1), mlp=None):
    """Rotated attention with one added to the softmax's sum, beside retention."""
    return {"type": "parallel_2", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot(dims, base)}, "left_scale": scales[0],
        "right": {"heads": lheads, "dim": ldim, "vdim": lvdim, "rot": rot(ldims, lbase), "decay": list(decay)}, "right_scale": scales[1]}}


def unit(width=48, blocks=3, conv=4, mlp=None):
    """A real-gated linear recurrent unit."""
    return {"type": "rglru", "mlp": mlp, "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def config(layers, vocab=131, width=48, eps=1e-5, scale=3.0, cap=12.0):
    return {"architecture": "Narezen", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "logit_softcap": cap}


CONFIGS = {
    # every mixer with and without a feed-forward, in two shapes each; one expert and several a token, no shared expert
    "mixed": config([tied(mlp=moe()), unit(mlp=moe(16, 7, 3, 24)), kept(mlp=moe(32, 4, 1, 16)), tied(4, 4, 40, 0.1, 2, 8, 36, 4.0, 16),
                     unit(40, 1, 2), kept(4, 1, 16, 32, 0.2, 0, 1e4, 4, 16, 8, 4, 100.0, (0.99, 0.3, 0.999, 0.8), (1.0, 0.5), moe(24, 3, 3, 0)),
                     unit(72, 9, 6, moe(8, 3, 1, 8))]),
    # one head, one tap, one expert, ranks and sizes of one: the values that make indices and states vanish
    # (the norm of a head that one key channel makes is all but the sign of q k, which every rounding near zero turns: a large eps)
    "ones": config([tied(1, 1, 16, 1.0, 1, 1, 7, 1.0, 1, (1.0, 1.0), moe(1, 1, 1, 1)), unit(16, 1, 1, moe(8, 2, 1, 3)),
                    kept(1, 1, 16, 16, 1.0, 2, 100.0, 1, 2, 9, 2, 100.0, (1.0,), (1.0, 1.0), moe(3, 2, 2, 1))], vocab=61, width=16, eps=0.1, scale=1.0, cap=1.0),
    # sizes the matrix-core kernels take, heads as columns that leave gaps of their own
    "wide": config([tied(8, 2, 32, 0.18, 4, 32, 64, 16.0, 16, (0.6, 0.9), moe(64, 8, 2, 128)), kept(8, 2, 64, 48, 0.12, 32, 1e4, 2, 64, 32, 64, 1e4,
                    (0.9, 0.995), (0.7, 1.2), moe(64, 4, 1, 64)), unit(128, 2, 4, moe(64, 4, 2, 64))], vocab=97, width=64),
    # the recurrent unit only: no layer keeps keys and values
    "recurrent": config([unit(64, 2, 4, moe()), unit(30, 5, 3), unit(96, 1, 5, moe(16, 2, 1, 8))], vocab=77, width=40, cap=30.0),
}


def _weight(n, shape, g, std=0.12):
    """A lively random weight by its name."""
    t = torch.randn(shape, generator=g)
    last = n.rsplit(".", 1)[-1]
    if last in ("norm1", "norm2", "norm1b", "norm2b", "norm"):
        return 1.0 + 0.3 * t
    if last == "conv":
        return 0.5 * t
    if last == "sink":
        return 1.0 + t
    if last == "router":
        return 1.5 * t * shape[-1] ** -0.5  # (scores that do not saturate, so that few choices are close)
    if last in ("ra", "ri"):
        return t * shape[-1] ** -0.5
    if n == "embed":
        return t
    if len(shape) == 1 or n.endswith(".b"):
        return 0.5 * t
    return t * std * (48.0 / shape[-1]) ** 0.5


def _named(specs, seed, std=0.12):
    g = torch.Generator().manual_seed(seed)
    return {n: _bf16(_weight(n, shape, g, std)) for s in specs for n, shape in (list(s.pieces) or [(s.name, s.shape)])}


def _spec(cfg):
    from pytorch_transformers_amd.config import AutoConfig
    from pytorch_transformers_amd.config.registry import lookup

    c = AutoConfig.from_dict(cfg)
    return lookup(c.model_type)[1](c)


def make_weights(cfg, seed):
    """Random weights by the design's tensor names, rounded to bfloat16 (so that both compute types hold the same
    numbers), as float64.  A layer's experts are alike (most of each is expert 0's): a router's choice between two all but equal
    scores, which bfloat16 rounding may turn, then moves the logits little; the experts' own test draws them freely."""
    w = _named(_spec(cfg).tensor_specs(), seed)
    for n in w:
        at = n.split(".")
        if len(at) == 4 and at[1] == "mlp" and at[2][0] == "e" and at[2] != "e0":
            w[n] = _bf16(0.95 * w[f"{at[0]}.mlp.e0.{at[3]}"] + 0.3 * w[n])
    return w


def file_config(cfg):
    """The configuration as a file has it: the inner size of the decays' product follows from the tensors."""
    cfg = json.loads(json.dumps(cfg))
    for l in cfg["layers"]:
        if l["type"] == "parallel":
            l["mixer"]["right"].pop("a_rank", None)
    return cfg


def save(folder, cfg, w):
    return write_model(folder, file_config(cfg), w)


def plain_all(cfg, w, reqs):
    return {rid: P.run_tokens(w, cfg, toks).float() for rid, toks in reqs.items()}


# ---- RMS norms around the stream ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,rel", [("float32", 3e-6), ("bfloat16", 5e-3)])
@pytest.mark.parametrize("width", [7, 16, 50, 64, 260, 1028, 2050, 4096, 8192])
def test_norms_around_the_stream(dtype, rel, width):
    """The norm behind a sublayer, the additions and the norm in front of the next one, together and each alone; all tokens
    and chosen ones; a sublayer's output whose rows lie apart."""
    from pytorch_transformers_amd import ops

    dt, M, eps, mult = TORCH[dtype], 6, 1e-3, 0.7
    x, y = _rand(M, width, seed=1, scale=2.0), _bf16(_rand(M, width, seed=2))
    add, vec = _rand(M, width, seed=3), _rand(width, seed=4)
    wy, w = 1 + 0.3 * _rand(width, seed=5), 1 + 0.3 * _rand(width, seed=6)
    f = lambda t: t.float().cuda()
    d = lambda t: t.double()
    behind = d(x) + mult * P.rms_norm(y, d(wy), eps)
    apart = torch.zeros(M, width + 24, dtype=dt, device="cuda")
    apart[:, :width] = y.to(dt).cuda()
    for y_dev in (y.to(dt).cuda(), apart[:, :width]):
        h, s = ops.layernorm_stream(dt, x=f(x), y=y_dev, post=(f(wy), None), mult=mult, pre=(f(w), None), eps=eps, rms=True)
        _close(s, behind, 3e-6, "stream")
        _close(h, P.rms_norm(behind, d(w), eps), rel + 3e-6, "norm")
        assert h.dtype == dt and s.dtype == torch.float32
    h, s = ops.layernorm_stream(dt, x=f(x), pre=(f(w), None), eps=eps, rms=True, want_wide=False)
    _close(h, P.rms_norm(d(x), d(w), eps), rel + 3e-6, "norm alone")
    assert s is None
    everything = behind + d(add) + d(vec)
    h, s = ops.layernorm_stream(dt, x=f(x), y=y.to(dt).cuda(), post=(f(wy), None), mult=mult, add=f(add), vec=f(vec), pre=(f(w), None), eps=eps, rms=True)
    _close(s, everything, 3e-6, "stream with further terms")
    _close(h, P.rms_norm(everything, d(w), eps), rel + 3e-6, "norm with further terms")
    rows = torch.tensor([4, 0, 4], dtype=torch.int32).cuda()
    h, _ = ops.layernorm_stream(dt, x=f(x), y=y.to(dt).cuda(), post=(f(wy), None), mult=mult, pre=(f(w), None), eps=eps, rms=True, rows=rows, want_wide=False)
    _close(h, P.rms_norm(behind, d(w), eps)[[4, 0, 4]], rel + 3e-6, "chosen rows")
    n, s = ops.layernorm_stream(dt, x=f(x), y=y.to(dt).cuda(), post=(f(wy), None), mult=mult, eps=eps, rms=True, want_narrow=True)
    _close(s, behind, 3e-6, "stream alone")
    _close(n, behind, rel, "stream in the compute type")
    with pytest.raises(ops.KernelError, match="bias"):
        ops.layernorm_stream(dt, x=f(x), pre=(f(w), f(w)), eps=eps, rms=True)


def test_norms_of_two_kinds_do_not_share_a_block():
    from pytorch_transformers_amd.parts import LayerNorm, RMSNorm, SandwichBlock

    rms = lambda n: RMSNorm(n, 8, 1e-5)
    with pytest.raises(ValueError, match="one kind"):
        SandwichBlock(None, None, rms("a"), LayerNorm("b", 8, 1e-5), None, None)
    with pytest.raises(ValueError, match="gain stored"):
        RMSNorm("c", 8, 1e-5, offset=1.0).affine()


# ---- capped logits ---------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("factor,cap", [(1.0, 30.0), (0.5, 2.0), (3.0, 0.0), (1.0, 0.25)])
def test_logits_are_scaled_and_capped(factor, cap):
    from pytorch_transformers_amd import ops

    x = torch.cat([_rand(500, seed=1, scale=20.0), torch.tensor([0.0, 1e-6, 1e4, -1e4, 3e-3])]).view(5, -1)
    got = ops.scale_(x.float().cuda(), factor, cap)
    want = x.float().double() * factor
    want = cap * torch.tanh(want / cap) if cap else want
    assert bool(((got.double().cpu() - want).abs() <= 4e-7 * want.abs() + 1e-30).all())


# ---- where attention writes its heads --------------------------------------------------------------------------------------
def _pools(nkv, d, n_pages, seed, dt):
    k, v = _bf16(_rand(n_pages, nkv, 64, d, seed=seed)), _bf16(_rand(n_pages, nkv, d, 64, seed=seed + 1))
    return k.to(dt).cuda(), v.to(dt).cuda()


@pytest.mark.parametrize("nh,nkv,d,keep", [(6, 2, 16, 12), (8, 1, 64, 64), (4, 4, 128, 100), (64, 1, 64, 48), (2, 1, 256, 4), (40, 2, 32, 28), (5, 5, 96, 96)])
def test_heads_go_where_they_are_wanted(nh, nkv, d, keep):
    """In every attention launch: the first elements of every head, scaled, into a block of columns of a wider matrix whose
    other columns stay as they are."""
    from pytorch_transformers_amd import ops

    mult, at = 0.375, 8
    i32 = lambda t: torch.tensor(t, dtype=torch.int32).cuda()
    table, sink = i32([[3, 0, 5, 1], [7, 2, 0, 0]]), _rand(nh, seed=3).cuda()
    for new in ([1, 1], [40, 70]):
        lens = [200, 70]
        cu, start = i32([0, new[0], sum(new)]), i32([n - m for n, m in zip(lens, new)])
        for dt in (torch.bfloat16, torch.float32):
            kp, vp = _pools(nkv, d, 8, 11, dt)
            q = _bf16(_rand(sum(new), nh, d, seed=13)).to(dt).cuda()
            if dt == torch.float32:
                seq = i32([0] * new[0] + [1] * new[1])
                pos = i32([lens[s] - new[s] + t for s in (0, 1) for t in range(new[s])])
                run = [lambda **kw: ops.attn_generic(q, kp, vp, table, seq, pos, None, d ** -0.5, sink=sink, **kw)]
            else:
                if new[0] == 1:
                    ways = [dict(n_splits=1, split_size=256), dict(n_splits=4, split_size=64)]
                    ways += [dict(n_splits=n, split_size=256 // n, decode_tiles=1, decode_waves=4) for n in (1, 2)
                             if ops.load_library().pta_attn_decode_waves_ok(d, 1, 4)]
                    if ops.attn_decode_shared_ok(d, nh // nkv):
                        ways += [dict(n_splits=n, split_size=256 // n, decode_waves=ops.SHARED_KEYS) for n in (1, 2)]
                else:
                    ways = [dict(prompt_wide=False)] + ([dict(prompt_wide=True)] if d <= 64 else [])
                run = [lambda w=w, **kw: ops.attn_mfma(q, kp, vp, table, cu, start, None, d ** -0.5, max_new=max(new), sink=sink, **w, **kw) for w in ways]
            for r in run:
                whole = r().view(-1, nh, d)[:, :, :keep].double() * mult
                wide = torch.full((sum(new), nh * keep + 24), 7.0, dtype=dt, device="cuda")
                r(into=(wide[:, at:at + nh * keep], keep, mult))
                got = wide[:, at:at + nh * keep].reshape(-1, nh, keep).double()
                tol = 1e-6 if dt == torch.float32 else 8e-3
                assert float((got - whole).abs().max()) <= tol * float(whole.abs().max())
                assert bool((wide[:, :at] == 7).all()) and bool((wide[:, at + nh * keep:] == 7).all())


def test_places_that_do_not_fit_are_refused():
    from pytorch_transformers_amd import ops

    kp, vp = _pools(1, 16, 2, 1, torch.bfloat16)
    q = torch.zeros(2, 2, 16, dtype=torch.bfloat16, device="cuda")
    i32 = lambda t: torch.tensor(t, dtype=torch.int32).cuda()
    args = (q, kp, vp, i32([[0], [1]]), i32([0, 1, 2]), i32([3, 5]), None, 0.25)
    out = torch.zeros(2, 64, dtype=torch.bfloat16, device="cuda")
    for into in ((out[:, :32], 17, 1.0), (out[:, :20], 10, 1.0), (out[:1, :32], 16, 1.0), (out[:, 1:33], 16, 1.0)):
        with pytest.raises(ops.KernelError):
            ops.attn_mfma(*args, max_new=1, into=into)
    assert bool((out == 0).all())


# ---- the mixers alone -----------------------------------------------------------------------------------------------------
def _mixer(layer, hidden, eps=1e-5):
    """The mixer of a model's one layer, its run order's entry and the cache groups it asks for."""
    spec = _spec(config([dict(layer, mlp=None)], width=hidden, eps=eps))
    return spec.blocks[0].mixer, spec.order[0], spec.cache_groups


def _plain_mixer(w, layer, x, eps=1e-5):
    seq = {"left": {}, "right": {}}
    return torch.stack([P.mixer_token(w, layer, "l0.mix", eps, x[pos], seq, pos) for pos in range(x.shape[0])])


SHAPES = [tied(), tied(4, 1, 16, 0.25, 2, 16, 16, 1.0, 4), tied(2, 2, 40, 0.1, 5, 8, 3, 0.5, 1, (1.5, -0.5)), tied(3, 1, 130, 0.1, 1, 33, 70, 16.0, 40),
          tied(20, 4, 16, 0.3, 2, 128, 128, 8.0, 24), tied(8, 2, 64, 0.12, 4, 64, 16, 16.0, 16), tied(1, 1, 8, 0.5, 1, 200, 40, 16.0, 8, (0.0, 1.0)),
          tied(64, 1, 64, 0.1, 1, 16, 200, 2.0, 64, (1.0, 0.0)), tied(5, 5, 12, 0.3, 3, 6, 5, 3.0, 33),
          kept(), kept(4, 1, 16, 32, 0.2, 0, 1e4, 4, 16, 8, 4, 100.0, (0.99, 0.3, 0.999, 0.8), (1.0, 0.5)), kept(2, 2, 40, 8, 0.15, 40, 1e4, 1, 1, 3, 0, 1e4, (1.0,)),
          kept(3, 1, 130, 40, 0.1, 72, 500.0, 2, 128, 128, 128, 1e4, (0.96875, 0.9990234375)), kept(8, 2, 64, 64, 0.12, 32, 1e4, 2, 33, 70, 32, 1e5, (0.0, 0.9)),
          kept(1, 1, 8, 13, 0.5, 2, 10.0, 1, 200, 40, 200, 1e4, (0.99,), (0.0, 1.0)), kept(6, 3, 24, 9, 0.3, 24, 1e4, 3, 5, 7, 4, 1e4, (0.5, 0.7, 0.9), (1.0, 0.0)),
          unit(), unit(16, 1, 1), unit(40, 5, 2), unit(128, 2, 4), unit(66, 3, 6), unit(1, 1, 3), unit(257, 1, 4), unit(96, 1, 16), unit(320, 2, 3)]


@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("layer", SHAPES, ids=lambda s: s["type"] + "-" + "-".join(
    str(v) for m in (s["mixer"], s["mixer"].get("left", {}), s["mixer"].get("right", {})) for v in m.values() if isinstance(v, (int, float))))
def test_mixer_alone(dtype, rel, layer):
    """Whole, token by token, in portions down to two tokens and across page borders, four sequences a step, and once more on
    slots and pages that were given back."""
    hidden, dt = 32, TORCH[dtype]
    mixer, call, groups = _mixer(layer, hidden)
    w = _named(mixer.all_tensor_specs(), seed=5, std=0.25)
    _load_part(mixer, w, dt)
    cuts = [[150], [64, 1, 1, 62, 2, 20], [1] * 20 + [130], [63, 2, 85]]
    xs = [_bf16(_rand(150, hidden, seed=40 + i)) for i in range(4)]
    outs = _run_in_cuts(lambda x, ctx: mixer.forward(x, ctx, call), groups, dt, xs, cuts, free_and_again=True)
    for i in range(4):
        _close(outs[i], _plain_mixer(w, layer, xs[i]), rel, f"{layer['type']} {layer['mixer']} sequence {i}")


@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("layer", [tied(1, 1, 8, 0.3, 3, 12, 20, 16.0, 7, (0.0, 1.0)), tied(1, 1, 8, 0.3, 2, 128, 128, 16.0, 16, (0.0, 1.0)),
                                   tied(1, 1, 8, 0.3, 1, 200, 40, 16.0, 5, (0.0, 1.0)), tied(1, 1, 8, 0.3, 2, 30, 72, 4.0, 16, (0.0, 1.0)),
                                   kept(1, 1, 8, 8, 0.3, 0, 1e4, 3, 12, 20, 12, 1e6, (0.999, 0.9, 0.99), (0.0, 1.0)),
                                   kept(1, 1, 8, 8, 0.3, 0, 1e4, 2, 64, 140, 64, 1e4, (0.9990234375, 1.0), (0.0, 1.0)),
                                   unit(48, 3, 4), unit(130, 1, 3)], ids=lambda s: s["type"] + str(s["mixer"].get("width", s["mixer"].get("right", {}).get("dim"))))
def test_states_over_prompts_cut_into_chunks(dtype, rel, layer):
    """Sequences long enough that the recurrence runs in chunks side by side, beside shorter ones and single tokens, with a
    state from before: the same as token by token.  Decays slow enough that what a chunk starts from reaches far."""
    hidden, dt = 24, TORCH[dtype]
    mixer, call, groups = _mixer(layer, hidden)
    w = _named(mixer.all_tensor_specs(), seed=7, std=0.25)
    for n in ("l0.mix.right.a2.b", "l0.mix.lam"):
        if n in w:
            w[n] = w[n] + (3.0 if n.endswith("b") else -5.0)
    _load_part(mixer, w, dt)
    cuts = [[700], [2, 257, 1, 440], [384, 1, 315], [1, 300, 399]]
    xs = [_bf16(_rand(700, hidden, seed=60 + i)) for i in range(4)]
    outs = _run_in_cuts(lambda x, ctx: mixer.forward(x, ctx, call), groups, dt, xs, cuts, free_and_again=True)
    for i in range(4):
        _close(outs[i], _plain_mixer(w, layer, xs[i]), rel, f"{layer['mixer']} sequence {i}")


@pytest.mark.parametrize("tokens", [9, 40, 300])
def test_a_channel_that_forgets_at_once_beside_one_that_keeps_everything(tokens):
    """Decays of zero (to the last bit) and of one among a head's key channels, in every way the recurrence runs: the kept
    channel sums all keys, the other shows the token's own alone, and nothing overflows."""
    from pytorch_transformers_amd import ops
    from pytorch_transformers_amd.cache.paged import PagedCache
    from pytorch_transformers_amd.engine.spec import CACHE_STATE, CacheGroupSpec

    N, V, dt = 4, 3, torch.float32
    proj = torch.zeros(tokens, 2 * N + 2 * V + 1)
    q, k, v, g, low = torch.split(proj, [N, N, V, V, 1], dim=1)
    k[:, 0] = k[:, 1] = 1.0
    q[::2, 0], q[1::2, 1] = 1.0, 1.0
    v.copy_(1.0 + torch.arange(tokens * V).view(tokens, V) % 7)
    g.fill_(30.0)  # (silu of it is itself)
    low.fill_(1.0)
    a2, bias = torch.tensor([[0.0], [-4000.0], [0.0], [500.0]]), torch.tensor([90.0, 0.0, -120.0, 0.0])
    cache = PagedCache([CacheGroupSpec("s", CACHE_STATE, 1, state_shape=(N * V,))], 1024, dt, "cuda:0", max_slots=2)
    ctx, _ = _ctx(cache, [cache.alloc()], [tokens], dt)
    dev = proj.cuda()
    qd, kd, vd, gd, ld = torch.split(dev, [N, N, V, V, 1], dim=1)
    out = ops.linear_state(qd, kd, vd, gd, cache.state_layer("s", 0), ctx, 1, N, V, channel_decay=(ld, a2.cuda(), bias.cuda(), 0.5), eps=1e-6, mult=1 / 30.0)
    o = torch.where(torch.arange(tokens)[:, None] % 2 == 0, v.cumsum(0), v)
    _close(out, P.unit_rms(o.double(), 1e-6), 1e-5, f"{tokens} tokens")


def test_gate_products_are_32_bit_in_a_bfloat16_model():
    """The recurrent unit's gates see every bit of u: two channels that nearly cancel in a gate's product (large, opposite
    weights) leave what a bfloat16 u would have rounded away."""
    from pytorch_transformers_amd import ops
    from pytorch_transformers_amd.cache.paged import PagedCache
    from pytorch_transformers_amd.engine.spec import CACHE_STATE, CacheGroupSpec

    W, M = 32, 40
    g = torch.Generator().manual_seed(3)
    x = torch.randn(M, W, generator=g).bfloat16()
    conv = torch.full((1, W), 1.0)
    cb = torch.zeros(W)
    cb[0::2] = 1.0 + torch.rand(16, generator=g) * 2 ** -10  # u[2i] - u[2i + 1] is of the size of bfloat16's steps
    cb[1::2] = 1.0
    x[:, 1::2] = x[:, 0::2]
    ra = torch.zeros(1, W, W)
    for i in range(0, W, 2):
        ra[0, i, i], ra[0, i, i + 1] = 1024.0, -1024.0
    lam, zero = torch.full((W,), -3.0), torch.zeros(W)
    for one_each in (False, True):
        cache = PagedCache([CacheGroupSpec("s", CACHE_STATE, 1, state_shape=(2 * W,))], 64 * M, torch.bfloat16, "cuda:0", max_slots=M)
        slots = [cache.alloc() for _ in range(M if one_each else 1)]
        ctx, _ = _ctx(cache, slots, [1] * M if one_each else [M], torch.bfloat16)
        yx = torch.cat([torch.full((M, W), 8.0), x.float()], dim=1).bfloat16().cuda()
        f = lambda t: t.float().cuda()
        gates = ops.pack_gates(ra.bfloat16().cuda(), torch.zeros_like(ra).bfloat16().cuda())
        got = ops.rglru(yx[:, :W], yx[:, W:], None, None, f(conv), f(cb), gates, f(zero), f(zero), f(lam), -8.0, cache.state_layer("s", 0), ctx)
        S, want = torch.zeros(W, dtype=torch.float64), []
        for t in range(M):
            u = x[t].double() + cb.double()
            log_a = -8.0 * P.sigmoid(ra[0].double() @ u.float().double()) * P.softplus(lam.double())
            S = (0 if one_each else 1) * torch.exp(log_a) * S + torch.sqrt(-torch.expm1(2 * log_a)) * 0.5 * u
            want.append(S * 8.0)
        _close(got, torch.stack(want), 6e-3, "one token each" if one_each else "a prompt")


# ---- experts whose weight multiplies their input ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("ff,experts,top,shared,hidden", [(24, 5, 2, 40, 48), (1, 1, 1, 1, 8), (64, 8, 1, 128, 64), (64, 6, 6, 64, 128), (40, 70, 3, 0, 32), (192, 4, 2, 320, 192)])
@pytest.mark.parametrize("rows", [1, 5, 40, 200])
def test_weights_on_the_experts_inputs(dtype, rel, ff, experts, top, shared, hidden, rows):
    from pytorch_transformers_amd import ops
    from pytorch_transformers_amd.engine.narezen import _feed_forward
    from pytorch_transformers_amd.config import AutoConfig

    dt, mlp = TORCH[dtype], moe(ff, experts, top, shared)
    part = _feed_forward(AutoConfig.from_dict(config([unit(mlp=mlp)], width=hidden)), "f", mlp)
    w = _named(part.all_tensor_specs(), seed=ff + rows, std=0.3)
    _load_part(part, w, dt)
    x = _bf16(_rand(rows, hidden, seed=1, scale=1.2))
    got = part.forward(x.to(dt).cuda(), None)
    want = torch.stack([P.routed_ff(w, "f", mlp, x[i]) for i in range(rows)])
    scores = (P.sigmoid(x @ w["f.router"].T)).sort(dim=1, descending=True)[0]
    clear = torch.ones(rows, dtype=torch.bool) if top == experts else scores[:, top - 1] - scores[:, top] > 1e-4
    assert int(clear.sum()) >= max(1, rows - 5)
    _close(got.cpu()[clear], want[clear], rel, f"{top} of {experts} experts of {ff}, shared {shared}")
    if top == 1 and experts > 1:  # a weight on the output instead would be another result
        out = torch.stack([P.sigmoid(w["f.router"] @ v).max() * P.glu_ff(w, f"f.e{int((w['f.router'] @ v).argmax())}", v) + P.glu_ff(w, "f.shared", v) for v in x])
        assert float((out - want).abs().max()) > rel * float(want.abs().max())
    ids, _ = ops.moe_route(x.to(dt).cuda(), part.router, top, "sigmoid", False, 1.0)
    for i in torch.nonzero(clear).flatten().tolist():
        assert set(ids[i].tolist()) == set(torch.topk(w["f.router"] @ x[i], top).indices.tolist())


# ---- sinks --------------------------------------------------------------------------------------------------------------
def test_a_heads_own_sink_is_that_heads_and_is_not_scaled():
    """Two heads equal in everything but their sinks; swapping the sinks swaps their outputs."""
    layer, hidden, dt = tied(2, 1, 16, 0.05, 1, 4, 4, 1.0, 1, (1.0, 0.0)), 32, torch.float32
    outs = []
    for sinks in ([-6.0, 2.5], [2.5, -6.0]):
        mixer, call, groups = _mixer(layer, hidden)
        w = _named(mixer.all_tensor_specs(), seed=9, std=0.25)
        w["l0.mix.left.q"][16:] = w["l0.mix.left.q"][:16]
        w["l0.mix.left.sink"] = _bf16(torch.tensor(sinks))
        _load_part(mixer, w, dt)
        x = _bf16(_rand(40, hidden, seed=1))
        got = _run_in_cuts(lambda t, ctx: mixer.forward(t, ctx, call), groups, dt, [x], [[30] + [1] * 10])[0]
        _close(got, _plain_mixer(w, layer, x), 3e-5, "two heads with sinks of their own")
        outs.append((got.double() @ torch.linalg.pinv(w["l0.mix.left.o"]).T).view(40, 2, 16))  # undo W_o: the heads side by side
    tol = 1e-4 * float(outs[0].abs().max())
    assert float((outs[0][:, 0] - outs[1][:, 1]).abs().max()) < tol
    assert float((outs[0][:, 0] - outs[0][:, 1]).abs().max()) > 100 * tol


@pytest.mark.parametrize("dtype,rel", DTYPES)
def test_one_joins_the_sum_without_a_value(dtype, rel):
    """A first token alone: its weight is e^s / (1 + e^s), which a softmax without the one would make 1."""
    layer, hidden, dt = kept(2, 1, 16, 16, 0.02, 0, 1e4, 1, 4, 4, 0, 1e4, (0.5,), (1.0, 0.0)), 32, TORCH[dtype]
    mixer, call, groups = _mixer(layer, hidden)
    w = _named(mixer.all_tensor_specs(), seed=3, std=0.25)
    _load_part(mixer, w, dt)
    x = _bf16(_rand(3, hidden, seed=2))
    got = _run_in_cuts(lambda t, ctx: mixer.forward(t, ctx, call), groups, dt, [x], [[1, 1, 1]])[0]
    want = _plain_mixer(w, layer, x)
    _close(got, want, rel, "first tokens")
    value = w["l0.mix.left.o"] @ (w["l0.mix.left.v"] @ x[0]).repeat(2)
    assert 0.3 < float(want[0].norm() / value.norm()) < 0.7


# ---- far keys --------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,rel", DTYPES)
@pytest.mark.parametrize("kind", ["parallel", "parallel_2"])
@pytest.mark.parametrize("query,key", [(500, 0), (500, 1), (500, 63), (500, 64), (500, 137), (200, 199), (200, 201), (191, 127),
                                       (192, 128), (64, 63), (64, 65), (63, 0), (9, 8), (2, 0), (1, 0), (300, 302)])
def test_one_loud_key_is_seen_from_wherever_it_lies_behind(dtype, rel, kind, query, key):
    """One key far back among hundreds, at a page's first and last place, among a sequence's first tokens, right behind the
    query, and ahead of it (where it must not be seen): fed whole and with the query decoded alone.  The plain side checks
    that the loud key shows exactly where it is visible."""
    hidden, half, d, dt = 32, 16, 24, TORCH[dtype]
    layer = tied(2, 1, d, 0.9, 1, 4, 4, 1.0, 1, (1.0, 0.0)) if kind == "parallel" else kept(2, 1, d, 20, 0.9, 0, 1e4, 1, 4, 4, 0, 1e4, (0.5,), (1.0, 0.0))
    mixer, call, groups = _mixer(layer, hidden)
    w = _named(mixer.all_tensor_specs(), seed=6, std=0.3)
    p = "l0.mix.left."
    # the first half of a head's key reads the first half of the input and makes the score; the values read the rest
    w[p + "k"][:d // 2, half:] = 0
    w[p + "k"][d // 2:, :half] = 0
    q = w[p + "k"].clone()
    q[d // 2:] = 0
    w[p + "q"] = q.repeat(2, 1)
    if kind == "parallel_2":
        w[p + "v"][:, :half] = 0
    n = max(query, key) + 2
    x = _bf16(_rand(n, hidden, seed=7))
    x[:, :half] = _bf16(0.3 * x[:, :half])
    _load_part(mixer, w, dt)
    loud = _bf16(_rand(half, seed=8) * 3.0)
    x[key, :half] = x[query, :half] = loud
    # (the query's own key reads the loud half as well: in a normed key its other half stands against it)
    x[key, half:] = _bf16(_rand(half, seed=9) * 0.5)
    x[query, half:] = _bf16(_rand(half, seed=10) * 3.0)
    want = _plain_mixer(w, layer, x)
    quiet = x.clone()
    quiet[key] = x[next(i for i in range(n) if i not in (key, query))]
    moved = float((_plain_mixer(w, layer, quiet)[query] - want[query]).abs().max()) > 0.1 * float(want[query].abs().max())
    assert moved == (key < query), "the test's loud key does not show where it should"
    first = min(key, query)
    for cuts in ([n], [query, 1, n - query - 1], [first + 1, query - first - 1, 1, n - query - 1] if query - first > 1 else [1] * n):
        got = _run_in_cuts(lambda t, ctx: mixer.forward(t, ctx, call), groups, dt, [x], [[c for c in cuts if c]])[0]
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


def test_the_stream_after_every_layer(tmp_path):
    """The 32-bit stream after every layer, last token of a prompt, against the plain model's."""
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
        _close(seen[i], want, 2e-5, f"stream after layer {i}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_decode_steps_equal_direct_ones(tmp_path, dtype):
    """Decode steps replayed from a captured graph give the bits of the same steps launched one by one, with batches that
    are padded to the captured size."""
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
    """A prompt of several hundred tokens (the recurrences in chunks, a dozen pages) beside a short one, then decoded."""
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
    assert {"embed", "final.norm", "head", "l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l0.mix.left.q", "l0.mix.left.k", "l0.mix.left.sink",
            "l0.mix.left.o", "l0.mix.right.q", "l0.mix.right.k", "l0.mix.right.v", "l0.mix.right.g", "l0.mix.right.o", "l0.mix.right.norm",
            "l0.mix.right.a1", "l0.mix.right.a2", "l0.mix.right.a2.b", "l0.mlp.router", "l0.mlp.e4.gate", "l0.mlp.e0.up", "l0.mlp.e1.down",
            "l0.mlp.shared.gate", "l0.mlp.shared.up", "l0.mlp.shared.down", "l1.mix.y", "l1.mix.y.b", "l1.mix.x", "l1.mix.x.b", "l1.mix.conv",
            "l1.mix.conv.b", "l1.mix.ra", "l1.mix.ra.b", "l1.mix.ri", "l1.mix.ri.b", "l1.mix.lam", "l1.mix.o", "l2.mix.left.v", "l2.mix.right.g"} <= names
    assert not any(n.startswith(("l3.mlp", "l3.norm2", "l0.mix.left.v", "l2.mix.left.sink", "l2.mix.right.norm", "l5.mlp.shared")) or n.endswith((".weight", ".bias"))
                   for n in names)
    for dtype in ("bfloat16", "float32"):
        model = AutoModelForCausalLM.from_pretrained(folder, dtype=dtype)
        cache = model.new_cache(256)
        logits = model.step(cache, [cache.alloc()], [[1, 2, 3]], "all")
        assert logits.shape == (3, cfg.vocab) and torch.isfinite(logits).all()


def test_the_command_line_generates_from_a_model_folder(tmp_path, capsys):
    """``run_generation`` on a folder of this design: greedy tokens as the plain model chooses them."""
    from pytorch_transformers_amd import run_generation

    cfg = CONFIGS["recurrent"]
    w = make_weights(cfg, seed=15)
    folder = save(tmp_path / "m", cfg, w)
    rc = run_generation.main(["--model_name_or_path", folder, "--model_type", "narezen", "--prompt_ids", "3,1,4,1,5",
                              "--length", "6", "--greedy", "--dtype", "float32"])
    assert rc == 0
    printed = [ln for ln in capsys.readouterr().out.splitlines() if ln and ln[0].isdigit()]
    assert [int(t) for t in printed[-1].split(",")] == [3, 1, 4, 1, 5] + P.greedy(w, cfg, [3, 1, 4, 1, 5], 6)


# ---- configurations drawn at random --------------------------------------------------------------------------------------
def draw_config(seed, large=False):
    import random

    r = random.Random(seed + (1000 if large else 0))
    sizes = (lambda small, big: r.choice(big if large else small))
    layers = []
    for i in range(r.randint(2, 5)):
        mlp = None
        if r.random() < 0.8:
            experts = r.randint(1, 9)
            mlp = moe(sizes([8, 30, 64], [64, 192]), experts, r.randint(1, min(experts, 3)), r.choice([0, 24, 128]))
        kind = r.choice(["tied", "kept", "unit"])
        kv, d = sizes([1, 2, 3], [1, 2, 4]), sizes([8, 12, 16, 40], [32, 48, 64, 128])
        heads, lheads = kv * r.choice([1, 2, 4]), sizes([1, 2, 3, 5], [2, 4, 8])
        ldim, lvdim = sizes([4, 12, 16, 40], [32, 64, 128]), sizes([5, 20, 48], [32, 64, 128])
        scales = (r.choice([0.5, 1.0, 0.8]), r.choice([0.7, 1.0, 1.2]))
        if kind == "tied":
            layers.append(tied(heads, kv, d, r.choice([0.1, 0.2]), lheads, ldim, lvdim, r.choice([1.0, 4.0, 16.0]), sizes([1, 7, 16], [16, 24, 40]), scales, mlp))
        elif kind == "kept":
            decay = [r.choice([0.5, 0.9, 0.984375, 0.9990234375]) for _ in range(lheads)]
            layers.append(kept(heads, kv, d, sizes([4, 8, 20, 48], [32, 64, 128]), r.choice([0.1, 0.2]), r.choice([0, 2, d // 2 // 2 * 2, d]), r.choice([100.0, 10000.0]),
                               lheads, ldim, lvdim, r.choice([0, 2, ldim]), r.choice([100.0, 1e6]), decay, scales, mlp))
        else:
            blocks = r.choice([1, 2, 3, 5])
            layers.append(unit(blocks * sizes([1, 8, 20, 33], [32, 64, 160]), blocks, r.randint(1, 6), mlp))
    return config(layers, vocab=sizes([50, 101], [300, 513]), width=sizes([16, 24, 50, 72], [128, 192, 320]), eps=r.choice([1e-5, 1e-6, 1e-3]),
                  scale=r.choice([1.0, 4.0, 12.0]), cap=r.choice([5.0, 30.0]))


@pytest.mark.parametrize("large,seed", [(False, s) for s in range(12)] + [(True, s) for s in range(8)])
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
            # (all requests' positions together: in bfloat16 a few may rest on a close choice of the routers)
            assert_model_close(torch.cat([got[r] for r in reqs]), torch.cat([want[r] for r in reqs]), rel, f"{json.dumps(cfg)} {dtype} {label}")
