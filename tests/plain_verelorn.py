"""A plain, slow implementation of the Verelorn design in float64 on the CPU: one function per mechanism, written from
the equations in each docstring, sharing no code with the package.  A sequence is walked token by token; what a
sequence keeps between tokens is, per layer, a dict: the last inputs of the convolution in front of the mixer, and
what the mixer keeps (attention: rotated keys and values; latent attention: latents and rotated key parts; the delta
rule: its states and the last inputs of its three convolutions).

``weights``: name -> float64 tensor, under the names of the weight file.  ``cfg``: the dict of ``config.json``.
"""
from __future__ import annotations

import math
from typing import Dict, List

import torch

F = torch.float64


def unit_rms(v: torch.Tensor, eps: float) -> torch.Tensor:
    """v / sqrt(mean(v^2) + eps) over the last dimension."""
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def model_norm(v: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """unit_rms(v) * (1 + w)."""
    return unit_rms(v, eps) * (1.0 + w)


def sigmoid(v):
    return 1.0 / (1.0 + torch.exp(-v))


def silu(v):
    return v * sigmoid(v)


def softplus(v: torch.Tensor) -> torch.Tensor:
    """ln(1 + e^v)."""
    return torch.logaddexp(v, torch.zeros_like(v))


def gelu_tanh(v: torch.Tensor) -> torch.Tensor:
    """v/2 (1 + tanh(sqrt(2/pi) (v + 0.044715 v^3)))."""
    return 0.5 * v * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (v + 0.044715 * v ** 3)))


def rotary_frequencies(rot: dict) -> List[float]:
    """f_i = base^(-2i/dims), i < dims/2.  With ``scaling`` (factor, low, high, original) and the wavelength l = 2 pi / f:
    l < original/high: f; l > original/low: f / factor; between: with s = (original/l - low) / (high - low), (1 - s) f /
    factor + s f."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        sc = rot.get("scaling")
        if sc:
            factor, low, high, original = (float(sc[k]) for k in ("factor", "low", "high", "original"))
            wave = 2.0 * math.pi / f
            if wave > original / low:
                f = f / factor
            elif not wave < original / high:
                s = (original / wave - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return out


def rotate(v: torch.Tensor, pos: int, rot: dict, layout: str) -> torch.Tensor:
    """The first ``dims`` elements of the last dimension turned by the position, the rest as they are.  Pairs: ``half``
    (i, i + dims/2), ``interleaved`` (2i, 2i + 1); (u, w) becomes (u cos a - w sin a, w cos a + u sin a), a = pos * f_i."""
    if not rot:
        return v
    half = int(rot["dims"]) // 2
    out = v.clone()
    for i, f in enumerate(rotary_frequencies(rot)):
        iu, iw = (i, i + half) if layout == "half" else (2 * i, 2 * i + 1)
        c, s = math.cos(pos * f), math.sin(pos * f)
        u, w = v[..., iu], v[..., iw]
        out[..., iu] = u * c - w * s
        out[..., iw] = w * c + u * s
    return out


def causal_conv(kept: List[torch.Tensor], now: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """sum_j w[:, j] * (input of taps - 1 - j tokens ago), the last column being the current token's; ``kept`` (oldest
    first, at most taps - 1 entries, missing ones are zeros) takes the current input in."""
    taps = w.shape[1]
    out = w[:, taps - 1] * now
    for back in range(1, taps):
        if back <= len(kept):
            out = out + w[:, taps - 1 - back] * kept[-back]
    kept.append(now)
    while len(kept) > taps - 1:
        kept.pop(0)
    return out


def hyper_input(streams: torch.Tensor, weights: torch.Tensor) -> torch.Tensor:
    """u = sum_s weights[s] x_s; streams [S, width]."""
    return (weights[:, None] * streams).sum(0)


def hyper_update(streams: torch.Tensor, mix: torch.Tensor, out: torch.Tensor, y: torch.Tensor) -> torch.Tensor:
    """x_t <- sum_s mix[s, t] x_s + out[t] y."""
    return torch.stack([sum(mix[s, t] * streams[s] for s in range(streams.shape[0])) + out[t] * y
                        for t in range(streams.shape[0])])


def attention_token(w, p: str, m: dict, h: torch.Tensor, kept: dict, pos: int) -> torch.Tensor:
    """q = W_q h + b_q in H heads, k = W_k h + b_k in G heads, v = k; q and k rotated (half layout); (k, v) is kept.  For
    every kept j and head g (key head g // (H/G)): s = q_g . k_j * scale; weights e^s / (sum_j e^s + e^sink_g); head g's
    weighted sum of values; the heads side by side times sigmoid(W_g h), through W_o."""
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q = (w[p + ".q"] @ h + w[p + ".q.b"]).view(H, d)
    k = (w[p + ".k"] @ h + w[p + ".k.b"]).view(G, d)
    v = k
    q, k = rotate(q, pos, m.get("rot"), "half"), rotate(k, pos, m.get("rot"), "half")
    kept.setdefault("k", []).append(k)
    kept.setdefault("v", []).append(v)
    ks, vs = torch.stack(kept["k"]), torch.stack(kept["v"])
    out = []
    for g in range(H):
        s = ks[:, g // (H // G)] @ q[g] * float(m["scale"])
        sink = w[p + ".sink"][g]
        top = max(float(s.max()), float(sink))
        e = torch.exp(s - top)
        a = e / (e.sum() + torch.exp(sink - top))
        out.append(a @ vs[:, g // (H // G)])
    return w[p + ".o"] @ (torch.cat(out) * sigmoid(w[p + ".g"] @ h))


def latent_attention_token(w, p: str, m: dict, eps: float, h: torch.Tensor, kept: dict, pos: int) -> torch.Tensor:
    """c_q = unit_rms(W_dq h) * dq.norm; q = W_uq c_q, per head [dim plain | rot_dim rotated].  Unless the layer reads
    another layer's (``kv_from``, then ``kept`` is that layer's and holds this token already): d = W_dkv h, c =
    unit_rms(d[:rank]) * dkv.norm, r = rotate(d[rank:]) (one for all heads), (c, r) is kept.  For every kept j and head
    g: s = (q_plain . (W_uk c_j)[g] + rotate(q_rot) . r_j) * scale; softmax over j; values (W_uv c_j)[g]; W_o on the
    heads side by side.  Interleaved pairs."""
    H, d, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (w[p + ".uq"] @ (unit_rms(w[p + ".dq"] @ h, eps) * w[p + ".dq.norm"])).view(H, d + dr)
    q_plain, q_rot = q[:, :d], rotate(q[:, d:], pos, m.get("rot"), "interleaved")
    if m.get("kv_from") is None:
        down = w[p + ".dkv"] @ h
        kept.setdefault("c", []).append(unit_rms(down[:R], eps) * w[p + ".dkv.norm"])
        kept.setdefault("r", []).append(rotate(down[R:], pos, m.get("rot"), "interleaved"))
    cs, rs = torch.stack(kept["c"]), torch.stack(kept["r"])
    keys = (cs @ w[p + ".uk"].T).view(-1, H, d)
    vals = (cs @ w[p + ".uv"].T).view(-1, H, dv)
    out = []
    for g in range(H):
        s = (keys[:, g] @ q_plain[g] + rs @ q_rot[g]) * float(m["scale"])
        out.append(torch.softmax(s, dim=-1) @ vals[:, g])
    return w[p + ".o"] @ torch.cat(out)


def delta_state_step(S: torch.Tensor, g, q, k, v, beta):
    """S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; returns (S, S^T q).  S: [dim, vdim]."""
    S = g[:, None] * S
    u = beta * (v - S.T @ k)
    S = S + torch.outer(k, u)
    return S, S.T @ q


def channel_delta_token(w, p: str, m: dict, eps: float, h: torch.Tensor, kept: dict) -> torch.Tensor:
    """q, k, v: silu of a causal convolution of W_q h, W_k h (G heads of dim), W_v h (H heads of vdim); q and k to unit
    length per head (1e-6 in the root), q times dim^(-1/2); beta = sigmoid(W_b h) per head; g = exp(-exp(A_log) *
    softplus(W_a2 W_a1 h + dt_bias)) per head and key channel; head i on q / k head i // (H/G) through
    delta_state_step; every head's result over its root mean square, times ``norm``, times sigmoid(W_g2 W_g1 h); W_o."""
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    made = {}
    for t in ("q", "k", "v"):
        made[t] = silu(causal_conv(kept.setdefault(t, []), w[f"{p}.{t}"] @ h, w[f"{p}.{t}.conv"]))
    q, k, v = made["q"].view(G, d), made["k"].view(G, d), made["v"].view(H, dv)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * d ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    beta = sigmoid(w[p + ".b"] @ h)
    a = (w[p + ".a2"] @ (w[p + ".a1"] @ h) + w[p + ".dt_bias"]).view(H, d)
    g = torch.exp(-torch.exp(w[p + ".A_log"])[:, None] * softplus(a))
    S = kept.setdefault("S", [torch.zeros(d, dv, dtype=F) for _ in range(H)])
    out = []
    for i in range(H):
        j = i // (H // G)
        S[i], o = delta_state_step(S[i], g[i], q[j], k[j], v[i], beta[i])
        out.append(unit_rms(o, eps) * w[p + ".norm"])
    return w[p + ".o"] @ (torch.cat(out) * sigmoid(w[p + ".g2"] @ (w[p + ".g1"] @ h)))


def dense_ff(w, p: str, h: torch.Tensor) -> torch.Tensor:
    """W_down (gelu_tanh(W_gate h) * (W_up h))."""
    return w[p + ".down"] @ (gelu_tanh(w[p + ".gate"] @ h) * (w[p + ".up"] @ h))


class Sequence:
    """What one sequence keeps: per layer the mixer's dict and the inputs of the convolution in front of it."""

    def __init__(self, cfg: dict):
        self.mixer = [{} for _ in cfg["layers"]]
        self.inputs = [[] for _ in cfg["layers"]]
        self.length = 0


def mixer_token(w, cfg: dict, i: int, h: torch.Tensor, seq: Sequence, pos: int) -> torch.Tensor:
    layer, eps, p = cfg["layers"][i], float(cfg["norm"]["eps"]), f"l{i}.mix"
    m = layer["mixer"]
    if layer["type"] == "attention":
        return attention_token(w, p, m, h, seq.mixer[i], pos)
    if layer["type"] == "latent_attention":
        return latent_attention_token(w, p, m, eps, h, seq.mixer[i if m.get("kv_from") is None else m["kv_from"]], pos)
    return channel_delta_token(w, p, m, eps, h, seq.mixer[i])


def step_token(w: Dict[str, torch.Tensor], cfg: dict, seq: Sequence, token: int, streams: List = None) -> torch.Tensor:
    """One token: every stream starts as model_norm(embed[token]); per sublayer u = hyper_input, y = sublayer of
    model_norm(u) (the mixer's with its convolution added), hyper_update; logits = head . model_norm(sum of the
    streams).  ``streams`` collects the sum of the streams after every layer."""
    eps = float(cfg["norm"]["eps"])
    pos = seq.length
    x = model_norm(w["embed"][token], w["embed.norm"], eps)
    xs = torch.stack([x] * int(cfg["streams"]))
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        h = model_norm(hyper_input(xs, w[p + ".hc1.in"]), w[p + ".norm1"], eps)
        h = h + causal_conv(seq.inputs[i], h, w[p + ".canon1"])
        y = mixer_token(w, cfg, i, h, seq, pos)
        xs = hyper_update(xs, w[p + ".hc1.mix"], w[p + ".hc1.out"], y)
        if layer.get("mlp") is not None:
            h = model_norm(hyper_input(xs, w[p + ".hc2.in"]), w[p + ".norm2"], eps)
            xs = hyper_update(xs, w[p + ".hc2.mix"], w[p + ".hc2.out"], dense_ff(w, p + ".mlp", h))
        if streams is not None:
            streams.append(xs.sum(0))
    seq.length += 1
    return w["head"] @ model_norm(xs.sum(0), w["final.norm"], eps)


def run_tokens(w, cfg: dict, tokens: List[int], seq: Sequence = None) -> torch.Tensor:
    """Logits [len(tokens), vocab] of a sequence fed token by token (on top of ``seq`` if given)."""
    seq = seq or Sequence(cfg)
    return torch.stack([step_token(w, cfg, seq, int(t)) for t in tokens])


def greedy(w, cfg: dict, prompt: List[int], new_tokens: int) -> List[int]:
    seq = Sequence(cfg)
    logits = run_tokens(w, cfg, prompt, seq)
    out = []
    for _ in range(new_tokens):
        out.append(int(torch.argmax(logits[-1])))
        logits = run_tokens(w, cfg, out[-1:], seq)
    return out
