"""A plain, slow implementation of the Narezen design in float64 on the CPU: one function per mechanism, written from the
equations in each docstring, sharing no code with the package.  A sequence is walked token by token; what a sequence
keeps between tokens is, per layer, a dict: an attention half's keys and values, a linear half's states, a recurrent
layer's state and its convolution's last inputs.

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


def rms_norm(v: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """unit_rms(v) * w."""
    return unit_rms(v, eps) * w


def sigmoid(v: torch.Tensor) -> torch.Tensor:
    return torch.exp(-torch.logaddexp(-v, torch.zeros_like(v)))


def silu(v: torch.Tensor) -> torch.Tensor:
    return v * sigmoid(v)


def softplus(v: torch.Tensor) -> torch.Tensor:
    """ln(1 + e^v)."""
    return torch.logaddexp(v, torch.zeros_like(v))


def gelu_tanh(v: torch.Tensor) -> torch.Tensor:
    """v/2 (1 + tanh(sqrt(2/pi) (v + 0.044715 v^3)))."""
    return 0.5 * v * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (v + 0.044715 * v ** 3)))


def rotate(v: torch.Tensor, pos: int, rot) -> torch.Tensor:
    """The first ``dims`` elements of the last dimension turned by the position, the rest as they are: the pair (i, i +
    dims/2), called (u, w), becomes (u cos a - w sin a, w cos a + u sin a) with a = pos * base^(-2i/dims)."""
    if not rot:
        return v
    dims, base = int(rot["dims"]), float(rot["base"])
    out = v.clone()
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        u, w = v[..., i], v[..., i + dims // 2]
        out[..., i] = u * math.cos(a) - w * math.sin(a)
        out[..., i + dims // 2] = w * math.cos(a) + u * math.sin(a)
    return out


def sunk_attention(qs: torch.Tensor, ks: torch.Tensor, vs: torch.Tensor, scale: float, sinks: torch.Tensor) -> torch.Tensor:
    """One token's queries [H, dim] over the kept keys [n, G, dim] and values [n, G, vdim]: for head g (key head g // (H/G))
    s_j = q_g . k_j * scale; sum_j e^(s_j) v_j / (sum_j e^(s_j) + e^(sinks[g])); the heads side by side."""
    per = qs.shape[0] // ks.shape[1]
    out = []
    for g in range(qs.shape[0]):
        s = ks[:, g // per] @ qs[g] * scale
        top = max(float(s.max()), float(sinks[g]))
        e = torch.exp(s - top)
        out.append(e @ vs[:, g // per] / (e.sum() + torch.exp(sinks[g] - top)))
    return torch.cat(out)


def tied_attention_token(w, p: str, m: dict, eps: float, h: torch.Tensor, kept: dict) -> torch.Tensor:
    """q = W_q h in H heads, k = W_k h in G heads, v = k; then q and k to unit_rms per head; no rotation; (k, v) is kept;
    attention with the learned sink of every head; W_o."""
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q, k = (w[p + ".q"] @ h).view(H, d), (w[p + ".k"] @ h).view(G, d)
    kept.setdefault("v", []).append(k)
    kept.setdefault("k", []).append(unit_rms(k, eps))
    o = sunk_attention(unit_rms(q, eps), torch.stack(kept["k"]), torch.stack(kept["v"]), float(m["scale"]), w[p + ".sink"])
    return w[p + ".o"] @ o


def plus_one_attention_token(w, p: str, m: dict, h: torch.Tensor, kept: dict, pos: int) -> torch.Tensor:
    """q = W_q h, k = W_k h, v = W_v h; q and k rotated; attention with one added to every head's sum (a sink of score
    zero); W_o."""
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    kept.setdefault("k", []).append(rotate((w[p + ".k"] @ h).view(G, d), pos, m.get("rot")))
    kept.setdefault("v", []).append((w[p + ".v"] @ h).view(G, dv))
    q = rotate((w[p + ".q"] @ h).view(H, d), pos, m.get("rot"))
    o = sunk_attention(q, torch.stack(kept["k"]), torch.stack(kept["v"]), float(m["scale"]), torch.zeros(H, dtype=F))
    return w[p + ".o"] @ o


def linear_state_step(S: torch.Tensor, a, q, k, v):
    """S <- diag(a) S + k v^T (a: a number, or one per row of S); returns (S, S^T q).  S: [dim, vdim]."""
    S = (a[:, None] if isinstance(a, torch.Tensor) and a.dim() == 1 else a) * S + torch.outer(k, v)
    return S, S.T @ q


def channel_decay_token(w, p: str, m: dict, eps: float, h: torch.Tensor, kept: dict) -> torch.Tensor:
    """q = W_q h * dim^(-1/2), k = W_k h, v = W_v h; a = sigmoid(W_a2 (W_a1 h) + a2.b)^(1/tau), one per head and key
    channel; linear_state_step per head; every head's result to unit_rms times ``norm``; the heads side by side times
    silu(W_g h); W_o."""
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q, k, v = (w[p + ".q"] @ h).view(H, d) * d ** -0.5, (w[p + ".k"] @ h).view(H, d), (w[p + ".v"] @ h).view(H, dv)
    z = w[p + ".a2"] @ (w[p + ".a1"] @ h) + w[p + ".a2.b"]
    a = torch.exp(-softplus(-z) / float(m["tau"])).view(H, d)
    S = kept.setdefault("S", [torch.zeros(d, dv, dtype=F) for _ in range(H)])
    out = []
    for i in range(H):
        S[i], o = linear_state_step(S[i], a[i], q[i], k[i], v[i])
        out.append(rms_norm(o, w[p + ".norm"], eps))
    return w[p + ".o"] @ (torch.cat(out) * silu(w[p + ".g"] @ h))


def retention_token(w, p: str, m: dict, eps: float, h: torch.Tensor, kept: dict, pos: int) -> torch.Tensor:
    """q = W_q h, k = W_k h, v = W_v h; q and k rotated, k then times dim^(-1/2); linear_state_step per head with its own
    constant decay; every head's result to unit_rms; the heads side by side times silu(W_g h); W_o."""
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = rotate((w[p + ".q"] @ h).view(H, d), pos, m.get("rot"))
    k = rotate((w[p + ".k"] @ h).view(H, d), pos, m.get("rot")) * d ** -0.5
    v = (w[p + ".v"] @ h).view(H, dv)
    S = kept.setdefault("S", [torch.zeros(d, dv, dtype=F) for _ in range(H)])
    out = []
    for i in range(H):
        S[i], o = linear_state_step(S[i], float(m["decay"][i]), q[i], k[i], v[i])
        out.append(unit_rms(o, eps))
    return w[p + ".o"] @ (torch.cat(out) * silu(w[p + ".g"] @ h))


def causal_conv(kept: List[torch.Tensor], now: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """b + sum_j w[:, j] * (input of taps - 1 - j tokens ago), the last column being the current token's; ``kept`` (oldest
    first, at most taps - 1 entries, missing ones are zeros) takes the current input in."""
    taps = w.shape[1]
    out = b + w[:, taps - 1] * now
    for back in range(1, taps):
        if back <= len(kept):
            out = out + w[:, taps - 1 - back] * kept[-back]
    kept.append(now)
    while len(kept) > taps - 1:
        kept.pop(0)
    return out


def rglru_gates(w, p: str, blocks: int, u: torch.Tensor):
    """u in ``blocks`` equal parts; part b: r_b = sigmoid(ra[b] u_b + ra.b[b]), i_b = sigmoid(ri[b] u_b + ri.b[b]); (r, i)."""
    out = []
    for t in ("ra", "ri"):
        out.append(torch.cat([sigmoid(w[f"{p}.{t}"][b] @ part + w[f"{p}.{t}.b"][b]) for b, part in enumerate(u.chunk(blocks))]))
    return out


def rglru_token(w, p: str, m: dict, h: torch.Tensor, kept: dict) -> torch.Tensor:
    """y = gelu_tanh(W_y h + y.b); u = causal_conv(W_x h + x.b); (r, i) = rglru_gates(u); log a = -8 r softplus(lam); S <-
    a S + sqrt(1 - a^2) i u; W_o (S * y)."""
    y = gelu_tanh(w[p + ".y"] @ h + w[p + ".y.b"])
    u = causal_conv(kept.setdefault("conv", []), w[p + ".x"] @ h + w[p + ".x.b"], w[p + ".conv"], w[p + ".conv.b"])
    r, i = rglru_gates(w, p, m["blocks"], u)
    log_a = -8.0 * r * softplus(w[p + ".lam"])
    S = kept.get("S", torch.zeros_like(u))
    kept["S"] = torch.exp(log_a) * S + torch.sqrt(-torch.expm1(2.0 * log_a)) * i * u
    return w[p + ".o"] @ (kept["S"] * y)


def glu_ff(w, p: str, h: torch.Tensor) -> torch.Tensor:
    """W_down (silu(W_gate h) * (W_up h))."""
    return w[p + ".down"] @ (silu(w[p + ".gate"] @ h) * (w[p + ".up"] @ h))


def routed_ff(w, p: str, mlp: dict, h: torch.Tensor) -> torch.Tensor:
    """s = sigmoid(W_router h); of the ``top`` experts with the largest s, the sum of expert(s h); plus shared(h)."""
    s = sigmoid(w[p + ".router"] @ h)
    out = torch.zeros_like(h)
    for e in torch.topk(s, mlp["router"]["top"]).indices.tolist():
        out = out + glu_ff(w, f"{p}.e{e}", s[e] * h)
    return out + glu_ff(w, p + ".shared", h) if mlp.get("shared") else out


class Sequence:
    """What one sequence keeps, per layer a dict for its mixer (of two halves: one each)."""

    def __init__(self, cfg: dict):
        self.mixer = [{"left": {}, "right": {}} for _ in cfg["layers"]]
        self.length = 0


def mixer_token(w, layer: dict, p: str, eps: float, h: torch.Tensor, kept: dict, pos: int) -> torch.Tensor:
    m = layer["mixer"]
    if layer["type"] == "rglru":
        return rglru_token(w, p, m, h, kept)
    l, r = m["left"], m["right"]
    if layer["type"] == "parallel":
        left = tied_attention_token(w, p + ".left", l, eps, h, kept["left"])
        right = channel_decay_token(w, p + ".right", r, eps, h, kept["right"])
    else:
        left = plus_one_attention_token(w, p + ".left", l, h, kept["left"], pos)
        right = retention_token(w, p + ".right", r, eps, h, kept["right"], pos)
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


def step_token(w: Dict[str, torch.Tensor], cfg: dict, seq: Sequence, token: int, streams: List = None) -> torch.Tensor:
    """One token: x = embed[token] * embedding.scale; per layer x <- x + norm1b(mixer(norm1(x))), x <- x + norm2b(ff(
    norm2(x))); logits = c tanh(head . final_norm(x) / c).  ``streams`` collects x after every layer."""
    eps, pos = float(cfg["norm"]["eps"]), seq.length
    x = w["embed"][token] * float(cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        y = mixer_token(w, layer, p + ".mix", eps, rms_norm(x, w[p + ".norm1"], eps), seq.mixer[i], pos)
        x = x + rms_norm(y, w[p + ".norm1b"], eps)
        if layer.get("mlp") is not None:
            y = routed_ff(w, p + ".mlp", layer["mlp"], rms_norm(x, w[p + ".norm2"], eps))
            x = x + rms_norm(y, w[p + ".norm2b"], eps)
        if streams is not None:
            streams.append(x)
    seq.length += 1
    c = float(cfg["logit_softcap"])
    return c * torch.tanh(w["head"] @ rms_norm(x, w["final.norm"], eps) / c)


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
