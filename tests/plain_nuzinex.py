"""A plain, slow Nuzinex in float64 on the CPU: one function per mechanism, written from the
equations, whole sequences at a time, with explicit loops over tokens where a mechanism is
recurrent.  It shares no code with the package; the tests compare the engine with it.

Notation: T tokens, h a sublayer's input [T, width]; weights are [out, in] and applied as x @ W.T.
``w`` maps tensor names to float64 tensors, ``pre`` is a prefix of tensor names ("l3.mix.").
``rnd`` rounds what the engine's bfloat16 mode hands to a matrix product or to the cache (identity: nothing is rounded).
"""

from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional, Tuple

import torch

F = torch.float64
UNIT_EPS = 1e-6            # inside the root that makes the delta memory's queries and keys unit vectors


def identity(x):
    return x


def round_bf16(x: torch.Tensor) -> torch.Tensor:
    return x.to(torch.float32).to(torch.bfloat16).to(F)


def to64(tensors: Mapping[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    return {k: (v.to(F) if v.is_floating_point() else v) for k, v in tensors.items()}


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-torch.abs(z))) + torch.clamp(z, min=0.0)


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.special.erf(z / math.sqrt(2.0)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ----------------------------------------------------------------------------- attention

def rotate(x: torch.Tensor, pos0: int, rot: Mapping, interleaved: bool) -> torch.Tensor:
    """x [T, heads, n]: the first ``dims`` elements of every head are turned in pairs by position * base^(-2i/dims); pair i
    is elements (2i, 2i+1), or (i, i + dims/2)."""
    T, dims = x.shape[0], int(rot["dims"])
    out = x.clone()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        f = float(rot["base"]) ** (-2.0 * i / dims)
        ang = torch.arange(pos0, pos0 + T, dtype=F) * f
        c, s = torch.cos(ang)[:, None], torch.sin(ang)[:, None]
        out[..., a] = x[..., a] * c - x[..., b] * s
        out[..., b] = x[..., b] * c + x[..., a] * s
    return out


def softmax_attention(q, k, v, scale, window: Optional[int]) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, V]; query head h reads key head h // (H / G); query i sees keys j <= i, with a
    window only those with i - j < window."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for hd in range(H):
        g = hd // per
        for i in range(T):
            lo = 0 if window is None else max(0, i - window + 1)
            s = (k[lo:i + 1, g] @ q[i, hd]) * scale
            e = torch.exp(s - s.max())
            out[i, hd] = (e[:, None] * v[lo:i + 1, g]).sum(0) / e.sum()
    return out


def attention_queries(h, w, pre, m, eps, interleaved, pos0=0):
    q = h @ w[pre + "q"].T
    if pre + "q.b" in w:
        q = q + w[pre + "q.b"]
    q = rms_norm(q, w[pre + "q.norm"], eps).view(h.shape[0], int(m["heads"]), int(m["dim"]))
    return rotate(q, pos0, m["rot"], interleaved)


def attention_keys_values(h, w, pre, m, eps, interleaved, pos0=0) -> Tuple[torch.Tensor, torch.Tensor]:
    G, T = int(m["kv_heads"]), h.shape[0]
    k, v = h @ w[pre + "k"].T, h @ w[pre + "v"].T
    if pre + "k.b" in w:
        k, v = k + w[pre + "k.b"], v + w[pre + "v.b"]
    k = rms_norm(k, w[pre + "k.norm"], eps).view(T, G, int(m["dim"]))
    return rotate(k, pos0, m["rot"], interleaved), v.view(T, G, int(m["vdim"]))


def attention_mixer(h, w, pre, m, eps, interleaved=True, kv=None, rnd=identity):
    """Returns (output, (keys, values) as a cache holds them); ``kv``: another layer's, read instead of making its own."""
    q = rnd(attention_queries(h, w, pre, m, eps, interleaved))
    if kv is None:
        kv = tuple(rnd(t) for t in attention_keys_values(h, w, pre, m, eps, interleaved))
    window = None if m.get("mask") is None else int(m["mask"]["size"])
    o = rnd(softmax_attention(q, kv[0], kv[1], float(m["scale"]), window).reshape(h.shape[0], -1))
    if pre + "g" in w:
        o = rnd(o * torch.sigmoid(h @ w[pre + "g"].T))
    return o @ w[pre + "o"].T, kv


# ----------------------------------------------------------------------------- memories

def causal_convolution(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """u [T, C], taps [C, K] (the last column is the current token's), zeros before the start."""
    T, C = u.shape
    K = taps.shape[1]
    out = torch.zeros(T, C, dtype=F)
    for t in range(T):
        for j in range(K):
            s = t - (K - 1) + j
            if s >= 0:
                out[t] += taps[:, j] * u[s]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def delta_recurrence(q, k, v, g, beta) -> torch.Tensor:
    """q, k [T, Hk, D], v [T, H, V], g, beta [T, H]; head h uses q and k of head h // (H / Hk).  A head's S [D, V] is decayed
    by g, k's value in it is replaced towards v by beta, then q reads it."""
    T, H, V = v.shape
    per = H // q.shape[1]
    out = torch.zeros(T, H, V, dtype=F)
    for hd in range(H):
        S = torch.zeros(q.shape[2], V, dtype=F)
        for t in range(T):
            kt, qt = k[t, hd // per], q[t, hd // per]
            S = g[t, hd] * S
            u = beta[t, hd] * (v[t, hd] - S.T @ kt)
            S = S + torch.outer(kt, u)
            out[t, hd] = S.T @ qt
    return out


def delta_mixer(h, w, pre, m, eps, rnd=identity):
    H, Hk, D, V, T = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), h.shape[0]
    conv = lambda n: silu(causal_convolution(h @ w[pre + n].T, w[pre + n + ".conv"]))
    q = unit(conv("q").view(T, Hk, D)) * D ** -0.5
    k = unit(conv("k").view(T, Hk, D))
    v = conv("v").view(T, H, V)
    beta = torch.sigmoid(h @ w[pre + "b"].T)
    g = torch.exp(-torch.exp(w[pre + "A_log"]) * softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"]))
    o = rms_norm(delta_recurrence(q, k, v, g, beta), w[pre + "norm"], eps)
    o = o.reshape(T, H * V) * silu(h @ w[pre + "g"].T)
    return rnd(o) @ w[pre + "o"].T


def parallel_mixer(h, w, pre, m, eps, rnd=identity):
    left, _ = attention_mixer(h, w, pre + "left.", m["left"], eps, interleaved=False, rnd=rnd)
    right = delta_mixer(h, w, pre + "right.", m["right"], eps, rnd=rnd)
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


def fading_recurrence(q, k, v, decay) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, V], one constant decay a head: S <- decay S + k v^T, o = S^T q."""
    T, H, V = v.shape
    out = torch.zeros(T, H, V, dtype=F)
    for hd in range(H):
        S = torch.zeros(q.shape[2], V, dtype=F)
        for t in range(T):
            S = float(decay[hd]) * S + torch.outer(k[t, hd], v[t, hd])
            out[t, hd] = S.T @ q[t, hd]
    return out


def lightning_mixer(h, w, pre, m, eps, rnd=identity):
    H, D, V, T = int(m["heads"]), int(m["dim"]), int(m["vdim"]), h.shape[0]
    q, k, v = (silu(h @ w[pre + n].T).view(T, H, d) for n, d in (("q", D), ("k", D), ("v", V)))
    o = rms_norm(fading_recurrence(q, k, v, m["decay"]).reshape(T, H * V), w[pre + "norm"], eps)
    return rnd(o * torch.sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


# ----------------------------------------------------------------------------- the rest of a layer

def dense(h, w, pre, rnd=identity):
    return rnd(gelu_erf(h @ w[pre + "up"].T)) @ w[pre + "down"].T


def token_side(x, tokens, i: int, dim: int, w, pre, eps, rnd=identity):
    """What a token's own row of the side table adds to the stream behind layer i."""
    e = w["side.embed"][torch.as_tensor(list(tokens), dtype=torch.long)][:, i * dim:(i + 1) * dim]
    g = gelu_tanh(rnd(x) @ w[pre + "side.gate"].T) * e
    return rms_norm(rnd(g) @ w[pre + "side.proj"].T, w[pre + "side.norm"], eps)


def forward(cfg, w, tokens, rnd=identity, stream_out: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence from its first token.  ``stream_out``: receives the stream after every layer."""
    eps, dim = float(cfg["norm"]["eps"]), int(cfg["token_side"]["dim"])
    x = w["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    caches = {}
    for i, L in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", L["mixer"]
        if L["type"] == "attention":
            y, caches[i] = attention_mixer(rnd(x), w, pre + "mix.", m, eps, kv=caches.get(m.get("kv_from")), rnd=rnd)
        elif L["type"] == "parallel":
            y = parallel_mixer(rnd(x), w, pre + "mix.", m, eps, rnd)
        else:
            y = lightning_mixer(rnd(x), w, pre + "mix.", m, eps, rnd)
        x = x + rms_norm(y, w[pre + "norm1"], eps) * w[pre + "ls1"]
        if L.get("mlp") is not None:
            x = x + rms_norm(dense(rnd(x), w, pre + "mlp.", rnd), w[pre + "norm2"], eps) * w[pre + "ls2"]
        x = x + token_side(x, tokens, i, dim, w, pre, eps, rnd)
        if stream_out is not None:
            stream_out.append(x.clone())
    return rnd(rms_norm(x, w["final.norm"], eps)) @ w["head"].T


def generate_greedy(cfg, w, prompt, new_tokens: int) -> List[int]:
    """The whole sequence recomputed for every new token; the largest logit wins, the lower index among equals."""
    toks, out = list(prompt), []
    for _ in range(new_tokens):
        nxt = int(torch.argmax(forward(cfg, w, toks)[-1]))
        toks.append(nxt)
        out.append(nxt)
    return out


def logits_error(got, want, quantile: float = 1.0) -> float:
    """Per row: the root mean square of the difference (its mean taken off) over that of the wanted row (its mean taken
    off); the given quantile over the rows."""
    g, r = torch.as_tensor(got, dtype=F), torch.as_tensor(want, dtype=F)
    if not torch.isfinite(g).all():
        return math.inf
    d = g - r
    d = d - d.mean(-1, keepdim=True)
    c = r - r.mean(-1, keepdim=True)
    err = torch.sqrt((d * d).mean(-1)) / torch.sqrt((c * c).mean(-1)).clamp_min(1e-30)
    return float(torch.quantile(err, quantile))
