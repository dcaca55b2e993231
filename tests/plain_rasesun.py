"""A plain, slow Rasesun in float64 on the CPU: one function per mechanism, written from the
equations, whole sequences at a time, with explicit loops over tokens where a mechanism is
recurrent.  It shares no code with the package; the tests compare the engine with it.

Notation: T tokens, h a sublayer's input [T, width]; weights are [out, in] and applied as x @ W.T.
``w`` maps tensor names to float64 tensors, ``pre`` is a prefix of tensor names ("l3.mix.").
``rnd`` rounds what the engine's bfloat16 mode hands to a matrix product or to the cache (identity: nothing is rounded).
"""

from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional

import torch

F = torch.float64


def identity(x):
    return x


def round_bf16(x: torch.Tensor) -> torch.Tensor:
    return x.to(torch.float32).to(torch.bfloat16).to(F)


def to64(tensors: Mapping[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    return {k: (v.to(F) if v.is_floating_point() else v) for k, v in tensors.items()}


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return rms_unit(x, eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-torch.abs(z))) + torch.clamp(z, min=0.0)


# ----------------------------------------------------------------------------- state-space mixer

def causal_convolution(u: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """u [T, C], taps [C, K] (the last column is the current token's), zeros before the start."""
    T, C = u.shape
    K = taps.shape[1]
    out = torch.zeros(T, C, dtype=F)
    for t in range(T):
        for j in range(K):
            s = t - (K - 1) + j
            if s >= 0:
                out[t] += taps[:, j] * u[s]
        out[t] += bias
    return out


def ssd_recurrence(x, B, C, dt, A_log, D) -> torch.Tensor:
    """x [T, heads, P], B, C [T, groups, N], dt [T, heads] (behind its softplus); a head's state S [N, P] is decayed by
    exp(-exp(A_log) dt), takes dt B x^T and is read by C; D x is added to the read-out."""
    T, H, P = x.shape
    G, N = B.shape[1], B.shape[2]
    out = torch.zeros(T, H, P, dtype=F)
    for hd in range(H):
        g = hd // (H // G)
        rate = math.exp(float(A_log[hd]))
        S = torch.zeros(N, P, dtype=F)
        for t in range(T):
            step = float(dt[t, hd])
            S = math.exp(-rate * step) * S + step * torch.outer(B[t, g], x[t, hd])
            out[t, hd] = S.T @ C[t, g] + D[hd] * x[t, hd]
    return out


def gated_part_norm(y, z, weight, parts: int, eps) -> torch.Tensor:
    """y silu(z), then each of ``parts`` equal stretches divided by its own root mean square, then the weight."""
    T, n = y.shape
    v = (y * silu(z)).view(T, parts, n // parts)
    return rms_unit(v, eps).reshape(T, n) * weight


def mamba2_mixer(h, w, pre, mixer, eps, rnd=identity):
    H, P, N, G = int(mixer["heads"]), int(mixer["vdim"]), int(mixer["state"]), int(mixer["groups"])
    T, inner = h.shape[0], H * P
    p = h @ w[pre + "in"].T
    z, xbc, dt = p[:, :inner], p[:, inner:2 * inner + 2 * G * N], p[:, 2 * inner + 2 * G * N:]
    u = silu(causal_convolution(xbc, w[pre + "conv"], w[pre + "conv.b"]))
    x, B, C = u[:, :inner].view(T, H, P), u[:, inner:inner + G * N].view(T, G, N), u[:, inner + G * N:].view(T, G, N)
    y = ssd_recurrence(x, B, C, softplus(dt + w[pre + "dt_bias"]), w[pre + "A_log"], w[pre + "D"])
    o = gated_part_norm(y.reshape(T, inner), z, w[pre + "norm"], int(mixer["norm_groups"]), eps)
    return rnd(o) @ w[pre + "o"].T


# ----------------------------------------------------------------------------- latent attention

def rotate_pairs(x: torch.Tensor, pos0: int, rot: Mapping) -> torch.Tensor:
    """x [T, heads, n]: elements 2i and 2i+1 of every head's first ``dims`` elements are turned by position * base^(-2i/dims)."""
    T = x.shape[0]
    dims = int(rot["dims"])
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F)
    ang = torch.arange(pos0, pos0 + T, dtype=F)[:, None] * f[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    out = x.clone()
    a, b = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = a * c - b * s
    out[..., 1:dims:2] = b * c + a * s
    return out


def window_attention(q, k, v, scale, window) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, V]; query i sees keys j with 0 <= i - j < window; ordinary softmax."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for hd in range(H):
        for i in range(T):
            lo = max(0, i - window + 1)
            s = (k[lo:i + 1, hd] @ q[i, hd]) * scale
            e = torch.exp(s - s.max())
            out[i, hd] = (e[:, None] * v[lo:i + 1, hd]).sum(0) / e.sum()
    return out


def latent_mixer(h, w, pre, mixer, eps, pos0=0, rnd=identity):
    H, D, R, V, L = (int(mixer[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    T = h.shape[0]
    cq = rnd(rms_norm(h @ w[pre + "dq"].T, w[pre + "dq.norm"], eps))
    q = (cq @ w[pre + "uq"].T).view(T, H, D + R)
    down = h @ w[pre + "dkv"].T
    c = rnd(rms_norm(down[:, :L], w[pre + "dkv.norm"], eps))
    kr = rnd(rotate_pairs(down[:, None, L:], pos0, mixer["rot"]))
    qr = rotate_pairs(q[..., D:], pos0, mixer["rot"])
    kn = (c @ w[pre + "uk"].T).view(T, H, D)
    v = (c @ w[pre + "uv"].T).view(T, H, V)
    o = window_attention(torch.cat([q[..., :D], qr], -1), torch.cat([kn, kr.expand(T, H, R)], -1), v, float(mixer["scale"]),
                         int(mixer["mask"]["size"]))
    o = o * torch.sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return rnd(o.reshape(T, -1)) @ w[pre + "o"].T


# ----------------------------------------------------------------------------- feed-forward

def xielu(z, act):
    p, q = softplus(act[0]), softplus(act[1])
    up = p * z * z + 0.5 * z
    down = (0.5 + q) * (torch.expm1(torch.clamp(z, max=0.0)) - z) + 0.5 * z
    return torch.where(z > 0, up, down)


def dense(h, w, pre, rnd=identity):
    return rnd(xielu(h @ w[pre + "up"].T, w[pre + "act"])) @ w[pre + "down"].T


def squared_relu(z):
    return torch.clamp(z, min=0.0) ** 2


def table_moe(h, tokens, w, pre, mlp, rnd=identity):
    """The token's row of the table names its experts; each weighs 1 / top."""
    top = int(mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens):
        for e in w[pre + "table"][int(tok)].tolist():
            a = rnd(squared_relu(h[t] @ w[f"{pre}e{int(e)}.up"].T))
            out[t] += (a @ w[f"{pre}e{int(e)}.down"].T) / top
    return out


# ----------------------------------------------------------------------------- the model

def layer_runs(cfg) -> List[int]:
    """The layers in the order they run."""
    n = len(cfg["layers"])
    loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    a, b, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    return list(range(a)) + list(range(a, b)) * times + list(range(b, n))


def forward(cfg, w, tokens, rnd=identity, stream_out: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence from its first token.  ``stream_out``: receives the stream after every layer run."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] * float(cfg["embedding"]["scale"])
    for i in layer_runs(cfg):
        L, pre = cfg["layers"][i], f"l{i}."
        h = rnd(rms_norm(x, w[pre + "norm1"], eps))
        mixer = mamba2_mixer if L["type"] == "mamba2" else latent_mixer
        x = x + rms_norm(mixer(h, w, pre + "mix.", L["mixer"], eps, rnd=rnd), w[pre + "norm1b"], eps)
        mlp = L.get("mlp")
        if mlp is not None:
            h = rnd(rms_norm(x, w[pre + "norm2"], eps))
            y = dense(h, w, pre + "mlp.", rnd) if mlp["kind"] == "dense" else table_moe(h, tokens, w, pre + "mlp.", mlp, rnd)
            x = x + rms_norm(y, w[pre + "norm2b"], eps)
        if stream_out is not None:
            stream_out.append(x.clone())
    z = rnd(rms_norm(x, w["final.norm"], eps)) @ w["head"].T
    cap = float(cfg["logit_softcap"])
    return cap * torch.tanh(z / cap)


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
