"""Plain, slow CPU implementation of the Zaronex design: one function per mechanism, float64 by default.

It is the oracle the GPU kernels are tested against and shares no code with ``lit_gpt``. It takes the raw
``config.json`` dictionary and a ``{name: tensor}`` dictionary of weights, runs one sequence from position 0 and walks
it token by token wherever the design is recurrent; attention masks are written out as the set of keys a position sees.

The design in short. ``X_0 = embed[token]``. Layers are pre-norm, ``x += mixer(N1 x)``, then ``x += ff(N2 x)`` when the
layer has a feed-forward (RMS norms, plain weights). After layer ``i`` the residual that goes on is a learned average over
the depth: ``x = sum_{j <= i+1} dwa_i[j] X_j``, where ``X_(i+1)`` is layer ``i``'s own result. Mixers:

* ``parallel`` - *left*: biased projections, rotary positions (half layout), a window of the last ``size`` tokens plus
  one mean key and mean value per block of ``pool`` tokens that has left the window entirely, a learned sink per head,
  an elementwise sigmoid output gate. *right*: gated linear attention with a decay per key channel,
  ``S <- diag(alpha) S + k v^T``, ``alpha = sigmoid(low-rank(h) + b)^(1/tau)``.
* ``parallel_2`` - *left*: RMS norm over the whole q / k projection, rotary positions (interleaved layout, frequencies
  divided by a factor), values rotated by their position and outputs rotated back by the query's, a plain window.
  *right*: the selective scan with a diagonal state matrix per channel (Mamba), short convolution ahead of it.
* ``latent_attention`` - queries through a normed latent, keys and values expanded from a cached normed latent plus one
  shared rotated key part (interleaved), a plain window, an elementwise sigmoid output gate.

The two branches of a ``parallel`` mixer are each RMS-normed over the width and averaged. Feed-forward:
``W_down (gelu_tanh(W_gate h) * W_up h)``. Logits: a head matrix on the final norm.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

DT = torch.float64


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.logaddexp(z, torch.zeros_like(z))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms_norm(x: torch.Tensor, w: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def frequencies(dims: int, base: float, factor: float = 1.0) -> List[float]:
    return [base ** (-2.0 * i / dims) / factor for i in range(dims // 2)]


def rot_frequencies(rot: Optional[dict]) -> List[float]:
    if not rot or not int(rot.get("dims", 0)):
        return []
    return frequencies(int(rot["dims"]), float(rot["base"]), float((rot.get("scaling") or {}).get("factor", 1.0)))


def rotate(x: torch.Tensor, positions: List[int], freqs: List[float], layout: str, sign: float = 1.0) -> torch.Tensor:
    """x (T, heads, dim): the pair number i of row t turns by sign * positions[t] * freqs[i]. layout "half": pair
    (i, i + n), "interleaved": pair (2i, 2i + 1), n = len(freqs); the other dims pass."""
    n = len(freqs)
    out = x.clone()
    for i, f in enumerate(freqs):
        a, b = (i, i + n) if layout == "half" else (2 * i, 2 * i + 1)
        ang = torch.tensor([sign * p * f for p in positions], dtype=x.dtype).unsqueeze(-1)
        c, s = torch.cos(ang), torch.sin(ang)
        u, v = x[..., a], x[..., b]
        out[..., a] = u * c - v * s
        out[..., b] = v * c + u * s
    return out


def pooled_blocks(t: torch.Tensor, pool: int) -> torch.Tensor:
    """Means of the complete blocks of ``pool`` rows of t (T, ...)."""
    n = t.shape[0] // pool
    return torch.stack([t[b * pool:(b + 1) * pool].mean(0) for b in range(n)]) if n else t[:0]


def window_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, size: int = 0, pool: int = 0,
                     sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """q (T, H, d), k (T, G, d), v (T, G, dv) -> (T, H, dv). Position i sees the tokens j with 0 <= i - j < size (size
    0: all j <= i) and, with ``pool``, the mean key / value of every block b of pool tokens with
    b pool + pool - 1 <= i - size; exp(sink[h]) joins the denominator."""
    T, H, _ = q.shape
    G = k.shape[1]
    kb, vb = (pooled_blocks(k, pool), pooled_blocks(v, pool)) if pool else (k[:0], v[:0])
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        lo = max(0, i - size + 1) if size else 0
        seen = [b for b in range(kb.shape[0]) if b * pool + pool - 1 <= i - size]
        for h in range(H):
            g = h // (H // G)
            keys = torch.cat([kb[seen, g], k[lo:i + 1, g]])
            vals = torch.cat([vb[seen, g], v[lo:i + 1, g]])
            s = (keys @ q[i, h]) * scale
            top = s.max() if sink is None else torch.maximum(s.max(), sink[h])
            e = torch.exp(s - top)
            den = e.sum() + (torch.exp(sink[h] - top) if sink is not None else 0.0)
            out[i, h] = (e / den) @ vals
    return out


def pooled_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    """The left branch of ``parallel``."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    pos = list(range(T))
    q = (h @ w["q"].T + w["q.b"]).view(T, H, d)
    k = (h @ w["k"].T + w["k.b"]).view(T, G, d)
    v = (h @ w["v"].T + w["v.b"]).view(T, G, dv)
    f = rot_frequencies(m.get("rot"))
    q, k = rotate(q, pos, f, "half"), rotate(k, pos, f, "half")
    mask = m.get("mask") or {}
    o = window_attention(q, k, v, float(m["scale"]), int(mask.get("size") or 0), int(mask.get("pool") or 0), w["sink"])
    o = o.reshape(T, H * dv) * torch.sigmoid(h @ w["g"].T)
    return o @ w["o"].T


def gated_linear_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    """The right branch of ``parallel``."""
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ w["q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w["k"].T).view(T, H, d)
    v = (h @ w["v"].T).view(T, H, dv)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    alpha = torch.exp(-softplus(-z) / float(m["tau"])).view(T, H, d)
    S = torch.zeros(H, d, dv, dtype=h.dtype)
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        S = alpha[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        o[t] = (S * q[t].unsqueeze(-1)).sum(1)
    o = rms_norm(o, w["norm"], eps).reshape(T, H * dv) * silu(h @ w["g"].T)
    return o @ w["o"].T


def rotated_value_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    """The left branch of ``parallel_2``."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    pos = list(range(T))
    q = rms_norm(h @ w["q"].T, w["q.norm"], eps).view(T, H, d)
    k = rms_norm(h @ w["k"].T, w["k.norm"], eps).view(T, G, d)
    v = (h @ w["v"].T).view(T, G, dv)
    f = rot_frequencies(m.get("rot"))
    q, k = rotate(q, pos, f, "interleaved"), rotate(k, pos, f, "interleaved")
    fv = frequencies(dv, float(m["rot"]["base"]))
    v = rotate(v, pos, fv, "interleaved")
    mask = m.get("mask") or {}
    o = window_attention(q, k, v, float(m["scale"]), int(mask.get("size") or 0))
    o = rotate(o, pos, fv, "interleaved", sign=-1.0)
    return o.reshape(T, H * dv) @ w["o"].T


def causal_conv(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """x (T, C), w (C, taps): out[t] = b + sum_k w[:, taps - 1 - k] x[t - k], zeros before the start."""
    T, C = x.shape
    taps = w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        acc = b.clone()
        for k in range(min(taps, t + 1)):
            acc = acc + w[:, taps - 1 - k] * x[t - k]
        out[t] = acc
    return out


def channel_scan(x: torch.Tensor, dt: torch.Tensor, A: torch.Tensor, B: torch.Tensor, C: torch.Tensor, D: torch.Tensor,
                 state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """x, dt (T, inner), A (inner, N), B, C (T, N): S <- exp(dt A) S + dt x B, y = S C + D x. Returns (y, S)."""
    S = torch.zeros_like(A) if state is None else state.clone()
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t].unsqueeze(-1) * A) * S + (dt[t] * x[t]).unsqueeze(-1) * B[t]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    """The right branch of ``parallel_2``."""
    inner, N, rank = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
    xz = h @ w["in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, w["conv"], w["conv.b"]))
    p = x @ w["x"].T
    dt = softplus(p[:, :rank] @ w["dt"].T + w["dt.b"])
    y, _ = channel_scan(x, dt, -torch.exp(w["A_log"]), p[:, rank:rank + N], p[:, rank + N:], w["D"])
    return (y * silu(z)) @ w["o"].T


def latent_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dr, dv, r = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    pos = list(range(T))
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).view(T, H, d + dr)
    ckr = h @ w["dkv"].T
    c = rms_norm(ckr[:, :r], w["dkv.norm"], eps)
    f = rot_frequencies(m.get("rot"))
    kr = rotate(ckr[:, r:].view(T, 1, dr), pos, f, "interleaved")
    qr = rotate(q[..., d:], pos, f, "interleaved")
    k = torch.cat([(c @ w["uk"].T).view(T, H, d), kr.expand(T, H, dr)], -1)
    v = (c @ w["uv"].T).view(T, H, dv)
    mask = m.get("mask") or {}
    o = window_attention(torch.cat([q[..., :d], qr], -1), k, v, float(m["scale"]), int(mask.get("size") or 0))
    o = o.reshape(T, H * dv) * torch.sigmoid(h @ w["g"].T)
    return o @ w["o"].T


def _sub(w: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def mixer(kind: str, h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    if kind == "latent_attention":
        return latent_attention(h, m, w, eps)
    wl, wr = _sub(w, "left."), _sub(w, "right.")
    if kind == "parallel":
        left, right = pooled_attention(h, m["left"], wl), gated_linear_attention(h, m["right"], wr, eps)
    elif kind == "parallel_2":
        left, right = rotated_value_attention(h, m["left"], wl, eps), mamba(h, m["right"], wr)
    else:
        raise ValueError(kind)
    return 0.5 * (rms_norm(left, w["left.out"], eps) + rms_norm(right, w["right.out"], eps))


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def depth_average(results: List[torch.Tensor], weights: torch.Tensor) -> torch.Tensor:
    """sum_j weights[j] results[j] over the embedding output and the results of the layers so far."""
    assert weights.numel() == len(results)
    return sum(weights[j] * results[j] for j in range(len(results)))


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=DT, layers_out: Optional[list] = None
            ) -> torch.Tensor:
    """Logits (T, vocab) of one sequence from position 0. ``layers_out``: receives the averaged residual after every
    layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens)]
    results = [x]
    for i, layer in enumerate(config["layers"]):
        lw = _sub(w, f"l{i}.")
        x = x + mixer(layer["type"], rms_norm(x, lw["norm1"], eps), layer["mixer"], _sub(lw, "mix."), eps)
        if layer.get("mlp"):
            x = x + feed_forward(rms_norm(x, lw["norm2"], eps), _sub(lw, "mlp."))
        results.append(x)
        x = depth_average(results, lw["dwa"])
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T
