"""Plain, slow CPU implementation of the Fazolorn design: one function per mechanism, float64 by default.

It is the oracle the GPU kernels are tested against and shares no code with ``lit_gpt``. It takes the raw
``config.json`` dictionary and a ``{name: tensor}`` dictionary of weights, runs one sequence from position 0 and walks
it token by token where the design is recurrent; attention masks are written out as the set of keys a position sees.

The design in short. ``x = embed[token]``. Pre-norm layers: ``x += mixer(N1 x)``, then ``x += ff(N2 x)`` when the layer
has a feed-forward (RMS norms, plain weights). A range of layers runs several passes with the same weights: ahead of
pass t's first layer ``x += step[t]``, and for t > 0 the embedding output joins again, ``x += embed[token]``. Mixers:

* ``mingru`` - an elementwise gated recurrence whose gates read the token alone: ``S <- (1 - z) S + z c`` with
  ``z = sigmoid(W_z h + b_z)`` and a positive candidate ``c`` of ``W_x h + b_x``; the output is ``W_o (S * silu(W_g h))``.
* ``attention`` - biased queries and keys, rotary positions (half layout), aligned chunks of the sequence, the keys as
  projected for values, and in place of the softmax a sigmoid per key: weight ``sigmoid(score + pb[head])``.
* ``latent_attention`` - queries through a normed latent, keys and values expanded from a cached normed latent plus one
  shared rotated key part (interleaved layout, YaRN-rescaled frequencies and a factor on cos and sin), causal softmax.

Feed-forwards: dense ``W_down (g sigmoid(1.702 g) (u + 1))`` with clamped g and u, or a mixture of experts
``W_down (silu(W_gate h) * W_up h)`` whose router takes sigmoid scores, chooses groups of neighbouring experts first and
then the experts in them. Logits: a head matrix on the final norm, times a constant.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

DT = torch.float64


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


# ------------------------------------------------------------------------------------------------ rotation
def rot_frequencies(rot: Optional[dict]) -> Tuple[List[float], float]:
    """(frequencies of the rotated pairs, factor of cos and sin). With ``scaling`` the slow frequencies are divided by
    ``factor``, the fast ones kept, and the pairs between the two corner indices blend linearly. A corner is the index at
    which a pair makes t full turns over ``original`` positions: base^(-2i / dims) original = 2 pi t, solved for i."""
    if not rot or not int(rot.get("dims", 0)):
        return [], 1.0
    dims, base = int(rot["dims"]), float(rot["base"])
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return plain, 1.0
    factor, original = float(sc["factor"]), float(sc["original"])

    def corner(turns: float) -> float:
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(corner(float(sc["fast"]))), 0)
    hi = min(math.ceil(corner(float(sc["slow"]))), dims - 1)
    out = []
    for i, f in enumerate(plain):
        slow = min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001)))
        out.append(f / factor * slow + f * (1.0 - slow))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x: torch.Tensor, positions: List[int], freqs: List[float], layout: str, mult: float = 1.0) -> torch.Tensor:
    """x (T, heads, dim): pair number i of row t turns by positions[t] * freqs[i] and is multiplied by ``mult``. layout
    "half": pair (i, i + n), "interleaved": pair (2i, 2i + 1), n = len(freqs); the other dims pass as they are."""
    n = len(freqs)
    out = x.clone()
    for i, f in enumerate(freqs):
        a, b = (i, i + n) if layout == "half" else (2 * i, 2 * i + 1)
        ang = torch.tensor([p * f for p in positions], dtype=x.dtype).unsqueeze(-1)
        c, s = torch.cos(ang) * mult, torch.sin(ang) * mult
        u, v = x[..., a], x[..., b]
        out[..., a] = u * c - v * s
        out[..., b] = v * c + u * s
    return out


# ------------------------------------------------------------------------------------------------ mixers
def mingru_scan(z: torch.Tensor, u: torch.Tensor, state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """z, u (T, n): gate and candidate inputs as projected. Returns (S of every token (T, n), the last S)."""
    S = torch.zeros_like(z[0]) if state is None else state.clone()
    out = torch.zeros_like(z)
    for t in range(z.shape[0]):
        gate = torch.sigmoid(z[t])
        cand = torch.where(u[t] >= 0, u[t] + 0.5, torch.sigmoid(u[t]))
        S = (1.0 - gate) * S + gate * cand
        out[t] = S
    return out, S


def mingru(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    S, _ = mingru_scan(h @ w["z"].T + w["z.b"], h @ w["x"].T + w["x.b"])
    assert S.shape[1] == int(m["width"])
    return (S * silu(h @ w["g"].T)) @ w["o"].T


def visible(i: int, size: int) -> List[int]:
    """Keys that position i sees: those up to its own, in its own aligned chunk of ``size`` positions (0: no chunks)."""
    return [j for j in range(i + 1) if not size or i // size == j // size]


def sigmoid_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, size: int, pb: torch.Tensor) -> torch.Tensor:
    """q (T, H, d), k (T, G, d), v (T, G, dv) -> (T, H, dv): weights sigmoid(score + pb[h]), not normalised."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        js = visible(i, size)
        for h in range(H):
            g = h // (H // G)
            out[i, h] = torch.sigmoid((k[js, g] @ q[i, h]) * scale + pb[h]) @ v[js, g]
    return out


def attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    T = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q = (h @ w["q"].T + w["q.b"]).view(T, H, d)
    k = (h @ w["k"].T + w["k.b"]).view(T, G, d)
    f, mult = rot_frequencies(m.get("rot"))
    pos = list(range(T))
    o = sigmoid_attention(rotate(q, pos, f, "half", mult), rotate(k, pos, f, "half", mult), k, float(m["scale"]),
                          int((m.get("mask") or {}).get("size") or 0), w["pb"])
    return o.reshape(T, H * d) @ w["o"].T


def softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float) -> torch.Tensor:
    """q, k (T, H, d), v (T, H, dv) -> (T, H, dv), causal."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        for h in range(H):
            out[i, h] = torch.softmax((k[:i + 1, h] @ q[i, h]) * scale, -1) @ v[:i + 1, h]
    return out


def latent_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dr, dv, r = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).view(T, H, d + dr)
    ckr = h @ w["dkv"].T
    c = rms_norm(ckr[:, :r], w["dkv.norm"], eps)
    f, mult = rot_frequencies(m.get("rot"))
    pos = list(range(T))
    qr = rotate(q[..., d:], pos, f, "interleaved", mult)
    kr = rotate(ckr[:, r:].view(T, 1, dr), pos, f, "interleaved", mult)
    k = torch.cat([(c @ w["uk"].T).view(T, H, d), kr.expand(T, H, dr)], -1)
    v = (c @ w["uv"].T).view(T, H, dv)
    o = softmax_attention(torch.cat([q[..., :d], qr], -1), k, v, float(m["scale"]))
    return o.reshape(T, H * dv) @ w["o"].T


# ------------------------------------------------------------------------------------------------ feed-forwards
def clamped_feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], limit: float) -> torch.Tensor:
    g = (h @ w["gate"].T).clamp(max=limit)
    u = (h @ w["up"].T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def route(z: torch.Tensor, correction: torch.Tensor, top: int, count: int, keep: int, scale: float) -> Dict[int, float]:
    """One token's router outputs z (experts,) -> {chosen expert: weight}."""
    E = z.numel()
    s = torch.sigmoid(z)
    choice = (s + correction).tolist()
    per = E // count
    group = [sum(sorted(choice[g * per:(g + 1) * per], reverse=True)[:2]) for g in range(count)]
    kept = sorted(range(count), key=lambda g: -group[g])[:keep]
    allowed = [e for e in range(E) if e // per in kept]
    chosen = sorted(allowed, key=lambda e: -choice[e])[:top]
    return {e: float(s[e]) * scale for e in chosen}


def sparse_feed_forward(h: torch.Tensor, f: dict, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    r = f["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ w["router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        picks = route(z[t], w["correction"], int(r["top"]), int(groups["count"]), int(groups["keep"]), float(r.get("scale", 1.0)))
        for e, wt in picks.items():
            a = silu(h[t] @ w[f"e{e}.gate"].T) * (h[t] @ w[f"e{e}.up"].T)
            out[t] += wt * (a @ w[f"e{e}.down"].T)
    return out


# ------------------------------------------------------------------------------------------------ the model
def _sub(w: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def mixer(kind: str, h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    if kind == "mingru":
        return mingru(h, m, w)
    if kind == "attention":
        return attention(h, m, w)
    assert kind == "latent_attention", kind
    return latent_attention(h, m, w, eps)


def feed_forward(f: dict, h: torch.Tensor, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    return clamped_feed_forward(h, w, float(f["limit"])) if f["kind"] == "dense" else sparse_feed_forward(h, f, w)


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=DT, layers_out: Optional[list] = None
            ) -> torch.Tensor:
    """Logits (T, vocab) of one sequence from position 0. ``layers_out``: receives the residual after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    first = w["embed"][torch.tensor(tokens)]
    x = first
    n = len(config["layers"])
    loop = config.get("loop") or {"start": 0, "stop": 0, "times": 1}
    start, stop = int(loop["start"]), int(loop["stop"])

    def run(i: int, x: torch.Tensor) -> torch.Tensor:
        layer, lw = config["layers"][i], _sub(w, f"l{i}.")
        x = x + mixer(layer["type"], rms_norm(x, lw["norm1"], eps), layer["mixer"], _sub(lw, "mix."), eps)
        if layer.get("mlp"):
            x = x + feed_forward(layer["mlp"], rms_norm(x, lw["norm2"], eps), _sub(lw, "mlp."))
        if layers_out is not None:
            layers_out.append(x.clone())
        return x

    for i in range(start):
        x = run(i, x)
    for t in range(int(loop["times"]) if stop > start else 0):
        if t:
            x = x + first
        x = x + w["loop.step"][t]
        for i in range(start, stop):
            x = run(i, x)
    for i in range(stop, n):
        x = run(i, x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T * float(config.get("logit_scale", 1.0))
