"""A plain, slow implementation of the Vabelorn decoder: whole sequences, no cache, one function per mechanism, in the dtype of the
tensors it is given (the tests hand it 64-bit copies of the weights).  It shares nothing with the package.

The design: token embedding; layers ``x <- x + norm1(mixer(x))``, ``x <- x + norm2(ff(x))`` (norms on the sublayers' outputs only), and after
them a per-layer token input, ``x <- x + norm(proj(gelu_tanh(gate x) * e))`` with ``e`` a slice of a second token table; two mixers
(RWKV-style time mixing with decays that depend on the token; grouped-query attention with normed queries and keys, frequencies stretched by
YaRN, normed and rotated values whose sum is turned back, and one added to the softmax's denominator); gated dense feed-forwards (silu) or
none; a final norm; the embedding table as the head, times a factor.

``forward(config, tensors, tokens, stored=None)`` returns ``(logits [T, vocab], the stream after every layer)``.  ``stored``: a function applied
to every tensor that separate kernels hand to each other in the engine (the yardstick of the bfloat16 engine's rounding).
"""
from __future__ import annotations

import math

import torch


def _same(x):
    return x


def rms(x, eps):
    """``x / sqrt(mean(x^2) + eps)`` over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------------------------------------- rotation

def plain_frequencies(dims: int, base: float):
    return [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]


def yarn_frequencies(dims: int, base: float, scaling: dict | None):
    """``(frequencies, magnitude)``: with ``scaling`` (``factor``, ``original``, ``fast``, ``slow``) frequency ``i`` is blended between itself (pairs that
    turn at least ``fast`` times over ``original`` positions) and itself over ``factor`` (pairs that turn at most ``slow`` times), linearly in
    ``i``, and cosine and sine are multiplied by the magnitude."""
    freqs = plain_frequencies(dims, base)
    if not scaling:
        return freqs, 1.0
    factor, original, fast, slow = (float(scaling[k]) for k in ("factor", "original", "fast", "slow"))

    def pair_of(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(float(base)))

    lo = max(math.floor(pair_of(fast)), 0)
    hi = min(math.ceil(pair_of(slow)), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_pairs(x, positions, freqs, magnitude=1.0, sign=1.0):
    """``x [T, heads, dim]``: of the first ``2 len(freqs)`` numbers of every head, the pair ``(2i, 2i + 1)`` turns by ``sign * position * freqs[i]``
    and is multiplied by ``magnitude``; the rest passes."""
    n = len(freqs)
    if n == 0:
        return x
    f = torch.tensor(freqs, dtype=x.dtype)
    a = sign * positions.to(x.dtype)[:, None, None] * f[None, None, :]
    c, s = torch.cos(a) * magnitude, torch.sin(a) * magnitude
    u, v, rest = x[..., 0: 2 * n: 2], x[..., 1: 2 * n: 2], x[..., 2 * n:]
    turned = torch.stack((u * c - v * s, v * c + u * s), dim=-1).flatten(-2)
    return torch.cat((turned, rest), dim=-1)


# ------------------------------------------------------------------------------------------------- mixers

def off_by_one_attention(q, k, v, scale):
    """Causal attention of one head, ``q, k [T, dim]``, ``v [T, vdim]``, with ``1 + sum exp(s)`` as the softmax's denominator."""
    T = q.shape[0]
    s = (q @ k.T) * scale
    s = s.masked_fill(torch.ones(T, T).triu(1).bool(), float("-inf"))
    top = torch.clamp(s.max(dim=-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - top)
    return (e / (torch.exp(-top) + e.sum(-1, keepdim=True))) @ v


def attention_mixer(h, w, m, eps, stored=_same):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q = stored(h @ w["q"].T).view(T, H, d)
    k = stored(h @ w["k"].T).view(T, G, d)
    v = stored(h @ w["v"].T).view(T, G, dv)
    q, k = rms(q, eps) * w["q.norm"], rms(k, eps) * w["k.norm"]
    rot = m.get("rot")
    base = 10000.0
    if rot:
        freqs, magnitude = yarn_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
        q, k = rotate_pairs(q, pos, freqs, magnitude), rotate_pairs(k, pos, freqs, magnitude)
        base = rot["base"]
    turn = plain_frequencies(dv, base) if rot else []
    v = rotate_pairs(rms(v, eps), pos, turn)
    q, k, v = stored(q), stored(k), stored(v)
    o = torch.stack([off_by_one_attention(q[:, n], k[:, n // (H // G)], v[:, n // (H // G)], m["scale"]) for n in range(H)], dim=1)
    o = rotate_pairs(o, pos, turn, sign=-1.0)
    return stored(o.reshape(T, H * dv)) @ w["o"].T


def token_shift(h, mu):
    """``h_t + (h_(t-1) - h_t) * mu``, with zeros before the first token."""
    before = torch.cat((torch.zeros_like(h[:1]), h[:-1]))
    return h + (before - h) * mu


def wkv_recurrence(r, k, v, decay, u):
    """``r, k, decay [T, heads, dim]``, ``v [T, heads, dim]``, ``u [heads, dim]``: per head ``o_t = (S + diag(u) k v^T)^T r``, then ``S <- diag(decay)
    S + k v^T``.  Returns the outputs and the last state."""
    T, H, d = r.shape
    S = torch.zeros(H, d, v.shape[2], dtype=r.dtype)
    out = []
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out.append(((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1))
        S = decay[t][:, :, None] * S + kv
    return torch.stack(out), S


def wkv_mixer(h, w, m, eps, stored=_same):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    mixed = {s: stored(token_shift(h, w[f"mu.{s}"])) for s in "rkvgw"}
    r, k, v = (stored(mixed[s] @ w[s].T).view(T, H, d) for s in "rkv")
    gate = silu(stored(mixed["g"] @ w["g"].T))
    decay = torch.exp(-torch.exp(torch.tanh(mixed["w"] @ w["w1"].T) @ w["w2"].T + w["w0"])).view(T, H, d)
    o, _ = wkv_recurrence(r, k, v, decay, w["u"])
    o = rms(o, eps).reshape(T, H * d) * w["norm"] * gate
    return stored(o) @ w["o"].T


# ------------------------------------------------------------------------------------------------- the rest of a layer

def gated_feed_forward(h, w, stored=_same):
    return stored(silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def side_input(x, e, w, eps, stored=_same):
    """What the per-layer token input adds to the stream ``x``; ``e [T, dim]``: the layer's slice of the tokens' rows."""
    g = stored(gelu_tanh(stored(x) @ w["gate"].T) * e)
    return rms(stored(g @ w["proj"].T), eps) * w["norm"]


def _below(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(config, tensors, tokens, stored=None):
    stored = stored or _same
    eps = config["norm"]["eps"]
    ids = torch.tensor(tokens)
    x = tensors["embed"][ids]
    side = tensors["side.embed"][ids] if "side.embed" in tensors else None
    after = []
    for i, layer in enumerate(config["layers"]):
        w = _below(tensors, f"l{i}.")
        mix = _below(w, "mix.")
        if layer["type"] == "wkv":
            y = wkv_mixer(x, mix, layer["mixer"], eps, stored)
        else:
            y = attention_mixer(stored(x), mix, layer["mixer"], eps, stored)
        x = x + rms(stored(y), eps) * w["norm1"]
        if layer.get("mlp"):
            x = x + rms(stored(gated_feed_forward(stored(x), _below(w, "mlp."), stored)), eps) * w["norm2"]
        if side is not None:
            n = config["token_side"]["dim"]
            x = x + side_input(x, side[:, i * n: (i + 1) * n], _below(w, "side."), eps, stored)
        after.append(x)
    h = stored(rms(x, eps) * tensors["final.norm"] * config["logit_scale"])
    return h @ tensors["embed"].T, after
