"""A plain, slow implementation of the Tilalorn decoder: whole sequences, no cache, one function per mechanism, in the dtype of the tensors it
is given (the tests hand it 64-bit copies of the weights).  It shares nothing with the package.

The design: token embedding; layers ``x <- x + m * mixer(norm1(x))``, ``x <- x + m * ff(norm2(x))`` with root-mean-square norms whose weight is
stored around zero; two mixers (attention over a cached latent with a rotated key part that all heads share, inside a window, its output
gated element by element; grouped-query attention without positions over all earlier keys, with biases, queries and keys of unit root mean
square, queries that grow with their position, capped scores, a gate per head, and layers that read an earlier layer's keys and values);
feed-forwards that are dense and gated (the tanh form of gelu) or routed over gated experts (silu) in groups; a final norm and the embedding
table as the head.

``forward(config, tensors, tokens, stored=None, gaps=None)`` returns ``(logits [T, vocab], the stream after every layer)``.  ``stored``: a
function applied to every tensor that separate kernels hand to each other in the engine (the yardstick of the bfloat16 engine's rounding).
``gaps``: a list that receives every router's margin of choice, token by token.
"""
from __future__ import annotations

import math

import torch


def _same(x):
    return x


def rms(x, eps):
    """``x / sqrt(mean(x^2) + eps)`` over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_rms_norm(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z * z * z)))


def silu(z):
    return z / (1.0 + torch.exp(-z))


# ------------------------------------------------------------------------------------------------- masks, positions

def mask_matrix(T: int, window: int | None, dtype=torch.float64):
    """``[T, T]``: 0 where the query of the row reads the key of the column, minus infinity elsewhere: keys that are not later and, with a
    window, lie fewer than ``window`` positions back."""
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    seen = back >= 0
    if window is not None:
        seen &= back < window
    return torch.where(seen, 0.0, float("-inf")).to(dtype)


def rotate_halves(x, positions, dims: int, base: float):
    """``x [T, ..., n]``: of the first ``dims`` numbers, number ``i`` and number ``i + dims / 2`` turn by ``position * base ** (-2 i / dims)``."""
    half = dims // 2
    out = x.clone()
    for i in range(half):
        a = positions.to(x.dtype) * float(base) ** (-2.0 * i / dims)
        a = a.reshape(-1, *([1] * (x.dim() - 2)))
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def query_temperature(positions, coef: float, every: int, dtype=torch.float64):
    """``1 + coef * ln(floor((p + 1) / every) + 1)`` at every position."""
    return 1.0 + coef * torch.log(((positions + 1) // every + 1).to(dtype))


def soft_cap(s, cap: float | None):
    return s if cap is None else cap * torch.tanh(s / cap)


# ------------------------------------------------------------------------------------------------- mixers

def latent_attention_mixer(h, w, m, eps, stored=_same):
    """``q = W_q h`` (per head ``dim`` plain and ``rot_dim`` rotated numbers); ``W_dkv h`` gives the latent ``c`` (normed, a plain weight) and one
    rotated key part; per head ``k = W_uk c``, ``v = W_uv c``; score ``(q . k + q_rot . k_rot) * scale`` inside the window; the heads side by side
    times ``sigmoid(W_g h)``; ``W_o``."""
    T = h.shape[0]
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    turn = lambda x: rotate_halves(x, pos, m["rot"]["dims"], m["rot"]["base"])
    q = stored(h @ w["q"].T).view(T, H, d + r)
    down = stored(h @ w["dkv"].T)
    c = stored(rms(down[:, :rank], eps) * w["dkv.norm"])
    k_rot = stored(turn(down[:, rank:]))
    q_rot = stored(turn(q[..., d:]))
    k = (c @ w["uk"].T).view(T, H, d)
    v = (c @ w["uv"].T).view(T, H, dv)
    mask = mask_matrix(T, (m.get("mask") or {}).get("size"), h.dtype)
    heads = []
    for n in range(H):
        s = (q[:, n, :d] @ k[:, n].T + q_rot[:, n] @ k_rot.T) * m["scale"]
        heads.append(torch.softmax(s + mask, dim=-1) @ v[:, n])
    out = torch.cat(heads, dim=-1) * torch.sigmoid(stored(h @ w["g"].T))
    return stored(out) @ w["o"].T


def keys_and_values(h, w, m, eps, stored=_same):
    """The keys (of unit root mean square per head) and values of an attention layer, ``[T, kv_heads, dim]`` and ``[T, kv_heads, vdim]``."""
    T, G = h.shape[0], m["kv_heads"]
    k = stored(rms(stored(h @ w["k"].T + w["k.b"]).view(T, G, m["dim"]), eps))
    v = stored(h @ w["v"].T + w["v.b"]).view(T, G, m["vdim"])
    return k, v


def attention_mixer(h, w, m, eps, kv, stored=_same):
    """``kv``: the keys and values it reads (its own or another layer's).  ``q = rms(W_q h + b_q)`` per head, times the temperature of its
    position; ``score = cap(q . k * scale)``; head ``n``'s output times ``sigmoid(W_g h)[n]``; ``W_o``."""
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    k, v = kv
    q = rms(stored(h @ w["q"].T + w["q.b"]).view(T, H, d), eps)
    if m.get("q_temp"):
        q = q * query_temperature(torch.arange(T), m["q_temp"]["coef"], m["q_temp"]["every"], h.dtype)[:, None, None]
    q = stored(q)
    gate = torch.sigmoid(stored(h @ w["g"].T))
    mask = mask_matrix(T, None, h.dtype)
    heads = []
    for n in range(H):
        g = n // (H // G)
        s = soft_cap(q[:, n] @ k[:, g].T * m["scale"], m.get("softcap"))
        heads.append(torch.softmax(s + mask, dim=-1) @ v[:, g] * gate[:, n: n + 1])
    return stored(torch.cat(heads, dim=-1)) @ w["o"].T


# ------------------------------------------------------------------------------------------------- feed-forwards

def gated_ff(h, w, prefix, act, stored=_same):
    return stored(act(h @ w[prefix + "gate"].T) * (h @ w[prefix + "up"].T)) @ w[prefix + "down"].T


def grouped_router(h, w, router: dict, gaps=None):
    """``s = softmax(W_r h)``.  With ``E`` experts, expert ``e`` belongs to group ``e // (E / count)``; the ``keep`` groups with the largest maxima of ``s``
    stay open, the ``top`` largest ``s`` among their experts are picked (the lower index wins a tie), and a pick weighs ``s * scale``.  Returns ``(chosen [T, top], weights [T, top])``.  ``gaps``: a list that receives, per token, the smallest ratio by which
    a choice (of a group, of an expert) leads what it leaves out."""
    s = torch.softmax(h @ w["router"].T, dim=-1)
    groups = router.get("groups") or {"count": 1, "keep": 1}
    count, keep = groups["count"], groups["keep"]
    size = s.shape[1] // count
    chosen, weights = [], []
    for row in s:
        best = [max(row[g * size: (g + 1) * size].tolist()) for g in range(count)]
        order = sorted(range(count), key=lambda g: (-best[g], g))
        allowed = [e for g in order[:keep] for e in range(g * size, (g + 1) * size)]
        ranked = sorted(allowed, key=lambda e: (-row[e].item(), e))
        picks = ranked[: router["top"]]
        if gaps is not None:
            gap = float("inf")
            if keep < count:
                gap = min(gap, math.log(best[order[keep - 1]] / best[order[keep]]))
            if router["top"] < len(ranked):
                gap = min(gap, math.log(row[picks[-1]].item() / row[ranked[router["top"]]].item()))
            gaps.append(gap)
        chosen.append(picks)
        weights.append([row[e].item() * router.get("scale", 1.0) for e in picks])
    return torch.tensor(chosen), torch.tensor(weights, dtype=h.dtype)


def routed_ff(h, w, mlp, stored=_same, gaps=None):
    chosen, weights = grouped_router(h, w, mlp["router"], gaps)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(chosen.shape[1]):
            out[t] = out[t] + weights[t, j] * stored(gated_ff(h[t: t + 1], w, f"e{int(chosen[t, j])}.", silu, stored))[0]
    return out


# ------------------------------------------------------------------------------------------------- the model

def under(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(config, tensors, tokens, stored=_same, gaps=None):
    eps, m = float(config["norm"]["eps"]), float(config["residual_mult"])
    x = tensors["embed"][torch.as_tensor(tokens)]
    after, kv = [], {}
    for i, layer in enumerate(config["layers"]):
        w = under(tensors, f"l{i}.")
        h = stored(offset_rms_norm(x, w["norm1"], eps))
        mix, spec = under(w, "mix."), layer["mixer"]
        if layer["type"] == "latent_attention":
            y = latent_attention_mixer(h, mix, spec, eps, stored)
        elif layer["type"] == "attention":
            source = spec.get("kv_from")
            if source is None:
                kv[i] = keys_and_values(h, mix, spec, eps, stored)
            y = attention_mixer(h, mix, spec, eps, kv[i if source is None else source], stored)
        else:
            raise ValueError(layer["type"])
        x = x + m * stored(y)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = stored(offset_rms_norm(x, w["norm2"], eps))
            ff = under(w, "mlp.")
            y = gated_ff(h, ff, "", gelu_tanh, stored) if mlp["kind"] == "dense" else routed_ff(h, ff, mlp, stored, gaps)
            x = x + m * stored(y)
        after.append(x.clone())
    h = stored(offset_rms_norm(x, tensors["final.norm"], eps))
    return h @ tensors["embed"].T, torch.stack(after)
