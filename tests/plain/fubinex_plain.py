"""A plain, slow Fubinex: one function per mechanism, written from the design's equations.

Everything is computed with dense score matrices and a loop over tokens, in the dtype of the tensors it is handed
(float64 in the tests). Nothing here is shared with the library: no kernel, no part, no cache. A mixer's function
takes the inputs of one sequence ``[T, width]`` and, optionally, what an earlier portion of the same sequence left
(``past``), and returns its outputs and what it leaves for the next portion.

Notation. ``rms(x) = x / sqrt(mean(x^2) + eps)``. Linear weights are ``[out, in]``. ``w`` is a dictionary of one
part's tensors by their short names (``"q"``, ``"a2.b"``, ...), ``c`` the part's entry of the configuration. Positions
count from 0 in every sequence; a portion's first position is the length of its past.
"""

from __future__ import annotations

import math

import torch


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, weight, groups, eps):
    """Each of ``groups`` equal consecutive parts of the vector divided by its own root mean square, the whole times a
    weight."""
    parts = [rms(p, eps) for p in x.chunk(groups, dim=-1)]
    return torch.cat(parts, -1) * weight


def silu(z):
    return z / (1 + torch.exp(-z))


# ------------------------------------------------------------------------------------------ rotations
def frequencies(rot):
    """``(f_i, factor on cos and sin)`` for i below dims/2; with ``scaling`` the stretched frequencies of YaRN."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=torch.float64), 1.0

    def dim_of(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(sc["factor"]) + 1.0


def _turns(pos, rot, x):
    f, both = frequencies(rot)
    a = pos.to(torch.float64)[:, None] * f[None, :]
    shape = (a.shape[0],) + (1,) * (x.dim() - 2) + (a.shape[1],)
    return (torch.cos(a) * both).reshape(shape).to(x.dtype), (torch.sin(a) * both).reshape(shape).to(x.dtype)


def rotate_halves(x, pos, rot):
    """``x [T, ..., D]``: entry ``i`` turns with entry ``i + dims/2``; entries from ``dims`` on pass."""
    if not rot:
        return x
    n = rot["dims"] // 2
    c, s = _turns(pos, rot, x)
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


def rotate_pairs(x, pos, rot):
    """``x [T, ..., D]``: entry ``2i`` turns with entry ``2i + 1``; entries from ``dims`` on pass."""
    if not rot:
        return x
    n = rot["dims"] // 2
    c, s = _turns(pos, rot, x)
    u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
    turned = torch.stack([u * c - v * s, v * c + u * s], -1).reshape(x.shape[:-1] + (2 * n,))
    return torch.cat([turned, x[..., 2 * n:]], -1)


# ------------------------------------------------------------------------------------------ attention
def causal_mask(pos_q, pos_k):
    return pos_k[None, :] <= pos_q[:, None]


def chunk_mask(pos_q, pos_k, size):
    """Row i sees key j <= i of its own chunk, chunks of ``size`` positions counted from position 0."""
    return causal_mask(pos_q, pos_k) & ((pos_q[:, None] // size) == (pos_k[None, :] // size))


def attend(q, k, v, mask, scale):
    """``q [Tq, H, D]``, ``k [Tk, G, D]``, ``v [Tk, G, Dv]`` -> ``[Tq, H, Dv]``; query head h reads head h // (H/G)."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        s = s.masked_fill(~mask, -math.inf)
        e = torch.exp(s - s.amax(-1, keepdim=True))
        out.append((e / e.sum(-1, keepdim=True)) @ v[:, g])
    return torch.stack(out, 1)


def chunked_attention(h, w, c, eps, past=None):
    """Grouped queries, a partial rotation over halves, then q and k divided by their root mean square per head; a
    row sees its own chunk."""
    H, G, D, Dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    T = h.shape[0]
    start = past["k"].shape[0] if past else 0
    pos = torch.arange(start, start + T)
    q, k, v = (h @ w["q"].T).view(T, H, D), (h @ w["k"].T).view(T, G, D), (h @ w["v"].T).view(T, G, Dv)
    q, k = rms(rotate_halves(q, pos, c.get("rot")), eps), rms(rotate_halves(k, pos, c.get("rot")), eps)
    if past:
        k, v = torch.cat([past["k"], k]), torch.cat([past["v"], v])
    keys = torch.arange(start + T)
    mask = chunk_mask(pos, keys, c["mask"]["size"]) if c.get("mask") else causal_mask(pos, keys)
    o = attend(q, k, v, mask, c["scale"])
    return o.reshape(T, H * Dv) @ w["o"].T, {"k": k, "v": v}


def latent_attention(h, w, c, eps, past=None, lent=None):
    """Queries through a normed latent; keys and values from a second normed latent ``c`` and one rotated key part
    ``r`` that all heads share. ``lent``: another layer's ``{"c", "r"}`` of every token so far, for a layer that has no
    latent of its own. Returns what the layer's own cache holds (or what it was lent)."""
    H, D, R, Dv = c["heads"], c["dim"], c["rot_dim"], c["vdim"]
    T = h.shape[0]
    if lent is not None:
        start = lent["c"].shape[0] - T
        cache = lent
    else:
        start = past["c"].shape[0] if past else 0
    pos = torch.arange(start, start + T)
    q = (rms(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T
    q = q.view(T, H, D + R)
    q_plain, q_rot = q[..., :D], rotate_pairs(q[..., D:], pos, c.get("rot"))
    if lent is None:
        down = h @ w["dkv"].T
        lat = rms(down[:, :c["kv_rank"]], eps) * w["dkv.norm"]
        rot = rotate_pairs(down[:, c["kv_rank"]:], pos, c.get("rot"))
        if past:
            lat, rot = torch.cat([past["c"], lat]), torch.cat([past["r"], rot])
        cache = {"c": lat, "r": rot}
    n = start + T
    k = torch.cat([(cache["c"] @ w["uk"].T).view(n, H, D), cache["r"][:, None, :].expand(n, H, R)], -1)
    v = (cache["c"] @ w["uv"].T).view(n, H, Dv)
    o = attend(torch.cat([q_plain, q_rot], -1), k, v, causal_mask(pos, torch.arange(n)), c["scale"])
    return o.reshape(T, H * Dv) @ w["o"].T, cache


# ------------------------------------------------------------------------------------------ linear attention
def linear_walk(q, k, v, decay, state):
    """Per head ``S <- diag(decay_t) S + k_t v_t^T``, ``o_t = S^T q_t`` with the new state. ``q, k, decay [T, H, D]``,
    ``v [T, H, Dv]``, ``state [H, D, Dv]``."""
    out = []
    for t in range(q.shape[0]):
        state = decay[t][:, :, None] * state + k[t][:, :, None] * v[t][:, None, :]
        out.append((state * q[t][:, :, None]).sum(1))
    return torch.stack(out), state


def gated_linear_attention(h, w, c, eps, past=None):
    """A decay per head, key channel and token, ``sigmoid(z)^(1/tau)``; the read-out normed per head with one weight
    for all heads, times ``silu`` of a gate."""
    H, D, Dv = c["heads"], c["dim"], c["vdim"]
    T = h.shape[0]
    q, k, v = (h @ w["q"].T).view(T, H, D) * D ** -0.5, (h @ w["k"].T).view(T, H, D), (h @ w["v"].T).view(T, H, Dv)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    decay = (1 / (1 + torch.exp(-z))) ** (1.0 / c["tau"])
    state = past["S"] if past else h.new_zeros(H, D, Dv)
    o, state = linear_walk(q, k, v, decay.view(T, H, D), state)
    o = rms(o, eps) * w["norm"]
    return (o.reshape(T, H * Dv) * silu(h @ w["g"].T)) @ w["o"].T, {"S": state}


def retention(h, w, c, eps, past=None):
    """A fixed decay per head; q and k rotated over halves, k scaled after that; the read-out divided by its root mean
    square per head, times ``silu`` of a gate."""
    H, D, Dv = c["heads"], c["dim"], c["vdim"]
    T = h.shape[0]
    start = past["n"] if past else 0
    pos = torch.arange(start, start + T)
    q = rotate_halves((h @ w["q"].T).view(T, H, D), pos, c.get("rot"))
    k = rotate_halves((h @ w["k"].T).view(T, H, D), pos, c.get("rot")) * D ** -0.5
    v = (h @ w["v"].T).view(T, H, Dv)
    decay = torch.tensor(c["decay"], dtype=h.dtype)[None, :, None].expand(T, H, D)
    state = past["S"] if past else h.new_zeros(H, D, Dv)
    o, state = linear_walk(q, k, v, decay, state)
    return (rms(o, eps).reshape(T, H * Dv) * silu(h @ w["g"].T)) @ w["o"].T, {"S": state, "n": start + T}


def parallel(h, w, c, eps, past=None):
    """Attention over chunks and gated linear attention side by side on the same input, each times a number."""
    past = past or {}
    left, past_l = chunked_attention(h, sub(w, "left."), c["left"], eps, past.get("left"))
    right, past_r = gated_linear_attention(h, sub(w, "right."), c["right"], eps, past.get("right"))
    return c["left_scale"] * left + c["right_scale"] * right, {"left": past_l, "right": past_r}


# ------------------------------------------------------------------------------------------ feed-forward
def poly_norm(z, act, eps):
    """``a N(z) + b N(z^2) + c N(z^3) + e`` with powers entry by entry and ``N`` the division by the vector's root mean
    square; ``act = (a, b, c, e)``."""
    a, b, c, e = act
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def feed_forward(h, w, eps):
    return poly_norm(h @ w["up"].T, w["act"], eps) @ w["down"].T


# ------------------------------------------------------------------------------------------ the model
def forward(cfg, t, tokens, past=None):
    """``(logits [T, vocab], stream after every layer [layers, T, width], past)`` of one portion of a sequence."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = t["embed"][torch.tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    new_past, streams = [], []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = group_norm(x, t[p + "norm1"], groups, eps)
        w, mine = sub(t, p + "mix."), past[i] if past else None
        if layer["type"] == "parallel":
            out, left = parallel(h, w, m, eps, mine)
        elif layer["type"] == "retention":
            out, left = retention(h, w, m, eps, mine)
        else:
            lent = new_past[m["kv_from"]] if m.get("kv_from") is not None else None
            out, left = latent_attention(h, w, m, eps, mine, lent)
        new_past.append(left)
        x = x + out
        if layer.get("mlp") is not None:
            x = x + feed_forward(group_norm(x, t[p + "norm2"], groups, eps), sub(t, p + "mlp."), eps)
        streams.append(x)
    return group_norm(x, t["final.norm"], groups, eps) @ t["head"].T, torch.stack(streams), new_past
