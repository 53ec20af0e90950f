"""A plain, slow Kaditar: one function per mechanism, written from the design's equations.

Everything is computed with dense score matrices in the dtype of the tensors it is handed, float64 in the tests.
Nothing here is shared with the library: no kernel, no part, no cache. ``forward`` takes the next tokens of one
sequence and, optionally, what an earlier portion left (the keys and values of every run of a layer), and returns
logits and the same afterwards.

Notation. Linear weights are ``[out, in]``. ``w`` is a dictionary of one part's tensors by their short names, ``c`` the
part's entry of the configuration.
"""

from __future__ import annotations

import torch


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------------------------------ differential attention
def rotate_pairs(x, pos, rot):
    """``x [T, ..., d]``: entries ``2i`` and ``2i + 1`` of the first ``dims`` turn together by ``pos * base^(-2i/dims)``."""
    if not rot or not rot["dims"]:
        return x
    n = rot["dims"] // 2
    angle = pos.to(x.dtype)[:, None] * rot["base"] ** (-2 * torch.arange(n, dtype=x.dtype) / rot["dims"])
    while angle.dim() < x.dim():
        angle = angle.unsqueeze(1)
    u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
    turned = torch.stack([u * angle.cos() - v * angle.sin(), v * angle.cos() + u * angle.sin()], -1)
    return torch.cat([turned.flatten(-2), x[..., 2 * n:]], -1)


def visible(rows, keys, window):
    """``[rows, keys]``: does the row at position i see the key at position j?"""
    back = rows[:, None] - keys[None, :]
    seen = back >= 0
    return seen & (back < window) if window else seen


def one_map(q, k, v, seen, scale):
    """Softmax attention of one head: ``q [T, d]``, ``k [n, d]``, ``v [n, dv]``."""
    score = (q @ k.T) * scale
    return torch.softmax(score.masked_fill(~seen, float("-inf")), -1) @ v


def difference(w, c):
    """The factor of the second map, one number for the layer."""
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + c["diff"]


def combine(a1, a2, lam, diff, eps):
    o = a1 - lam * a2
    return o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps) * (1 - diff)


def attention(h, w, c, eps, past=None):
    T, H, G, D, Dv = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    start = 0 if past is None else past[0].shape[0]
    pos = torch.arange(start, start + T)
    q = rotate_pairs((h @ w["q"].T + w["q.b"]).view(T, H, 2, D), pos, c.get("rot"))
    k = rotate_pairs((h @ w["k"].T + w["k.b"]).view(T, G, 2, D), pos, c.get("rot"))
    v = (h @ w["v"].T + w["v.b"]).view(T, G, Dv)
    if past is not None:
        k, v = torch.cat([past[0], k]), torch.cat([past[1], v])
    seen = visible(pos, torch.arange(k.shape[0]), (c.get("mask") or {}).get("size"))
    lam = difference(w, c)
    heads = []
    for a in range(H):
        g = a // (H // G)
        a1, a2 = (one_map(q[:, a, m], k[:, g, m], v[:, g], seen, c["scale"]) for m in (0, 1))
        heads.append(combine(a1, a2, lam, c["diff"], eps))
    return torch.cat(heads, -1) @ w["o"].T, (k, v)


# ------------------------------------------------------------------------------------------ feed-forwards
def glu(h, w, act, prefix=""):
    return (act(h @ w[prefix + "gate"].T) * (h @ w[prefix + "up"].T)) @ w[prefix + "down"].T


def dense(h, w):
    return glu(h, w, torch.relu)


def route(h, w, c):
    """``(chosen [T, top], weights [T, top])``."""
    best = (h @ w["router"].T + w["router.b"]).topk(c["router"]["top"], -1)
    return best.indices, torch.softmax(best.values, -1)


def moe(h, w, c):
    chosen, weights = route(h, w, c)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t].tolist(), weights[t]):
            out[t] += a * glu(h[t:t + 1], w, silu, f"e{e}.")[0]
    if c.get("shared"):
        out = out + torch.sigmoid(h @ w["shared.sg"].T) * glu(h, w, silu, "shared.")
    return out


# ------------------------------------------------------------------------------------------ the model
def part(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def order(cfg):
    """The layers as they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def mixed_streams(streams, hc, y):
    """Every copy from the old ones: ``mix`` is indexed ``[from, to]``."""
    n = len(streams)
    return [sum(hc["mix"][s, t] * streams[s] for s in range(n)) + hc["out"][t] * y for t in range(n)]


def capped(logits, cap):
    return cap * torch.tanh(logits / cap) if cap else logits


def forward(cfg, tensors, tokens, state=None, taps=None):
    """Logits ``[T, vocab]`` of one sequence's next ``tokens`` after what ``state`` holds (None: a new sequence),
    and the state afterwards. ``taps``: a list that receives the sum of the streams after every run of a layer."""
    eps, runs = cfg["norm"]["eps"], order(cfg)
    x0 = tensors["embed"][torch.as_tensor(tokens)]
    streams = [x0.clone() for _ in range(cfg["streams"])]
    state = list(state) if state is not None else [None] * len(runs)
    for r, i in enumerate(runs):
        layer = cfg["layers"][i]
        for q, kind in [(1, "mix")] + ([(2, "mlp")] if layer["mlp"] is not None else []):
            hc, w = part(tensors, f"l{i}.hc{q}."), part(tensors, f"l{i}.{kind}.")
            u = sum(hc["in"][s] * streams[s] for s in range(len(streams)))
            h = layer_norm(u, tensors[f"l{i}.norm{q}"], tensors[f"l{i}.norm{q}.b"], eps)
            if kind == "mix":
                y, state[r] = attention(h, w, layer["mixer"], eps, state[r])
            elif layer["mlp"]["kind"] == "dense":
                y = dense(h, w)
            else:
                y = moe(h, w, layer["mlp"])
            streams = mixed_streams(streams, hc, y)
        if taps is not None:
            taps.append(sum(streams))
    x = layer_norm(sum(streams), tensors["final.norm"], tensors["final.norm.b"], eps)
    return capped(x @ tensors["embed"].T, cfg.get("logit_softcap")), state
