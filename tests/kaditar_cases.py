"""Small Kaditar configurations with weights of the tests' own making.

The weights are drawn here, not by the library: matrices ``N(0, 1 / in)`` so that activations stay of order one, norm
weights around one and their biases around zero, the copies' mixing matrices near the unit matrix, the vectors behind the
maps' factor large enough that it moves, router biases that set the experts further apart than the tokens do (so that
few choices are a rounding apart), everything rounded to bfloat16 so that both precisions read the same numbers.
"""

from __future__ import annotations

import json
import os

import torch
from safetensors.torch import save_file


def attention(heads, kv_heads, dim, vdim, window=None, rot=None, base=1000.0, scale=None, diff=0.4):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff,
                      "mask": {"size": window} if window else None, "rot": {"dims": rot, "base": base} if rot else None,
                      "scale": scale if scale is not None else dim ** -0.5}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top},
            "shared": {"ff": shared} if shared else None}


def with_mlp(layer, mlp=None):
    return {**layer, "mlp": mlp}


def config(width, vocab, streams, layers, eps=1e-5, softcap=20.0, loop=None):
    return {"architecture": "Kaditar", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps},
            "logit_softcap": softcap, "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None,
            "layers": [l if "mlp" in l else with_mlp(l) for l in layers]}


# A: three copies; values twice as wide as a map's keys (nothing padded), a window shorter than a page and one a token
# longer than a page; both feed-forwards and a layer without one; layers 1 and 2 twice.
CASE_A = config(64, 200, 3, [
    with_mlp(attention(4, 2, 16, 32, window=20, rot=8), dense(96)),
    with_mlp(attention(2, 2, 24, 48, window=65, rot=24, base=1e5), moe(8, 3, 32, shared=40)),
    attention(6, 2, 8, 16, window=40, rot=2, base=200.0),
    with_mlp(attention(4, 1, 32, 64, window=64, rot=16), moe(6, 2, 24))], loop=(1, 3, 2))
# B: one copy; sizes that are no multiples of 8, values narrower than keys and wider than both maps; no window, no
# rotation, no cap; the whole model three times.
CASE_B = config(76, 131, 1, [
    with_mlp(attention(3, 3, 20, 12, rot=6, base=500.0, diff=0.0), moe(5, 5, 20, shared=12)),
    with_mlp(attention(4, 2, 13, 50, window=9, scale=0.5, diff=0.8), dense(70))], eps=1e-6, softcap=None, loop=(0, 2, 3))
# C: eight copies; one head; more than sixteen maps to a kv head; maps whose keys and values exceed what the matrix-core
# kernels take; a window of the row alone; one expert of many.
CASE_C = config(96, 300, 8, [
    with_mlp(attention(1, 1, 40, 80, window=130, rot=20), dense(33)),
    with_mlp(attention(18, 2, 8, 24, window=1, rot=8), dense(64)),
    with_mlp(attention(2, 1, 136, 40, window=70, rot=64, base=1e6), moe(1, 1, 48)),
    with_mlp(attention(2, 2, 16, 200, rot=16), moe(30, 1, 16, shared=24))], softcap=5.0)
CASES = {"A": CASE_A, "B": CASE_B, "C": CASE_C}


def tensors_for(cfg: dict, seed: int) -> dict[str, torch.Tensor]:
    """Every tensor the configuration names, as bfloat16-exact float32."""
    g = torch.Generator().manual_seed(seed)
    W, S = cfg["width"], cfg["streams"]
    out: dict[str, torch.Tensor] = {}

    def mat(name, o, i, gain=1.0):
        out[name] = gain * torch.randn(o, i, generator=g) / i ** 0.5

    def vec(name, n, mean=0.0, std=0.1):
        out[name] = mean + std * torch.randn(n, generator=g)

    def norm(name):
        vec(name, W, 1.0)
        vec(name + ".b", W, 0.0, 0.2)

    def glu(p, ff):
        mat(p + "gate", ff, W, 1.5); mat(p + "up", ff, W, 1.5); mat(p + "down", W, ff)

    out["embed"] = torch.randn(cfg["vocab"], W, generator=g)
    norm("final.norm")
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        for q in (1, 2) if layer["mlp"] is not None else (1,):
            norm(f"{p}norm{q}")
            vec(f"{p}hc{q}.in", S, 1.0 / S, 0.2)
            vec(f"{p}hc{q}.out", S, 0.7, 0.3)
            out[f"{p}hc{q}.mix"] = torch.eye(S) * 0.8 + 0.15 * torch.randn(S, S, generator=g)
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n, rows in (("q", 2 * H * D), ("k", 2 * G * D), ("v", G * Dv)):
            mat(p + "mix." + n, rows, W)
            vec(p + f"mix.{n}.b", rows, 0.0, 0.5)
        for n in ("lq1", "lk1", "lq2", "lk2"):
            vec(p + "mix." + n, D, 0.5 / D ** 0.5, 0.5 / D ** 0.5)
        mat(p + "mix.o", W, H * Dv)
        mlp = layer["mlp"]
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            glu(p + "mlp.", mlp["ff"])
            continue
        E = mlp["router"]["experts"]
        for e in range(E):
            glu(f"{p}mlp.e{e}.", mlp["expert"]["ff"])
        mat(p + "mlp.router", E, W, 0.7)
        vec(p + "mlp.router.b", E, 0.0, 2.0)
        if mlp["shared"]:
            glu(p + "mlp.shared.", mlp["shared"]["ff"])
            mat(p + "mlp.shared.sg", 1, W, 2.0)
    return {k: v.to(torch.bfloat16).to(torch.float32) for k, v in out.items()}


def write_dir(path: str, cfg: dict, tensors: dict[str, torch.Tensor]) -> str:
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()}, os.path.join(path, "model.safetensors"))
    return path


def double(tensors):
    return {k: v.double() for k, v in tensors.items()}


def random_config(rng) -> dict:
    """A configuration drawn with ``rng`` (a ``random.Random``): sizes, head counts, the order of layers and which of them
    repeat, where feed-forwards sit and of which kind, windows, rotations and the number of copies all vary."""
    layers = []
    for _ in range(rng.randrange(1, 6)):
        kv = rng.choice([1, 1, 2, 3, 4])
        dim = rng.choice([4, 7, 8, 16, 20, 24, 32, 64, 80, 128])
        rot = rng.choice([None, 2, dim // 2 // 2 * 2, dim // 2 * 2]) or None
        layer = attention(kv * rng.choice([1, 2, 3, 8]), kv, dim, rng.choice([8, dim, 2 * dim, 2 * dim, 72, 30, 256]),
                          window=rng.choice([None, 1, 2, 17, 63, 64, 65, 128, 129, 1000]), rot=rot,
                          base=rng.choice([100.0, 1e4, 1e6]), scale=rng.choice([None, 0.3, 0.05]), diff=rng.choice([0.0, 0.2, 0.5, 0.8]))
        kind = rng.choice(["none", "dense", "moe", "moe"])
        experts = rng.choice([1, 2, 3, 7, 16, 70])
        mlp = dense(rng.choice([48, 100, 256])) if kind == "dense" else \
            moe(experts, rng.randrange(1, min(experts, 6) + 1), rng.choice([8, 24, 64, 100]), shared=rng.choice([None, 16, 72])) \
            if kind == "moe" else None
        layers.append(with_mlp(layer, mlp))
    loop = None
    if rng.random() < 0.6:
        start = rng.randrange(len(layers))
        loop = (start, rng.randrange(start + 1, len(layers) + 1), rng.choice([1, 2, 3]))
    return config(rng.choice([64, 68, 90, 128, 192, 256, 320]), rng.randrange(100, 600), rng.choice([1, 2, 3, 4, 6]), layers,
                  eps=rng.choice([1e-6, 1e-5, 1e-3]), softcap=rng.choice([None, 4.0, 15.0, 50.0]), loop=loop)
