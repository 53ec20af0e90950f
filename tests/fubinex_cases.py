"""Small Fubinex configurations with weights of the tests' own making.

The weights are drawn here, not by the library: matrices ``N(0, 1 / in)`` so that activations stay of order one, norm
weights around one, decays that span the range from "forgets at once" to "keeps everything", everything rounded to
bfloat16 so that both precisions read the same numbers.
"""

from __future__ import annotations

import json
import os

import torch
from safetensors.torch import save_file


def chunks(heads, kv_heads, dim, vdim, chunk=None, rot=None, base=1000.0, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5}
    if chunk:
        m["mask"] = {"size": chunk}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
    return m


def gated(heads, dim, vdim, rank, tau=16.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}


def parallel(left, right, left_scale=0.7, right_scale=1.1):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def retention(heads, dim, vdim, decay, rot=None, base=1000.0):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
    return {"type": "retention", "mixer": m}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, rot=None, base=1000.0, scaling=None, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
        if scaling:
            m["rot"]["scaling"] = scaling
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def with_ff(layer, ff=None):
    return {**layer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(width, vocab, layers, eps=1e-5, groups=1, embed=1.0):
    return {"architecture": "Fubinex", "vocab": vocab, "width": width, "embedding": {"scale": embed},
            "norm": {"eps": eps, "groups": groups}, "layers": [l if "mlp" in l else with_ff(l) for l in layers]}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}
# A: all kinds; heads of equal key and value width (the matrix cores' sizes) over chunks shorter than a page; a latent
# that the next layer and a later one read too; a layer without a feed-forward.
CASE_A = config(64, 200, [
    with_ff(parallel(chunks(4, 2, 32, 32, chunk=24, rot=16), gated(2, 16, 24, 5, tau=8.0)), 72),
    with_ff(latent(4, 16, 8, 40, 24, 32, rot=8, base=100.0, scaling=YARN), 96),
    retention(2, 16, 16, [0.9, 0.998], rot=16),
    with_ff(latent(2, 24, 8, 16, 20, 32, rot=8, base=100.0, scaling=YARN, kv_from=1), 40),
    with_ff(parallel(chunks(2, 1, 16, 48, chunk=65, rot=16), gated(3, 24, 16, 4)), 64),
    with_ff(latent(3, 8, 8, 24, 16, 32, rot=8, base=100.0, scaling=YARN, kv_from=1), 56)], groups=2, embed=3.0)
# B: sizes that are no multiples of 8; no chunks, no rotations; a norm in three parts; tau 1; decays that forget within a
# token or two; heads as many as key/value heads.
CASE_B = config(75, 131, [
    with_ff(latent(3, 12, 6, 20, 10, 14), 33),
    with_ff(parallel(chunks(3, 3, 20, 12), gated(3, 10, 6, 3, tau=1.0), 1.0, 1.0), 50),
    with_ff(retention(3, 20, 10, [0.02, 0.5, 1.0]), 21),
    with_ff(latent(5, 6, 6, 8, 12, 14, kv_from=0), 64)], eps=1e-6, groups=3)
# C: chunks of exactly a page and of more than one; more query heads than a tile of the matrix cores has columns; parts
# of a norm that are no multiples of 8 wide; rotations over part of a head; two latents, each read twice.
CASE_C = config(96, 300, [
    with_ff(parallel(chunks(6, 2, 32, 32, chunk=64, rot=8, base=1e4), gated(1, 40, 72, 7, tau=4.0), 0.5, -0.6), 112),
    with_ff(latent(20, 8, 16, 8, 32, 40, rot=16, base=5e3), 64),
    with_ff(latent(2, 32, 32, 64, 48, 24, rot=24, base=1e4, scaling={"factor": 2.0, "original": 32, "fast": 4.0, "slow": 0.5}), 48),
    with_ff(retention(4, 32, 64, [0.8, 0.97, 0.99, 0.9999], rot=20, base=1e5), 80),
    with_ff(latent(4, 16, 16, 16, 16, 40, rot=16, base=5e3, kv_from=1), 32),
    latent(6, 16, 32, 32, 16, 24, rot=24, base=1e4, scaling={"factor": 2.0, "original": 32, "fast": 4.0, "slow": 0.5}, kv_from=2),
    with_ff(parallel(chunks(4, 4, 48, 16, chunk=130, rot=48), gated(2, 8, 8, 2)), 40)], groups=8, embed=0.5)
CASES = {"A": CASE_A, "B": CASE_B, "C": CASE_C}


def tensors_for(cfg: dict, seed: int) -> dict[str, torch.Tensor]:
    """Every tensor the configuration names, as bfloat16-exact float32."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    out: dict[str, torch.Tensor] = {}

    def mat(name, o, i, gain=1.0):
        out[name] = gain * torch.randn(o, i, generator=g) / i ** 0.5

    def vec(name, n, mean=0.0, std=0.1):
        out[name] = mean + std * torch.randn(n, generator=g)

    def linear(p, m):
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        # a key leans on the query of its own token: q . k of a token stays away from zero, where the read-out, which is
        # divided by its own size, would turn on the last bit of either
        mat(p + "q", H * D, W, 1.4); mat(p + "k", H * D, W, 0.8); mat(p + "v", H * Dv, W, 1.4)
        out[p + "k"] += out[p + "q"]
        mat(p + "g", H * Dv, W, 2.0); mat(p + "o", W, H * Dv)

    out["embed"] = torch.randn(V, W, generator=g)
    mat("head", V, W, 2.0)
    vec("final.norm", W, 1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        vec(p + "norm1", W, 1.0)
        p += "mix."
        if layer["type"] == "parallel":
            l, r = m["left"], m["right"]
            mat(p + "left.q", l["heads"] * l["dim"], W, 1.4); mat(p + "left.k", l["kv_heads"] * l["dim"], W, 1.4)
            mat(p + "left.v", l["kv_heads"] * l["vdim"], W, 1.4); mat(p + "left.o", W, l["heads"] * l["vdim"])
            linear(p + "right.", r)
            mat(p + "right.a1", r["decay_rank"], W, 2.0); mat(p + "right.a2", r["heads"] * r["dim"], r["decay_rank"], 2.0)
            vec(p + "right.a2.b", r["heads"] * r["dim"], 1.0, 2.0)
            vec(p + "right.norm", r["vdim"], 1.0, 0.3)
        elif layer["type"] == "retention":
            linear(p, m)
        else:
            H, D, R, Dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
            mat(p + "dq", m["q_rank"], W, 2.0); vec(p + "dq.norm", m["q_rank"], 1.0, 0.3)
            mat(p + "uq", H * (D + R), m["q_rank"], 1.4)
            if m.get("kv_from") is None:
                mat(p + "dkv", m["kv_rank"] + R, W, 1.5); vec(p + "dkv.norm", m["kv_rank"], 1.0, 0.3)
            mat(p + "uk", H * D, m["kv_rank"], 1.4); mat(p + "uv", H * Dv, m["kv_rank"], 1.4)
            mat(p + "o", W, H * Dv)
        p = f"l{i}."
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            vec(p + "norm2", W, 1.0)
            mat(p + "mlp.up", ff, W, 1.2); mat(p + "mlp.down", W, ff)
            out[p + "mlp.act"] = torch.tensor([0.7, 0.5, -0.6, 0.1]) + 0.2 * torch.randn(4, generator=g)
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
    """A configuration drawn with ``rng`` (a ``random.Random``): sizes, head counts, the order of layers, chunks, decays,
    rotations, which layers read whose latent, and where feed-forwards sit all vary."""
    groups = rng.choice([1, 2, 3, 5])
    width = groups * rng.choice([16, 24, 31, 40])
    layers, lenders = [], []
    for i in range(rng.randrange(2, 7)):
        kind = rng.choice(["parallel", "retention", "latent_attention", "latent_attention"])
        if kind == "parallel":
            kv, dim = rng.choice([1, 2, 3]), rng.choice([8, 16, 32, 48, 64, 100])
            left = chunks(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([dim, 8, 40, 72]),
                          chunk=rng.choice([None, 1, 2, 17, 63, 64, 65, 128, 1000]), rot=rng.choice([None, 2, dim // 4 * 2, dim]),
                          base=rng.choice([100.0, 1e4]), scale=rng.choice([None, 0.3, 0.05]))
            right = gated(rng.choice([1, 2, 3]), rng.choice([8, 16, 30, 64]), rng.choice([8, 16, 50, 64]), rng.choice([1, 4, 16]),
                          tau=rng.choice([1.0, 2.5, 16.0]))
            layer = parallel(left, right, rng.choice([1.0, 0.3]), rng.choice([1.0, -0.8]))
        elif kind == "retention":
            heads, dim = rng.choice([1, 2, 3]), rng.choice([8, 16, 30, 64, 130])
            layer = retention(heads, dim, rng.choice([8, 16, 50, 96]), [rng.choice([0.01, 0.6, 0.97, 0.9995, 1.0]) for _ in range(heads)],
                              rot=rng.choice([None, 2, dim // 4 * 2, dim]), base=rng.choice([100.0, 1e4]))
        else:
            heads, dim, vdim, q_rank = rng.choice([1, 2, 3, 6, 17]), rng.choice([8, 16, 30]), rng.choice([8, 16, 40, 72]), rng.choice([16, 40])
            if lenders and rng.random() < 0.5:
                j = rng.choice(lenders)
                m = layers[j]["mixer"]
                rot = m.get("rot") or {}
                layer = latent(heads, dim, m["rot_dim"], vdim, q_rank, m["kv_rank"], rot=rot.get("dims"), base=rot.get("base", 1.0),
                               scaling=rot.get("scaling"), kv_from=j)
            else:
                rot_dim = rng.choice([4, 8, 16, 24])
                layer = latent(heads, dim, rot_dim, vdim, q_rank, rng.choice([12, 32, 70, 136]),
                               rot=rng.choice([None, 2, rot_dim // 4 * 2, rot_dim]), base=rng.choice([100.0, 1e4]),
                               scaling=rng.choice([None, {"factor": 4.0, "original": 32, "fast": 8.0, "slow": 1.0}]))
                lenders.append(i)
        layers.append(with_ff(layer, rng.choice([None, 8, 24, 67, 100])))
    return config(width, rng.randrange(100, 600), layers, eps=rng.choice([1e-6, 1e-5]), groups=groups, embed=rng.choice([1.0, 8.0]))
