"""Kaditar: from ``KaditarConfig`` to a model plan.

A decoder on several copies of a float32 residual stream. A sublayer reads a learned weighted sum of the copies through
a layer norm (a weight and a bias), and its output goes back to all copies at once, which are mixed with one another by
a learned matrix on the way; the stream's value at the end is the sum of the copies. The mixer is differential
attention over a sliding window: two maps a head over the same values, of which the second is subtracted (weighed by
one learned number per layer) from the first, an rms norm without a weight on the difference; biases on q, k and v, a
rotation of neighbouring pairs on a part of every map. The feed-forward is a dense unit gated by relu, or routed
experts gated by silu: the largest router logits (with a bias) choose, the softmax over the chosen ones weighs, and a
shared expert is added times one sigmoid gate per token; a layer may have none. A run of layers may be looped: it
runs ``times`` times with the same weights, each pass with cache lines of its own. A final layer norm, the embedding
table as the output head, and logits capped with a tanh.

What the design fixes rather than the file: relu in the dense unit, silu in the experts. Checkpoint names: ``embed``,
``final.norm``, ``final.norm.b`` and per layer ``l<i>.norm1``, ``norm2`` (and ``.b``), ``l<i>.hc1.{in,out,mix}``, ``hc2.*``,
``l<i>.mix.*``, ``l<i>.mlp.*``.
"""

from __future__ import annotations

from ..config.base import layer_order
from ..config.kaditar import KaditarConfig
from ..config.plan import LayerSpec, ModelPlan, PartSpec, Run
from . import register_architecture


def _norm(cfg: KaditarConfig, name: str) -> PartSpec:
    return PartSpec("stream_layernorm", dict(size=cfg.width, eps=cfg.norm_eps, bias=True), {"weight": name, "bias": name + ".b"})


def _route(cfg: KaditarConfig, p: str) -> PartSpec:
    return PartSpec("stream_route", dict(streams=cfg.streams), {"read": p + "in", "write": p + "out", "mix": p + "mix"})


def _mixer(cfg: KaditarConfig, m: dict, p: str, positions: dict[str, PartSpec]) -> PartSpec:
    rot, name = m["rot"], None
    if rot is not None:
        spec = PartSpec("pair_rotary", dict(dims=rot["dims"], base=rot["base"]))
        name = next((n for n, s in positions.items() if s == spec), None)     # layers with equal rotations share tables
        if name is None:
            name = f"rotary{len(positions)}"
            positions[name] = spec
    return PartSpec(
        "differential_attention",
        dict(hidden_size=cfg.width, num_heads=m["heads"], num_kv_heads=m["kv_heads"], head_dim=m["dim"],
             value_dim=m["vdim"], scale=m["scale"], diff=m["diff"], norm_eps=cfg.norm_eps, positions=name,
             window=m["mask"]["size"] if m["mask"] else None),
        {"q_proj": p + "q", "k_proj": p + "k", "v_proj": p + "v", "o_proj": p + "o", "q_bias": p + "q.b",
         "k_bias": p + "k.b", "v_bias": p + "v.b", **{n: p + n for n in ("lq1", "lk1", "lq2", "lk2")}})


def _mlp(cfg: KaditarConfig, mlp: dict, p: str) -> PartSpec:
    if mlp["kind"] == "dense":
        return PartSpec("reglu", dict(hidden_size=cfg.width, intermediate_size=mlp["ff"]),
                        {"gate_proj": p + "gate", "up_proj": p + "up", "down_proj": p + "down"})
    r, shared = mlp["router"], mlp["shared"]
    names = {"router": p + "router", "router_bias": p + "router.b"}
    for e in range(r["experts"]):
        for t in ("gate", "up", "down"):
            names[f"e{e}_{t}"] = f"{p}e{e}.{t}"
    if shared:
        names.update({"shared_gate": p + "shared.gate", "shared_up": p + "shared.up", "shared_down": p + "shared.down",
                      "shared_weight": p + "shared.sg"})
    return PartSpec(
        "routed_experts",
        dict(hidden_size=cfg.width, experts=r["experts"], top=r["top"], intermediate_size=mlp["expert"]["ff"],
             shared=(shared["ff"],) if shared else None, unit="silu", score="chosen_softmax", correction=False,
             logit_bias=True),
        names)


def kaditar_plan(cfg: KaditarConfig) -> ModelPlan:
    positions: dict[str, PartSpec] = {}
    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        parts = {"mixer_route": _route(cfg, p + "hc1."), "mixer_norm": _norm(cfg, p + "norm1"),
                 "mixer": _mixer(cfg, layer.mixer, p + "mix.", positions)}
        block = "hyper_mixer"
        if layer.mlp is not None:
            parts.update({"ffn_route": _route(cfg, p + "hc2."), "ffn_norm": _norm(cfg, p + "norm2"),
                          "ffn": _mlp(cfg, layer.mlp, p + "mlp.")})
            block = "hyper"
        layers.append(LayerSpec(block, parts))
    order = layer_order(len(layers), cfg.loop)
    return ModelPlan(
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        embedding=PartSpec("token_embedding", dict(vocab_size=cfg.vocab, hidden_size=cfg.width), {"weight": "embed"}),
        layers=tuple(layers),
        schedule=tuple(Run(i, line, True) for line, (i, _) in enumerate(order)),     # a pass keeps lines of its own
        final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("lm_head", dict(vocab_size=cfg.vocab, hidden_size=cfg.width, softcap=cfg.logit_softcap),
                      {"weight": "embed"}),
        positions=positions,
        max_positions=None,
    )


register_architecture(KaditarConfig.architecture, KaditarConfig, kaditar_plan)
