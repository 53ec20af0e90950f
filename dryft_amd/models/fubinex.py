"""Fubinex: from ``FubinexConfig`` to a model plan.

A decoder on a float32 residual stream that starts as the embedding times a factor, with a norm in front of every
sublayer and none behind it: ``x <- x + mixer(norm1(x))``, ``x <- x + ff(norm2(x))``. The norm is an rms norm taken in
``norm.groups`` equal consecutive parts of the vector. A layer's mixer is one of three kinds:

* ``parallel``: two mixers on the same input, each output times a number of its own. On the left grouped-query
  attention over chunks (a row sees the earlier keys of its own run of ``mask.size`` positions, counted from position
  0), with a partial rotation over halves after which q and k are divided by their root mean square per head; on the
  right gated linear attention: a matrix state per head with a decay per key channel and token,
  ``sigmoid(z)^(1 / tau)`` with ``z`` from a low-rank projection, read out with one norm weight for all heads and gated
  by ``silu``;
* ``retention``: linear attention with a fixed decay per head, q and k rotated over halves;
* ``latent_attention``: queries and keys/values through normed low-rank latents, one rotated key part shared by all
  heads (neighbouring features turn together, frequencies stretched as in YaRN), causal. The latent and the rotated
  key part are what the cache holds. A layer with ``kv_from`` has neither projection nor cache of its own: it reads
  the line that the earlier layer writes, with its own projections from the latent to keys and values.

The feed-forward is ``down(act(up h))`` with a polynomial of the vector and its element-wise powers, each normed over
the vector; a layer may have none. A final norm of the same kind, and an output head of its own. Checkpoint names:
``embed``, ``head``, ``final.norm`` and per layer ``l<i>.norm1``, ``norm2``, ``l<i>.mix.*`` (``left.*``, ``right.*`` in a
parallel layer), ``l<i>.mlp.*``.
"""

from __future__ import annotations

from ..config.fubinex import FubinexConfig
from ..config.plan import LayerSpec, ModelPlan, PartSpec, Run
from . import register_architecture


def _norm(cfg: FubinexConfig, name: str) -> PartSpec:
    return PartSpec("stream_rmsnorm", dict(size=cfg.width, eps=cfg.norm_eps, groups=cfg.norm_groups), {"weight": name})


def _position(positions: dict[str, PartSpec], kind: str, rot: dict | None) -> str | None:
    """The name of the tables for a rotation; layers with equal rotations share them."""
    if rot is None:
        return None
    spec = PartSpec(kind, dict(dims=rot["dims"], base=rot["base"], scaling=rot["scaling"]))
    name = next((n for n, s in positions.items() if s == spec), None)
    if name is None:
        name = f"rotary{len(positions)}"
        positions[name] = spec
    return name


_LEFT_NAMES = {"q_proj": "q", "k_proj": "k", "v_proj": "v", "o_proj": "o"}
_LINEAR_NAMES = {"q_proj": "q", "k_proj": "k", "v_proj": "v", "g_proj": "g", "o_proj": "o"}
_RIGHT_NAMES = {**_LINEAR_NAMES, "decay_down": "a1", "decay_up": "a2", "decay_bias": "a2.b", "out_norm": "norm"}
_LATENT_NAMES = {"q_down": "dq", "q_norm": "dq.norm", "q_up": "uq", "k_up": "uk", "v_up": "uv", "o_proj": "o"}
_OWN_LATENT_NAMES = {"kv_down": "dkv", "kv_norm": "dkv.norm"}


def _parallel(cfg: FubinexConfig, m: dict, p: str, positions: dict[str, PartSpec]) -> PartSpec:
    l, r = m["left"], m["right"]
    left = PartSpec(
        "gqa_attention",
        dict(hidden_size=cfg.width, num_heads=l["heads"], num_kv_heads=l["kv_heads"], head_dim=l["dim"], value_dim=l["vdim"],
             scale=l["scale"], positions=_position(positions, "half_rotary", l["rot"]), qk_unit_eps=cfg.norm_eps,
             chunk=l["mask"]["size"] if l["mask"] else None, float_weights=True, pad_pages=True))
    right = PartSpec(
        "linear_attention",
        dict(hidden_size=cfg.width, num_heads=r["heads"], key_dim=r["dim"], value_dim=r["vdim"], norm_eps=cfg.norm_eps,
             q_scale=r["dim"] ** -0.5, channel_decay=(r["decay_rank"] or -1, r["tau"]), out_norm=True))
    names = {"left." + k: p + "left." + v for k, v in _LEFT_NAMES.items()}
    names.update({"right." + k: p + "right." + v for k, v in _RIGHT_NAMES.items()})
    return PartSpec("parallel_mixers",
                    dict(hidden_size=cfg.width, branches={"left": left, "right": right}, norm_eps=cfg.norm_eps,
                         scales={"left": m["left_scale"], "right": m["right_scale"]}),
                    names)


def _retention(cfg: FubinexConfig, m: dict, p: str, positions: dict[str, PartSpec]) -> PartSpec:
    return PartSpec(
        "linear_attention",
        dict(hidden_size=cfg.width, num_heads=m["heads"], key_dim=m["dim"], value_dim=m["vdim"], norm_eps=cfg.norm_eps,
             k_scale=m["dim"] ** -0.5, head_decay=m["decay"], positions=_position(positions, "half_rotary", m["rot"])),
        {k: p + v for k, v in _LINEAR_NAMES.items()})


def _latent(cfg: FubinexConfig, m: dict, p: str, positions: dict[str, PartSpec], index: int) -> PartSpec:
    own = m["kv_from"] is None
    names = {**_LATENT_NAMES, **(_OWN_LATENT_NAMES if own else {})}
    return PartSpec(
        "cached_latent_attention",
        dict(hidden_size=cfg.width, num_heads=m["heads"], head_dim=m["dim"], rot_dim=m["rot_dim"], value_dim=m["vdim"],
             q_rank=m["q_rank"], kv_rank=m["kv_rank"], scale=m["scale"], norm_eps=cfg.norm_eps,
             positions=_position(positions, "pair_rotary", m["rot"]), own_latent=own,
             name=f"latent{index if own else m['kv_from']}"),
        {k: p + v for k, v in names.items()})


def fubinex_plan(cfg: FubinexConfig) -> ModelPlan:
    positions: dict[str, PartSpec] = {}
    layers, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer.mixer
        if layer.type == "parallel":
            mixer = _parallel(cfg, m, p + "mix.", positions)
        elif layer.type == "retention":
            mixer = _retention(cfg, m, p + "mix.", positions)
        else:
            mixer = _latent(cfg, m, p + "mix.", positions, i)
        parts = {"mixer_norm": _norm(cfg, p + "norm1"), "mixer": mixer}
        block = "pre_norm_mixer"
        if layer.mlp is not None:
            parts["ffn_norm"] = _norm(cfg, p + "norm2")
            parts["ffn"] = PartSpec("poly_norm_mlp", dict(hidden_size=cfg.width, intermediate_size=layer.mlp["ff"], eps=cfg.norm_eps),
                                    {"up_proj": p + "mlp.up", "down_proj": p + "mlp.down", "act": p + "mlp.act"})
            block = "pre_norm"
        layers.append(LayerSpec(block, parts))
        lender = m.get("kv_from")
        schedule.append(Run(i, i, True) if lender is None else Run(i, lender, False))
    return ModelPlan(
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        embedding=PartSpec("token_embedding", dict(vocab_size=cfg.vocab, hidden_size=cfg.width, scale=cfg.embedding_scale),
                           {"weight": "embed"}),
        layers=tuple(layers),
        schedule=tuple(schedule),
        final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("lm_head", dict(vocab_size=cfg.vocab, hidden_size=cfg.width), {"weight": "head"}),
        positions=positions,
        max_positions=None,
    )


register_architecture(FubinexConfig.architecture, FubinexConfig, fubinex_plan)
