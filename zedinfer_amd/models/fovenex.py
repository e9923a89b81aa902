"""Fovenex: the description of the design in parts.

A decoder whose layers are listed one by one in config.json, over several residual streams a token, all equal to the
embedding's row at first and added up before the final norm.  A sublayer reads one weighted sum of the streams through a
layer norm without bias; its result, times a gain per channel and a constant, goes back into all streams, which are mixed
with each other at the same time (hyper-connections).  The mixer is grouped-query attention whose heads are differences of two
softmax maps ("attention": normed and turned queries and keys, slowed frequencies, one gate a head), or windowed attention over
latents with query latents and an elementwise gate ("latent_attention": a layer may read the latents of an earlier one).
The feed-forward is dense with a tanh-form GELU and no gate, or absent.

Tensor names: ``embed``, ``l<i>.norm1`` / ``.norm2``, ``l<i>.ls1`` / ``.ls2``, ``l<i>.hc1`` / ``.hc2`` (``.in``, ``.out``,
``.mix`` added), ``l<i>.mix.q`` / ``.k`` / ``.v`` / ``.q.norm`` / ``.k.norm`` / ``.lq1`` / ``.lk1`` / ``.lq2`` / ``.lk2`` /
``.g`` / ``.o`` (attention), ``l<i>.mix.dq`` / ``.dq.norm`` / ``.uq`` / ``.dkv`` / ``.dkv.norm`` / ``.uk`` / ``.uv`` / ``.g`` /
``.o`` (latent attention), ``l<i>.mlp.up`` / ``.down``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from ..config.forward_config import LayerSpec, ModelForwardConfig, PartSpec, ScheduleStep
from ..config.model_config import FovenexConfig
from ..config.registry import register_architecture


def _mixer(cfg: FovenexConfig, i: int) -> PartSpec:
    layer, p, H = cfg.layers[i], f"l{i}.mix.", cfg.hidden_size
    m, window = layer["mixer"], int((layer["mixer"].get("mask") or {}).get("size", 0))
    rot = m.get("rot")
    if layer["type"] == "attention":
        position = PartSpec("none")
        if rot:
            position = PartSpec("rope_neox", {"head_dim": int(m["dim"]), "rotary_dim": int(rot["dims"]), "theta": float(rot["base"]),
                                              "scaling": dict(rot["scaling"]) if rot.get("scaling") else None})
        names = {x: p + x for x in ("q", "k", "v", "lq1", "lk1", "lq2", "lk2", "g", "o")}
        names.update({"q_norm": p + "q.norm", "k_norm": p + "k.norm"})
        return PartSpec(
            "difference_attention",
            {"hidden_size": H, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
             "value_dim": int(m["vdim"]), "scale": float(m["scale"]), "diff": float(m["diff"]), "eps": cfg.norm_eps, "window": window,
             "position": position, "qk_norm": True, "gate": True}, names)
    r = int(m["rot_dim"])
    shares = m.get("kv_from") is not None
    position = PartSpec("rope_pairs", {"head_dim": r, "rotary_dim": int(rot["dims"]), "theta": float(rot["base"]),
                                       "scaling": dict(rot["scaling"]) if rot.get("scaling") else None})
    names = {x: p + x for x in ("dq", "uq", "uk", "uv", "g", "o")}
    names["dq_norm"] = p + "dq.norm"
    if not shares:
        names.update({"dkv": p + "dkv", "dkv_norm": p + "dkv.norm"})
    return PartSpec(
        "latent_attention",
        {"hidden_size": H, "heads": int(m["heads"]), "dim": int(m["dim"]), "rot_dim": r, "vdim": int(m["vdim"]),
         "kv_rank": int(m["kv_rank"]), "scale": float(m["scale"]), "window": window, "eps": cfg.norm_eps, "shares_cache": shares,
         "q_rank": int(m["q_rank"]) if m.get("q_rank") is not None else -1, "gate": True, "pairing": "halves", "position": position},
        names)


def _norm(cfg: FovenexConfig, name: str) -> PartSpec:
    return PartSpec("layernorm", {"dim": cfg.hidden_size, "eps": cfg.norm_eps, "bias": False}, {"weight": name})


def _connection(cfg: FovenexConfig, i: int, q: int) -> PartSpec:
    """Of sublayer ``q`` (1: mixer, 2: feed-forward) of layer ``i``."""
    names = {x: f"l{i}.hc{q}.{x}" for x in ("in", "out", "mix")}
    names["scale"] = f"l{i}.ls{q}"
    return PartSpec("hyper", {"streams": cfg.streams, "hidden_size": cfg.hidden_size, "mult": cfg.residual_mult, "scale": True}, names)


def fovenex_forward_config(cfg: FovenexConfig) -> ModelForwardConfig:
    H = cfg.hidden_size
    layers, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        mlp, none = layer.get("mlp"), PartSpec("none")
        ff = none if mlp is None else PartSpec("activated_mlp", {"hidden_size": H, "intermediate_size": int(mlp["ff"]),
                                                                 "activation": "gelu_tanh"},
                                               {"up": f"l{i}.mlp.up", "down": f"l{i}.mlp.down"})
        layers.append(LayerSpec("connected", _mixer(cfg, i), ff,
                                {"input": _norm(cfg, f"l{i}.norm1"), "post_mixer": none if mlp is None else _norm(cfg, f"l{i}.norm2")},
                                {"mixer": _connection(cfg, i, 1), "feed_forward": none if mlp is None else _connection(cfg, i, 2)}))
        # a layer that reads another layer's latents runs on that layer's cache and stores nothing
        src = layer["mixer"].get("kv_from") if layer["type"] == "latent_attention" else None
        schedule.append(ScheduleStep(layer=i, cache=i if src is None else int(src), writes_cache=src is None))
    fc = ModelForwardConfig(
        architecture="Fovenex", hidden_size=H, vocab_size=cfg.vocab_size,
        embedding=PartSpec("token", {"vocab_size": cfg.vocab_size, "hidden_size": H}, {"weight": "embed"}),
        layers=tuple(layers), schedule=tuple(schedule), final_norm=_norm(cfg, "final.norm"),
        lm_head=PartSpec("linear", {"vocab_size": cfg.vocab_size, "hidden_size": H, "tied_to": None}, {"weight": "head"}),
        streams=cfg.streams, eos_token_ids=cfg.eos_token_ids, max_position_embeddings=0,
        # a layer without a feed-forward may still carry what would stand around it
        ignorable_tensors=tuple(f"l{i}.{n}" for i, layer in enumerate(cfg.layers) if layer.get("mlp") is None
                                for n in ("norm2", "ls2", "hc2.in", "hc2.out", "hc2.mix")),
        family={"mixers": [layer["type"] for layer in cfg.layers], "norm_eps": cfg.norm_eps})
    fc.validate()
    return fc


register_architecture("Fovenex", FovenexConfig, fovenex_forward_config, aliases=("fovenex",))
