"""Kefisun: the description of the design in parts.

A decoder whose layers are listed one by one in config.json.  A layer is pre-norm, x <- x + mixer(h), x <- x + ff(n2(x)),
with RMS norms whose gain is stored around zero (1 + w); what the mixer reads is the normed stream plus a causal
convolution of it over time on each channel.  The mixer is grouped-query attention under a sliding window, without
rotation ("attention": q, k and v pass a short convolution, q and k an RMS norm over the whole projection, a
logarithm of the distance is taken off the scores, values are mixed with the first such layer's, a sigmoid gate
multiplies the heads), or the delta rule with a decay per key channel from a low-rank gate ("channel_delta").  The
feed-forward is dense, clamped and gated, with biases, or absent.  The embedding's rows are scaled; the logits are
the product with the unscaled table times a constant.

Tensor names: ``embed``, ``l<i>.norm1`` / ``.norm2`` / ``.canon1``, ``l<i>.mix.q`` / ``.k`` / ``.v`` (``.conv`` added,
for attention ``.norm`` at q and k too), ``l<i>.mix.vmix`` / ``.r1`` / ``.r2`` / ``.g`` / ``.o`` (attention),
``l<i>.mix.b`` / ``.A_log`` / ``.a1`` / ``.a2`` / ``.dt_bias`` / ``.g1`` / ``.g2`` / ``.norm`` / ``.o`` (channel_delta),
``l<i>.mlp.gate`` / ``.up`` / ``.down`` (``.b`` added), ``final.norm``.
"""
from __future__ import annotations

from ..config.forward_config import LayerSpec, ModelForwardConfig, PartSpec, default_schedule
from ..config.model_config import KefisunConfig
from ..config.registry import register_architecture


def _mixer(cfg: KefisunConfig, i: int) -> PartSpec:
    layer, p, H = cfg.layers[i], f"l{i}.mix.", cfg.hidden_size
    m = layer["mixer"]
    if layer["type"] == "attention":
        mask = m.get("mask") or {}
        mixing = cfg.value_mixing_layers()
        value_mix = None if i not in mixing else ("first" if i == mixing[0] else "mix")
        names = {"o": p + "o", "g": p + "g", "r1": p + "r1", "r2": p + "r2", "q_norm": p + "q.norm", "k_norm": p + "k.norm"}
        for x in ("q", "k", "v"):
            names.update({x: p + x, x + "_conv": p + x + ".conv"})
        if value_mix == "mix":
            names["vmix"] = p + "vmix"
        sub = PartSpec(
            "conv_attention",
            {"hidden_size": H, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
             "value_dim": int(m["vdim"]), "conv": int(m["conv"]), "scale": float(m["scale"]),
             "window": int(mask.get("size", 0) or 0), "eps": cfg.norm_eps, "position": PartSpec("none"), "bias": False,
             "sink": False, "log_distance": True, "gate": True, "value_mix": value_mix},
            names)
    else:
        names = {x: p + x for x in ("q", "k", "v", "b", "A_log", "a1", "a2", "dt_bias", "g1", "g2", "norm", "o")}
        names.update({x + "_conv": p + x + ".conv" for x in ("q", "k", "v")})
        sub = PartSpec(
            "channel_delta_rule",
            {"hidden_size": H, "heads": int(m["heads"]), "kv_heads": int(m["kv_heads"]), "dim": int(m["dim"]),
             "vdim": int(m["vdim"]), "conv": int(m["conv"]), "eps": cfg.norm_eps,
             "decay_rank": int(m.get("decay_rank", -1)), "gate_rank": int(m.get("gate_rank", -1))},
            names)
    return PartSpec("input_convolution", {"hidden_size": H, "taps": cfg.canon_taps, "mixer": sub},
                    {"taps": f"l{i}.canon1", **{f"mixer.{k}": v for k, v in sub.weights.items()}})


def _feed_forward(cfg: KefisunConfig, i: int) -> PartSpec:
    mlp, p = cfg.layers[i].get("mlp"), f"l{i}.mlp."
    if mlp is None:
        return PartSpec("none")
    names = {x: p + x for x in ("gate", "up", "down")}
    names.update({x + "_bias": p + x + ".b" for x in ("gate", "up", "down")})
    return PartSpec("clamped_mlp", {"hidden_size": cfg.hidden_size, "intermediate_size": int(mlp["ff"]),
                                    "limit": float(mlp["limit"]), "bias": True}, names)


def _norm(cfg: KefisunConfig, name: str, gain_scale: float = 1.0) -> PartSpec:
    return PartSpec("rmsnorm", {"dim": cfg.hidden_size, "eps": cfg.norm_eps, "add_one": True, "gain_scale": gain_scale},
                    {"weight": name})


def kefisun_forward_config(cfg: KefisunConfig) -> ModelForwardConfig:
    H = cfg.hidden_size
    layers = []
    for i, layer in enumerate(cfg.layers):
        has_ff = layer.get("mlp") is not None
        layers.append(LayerSpec("prenorm", _mixer(cfg, i), _feed_forward(cfg, i),
                                {"input": _norm(cfg, f"l{i}.norm1"),
                                 "post_mixer": _norm(cfg, f"l{i}.norm2") if has_ff else PartSpec("none")}))
    fc = ModelForwardConfig(
        architecture="Kefisun", hidden_size=H, vocab_size=cfg.vocab_size,
        embedding=PartSpec("token", {"vocab_size": cfg.vocab_size, "hidden_size": H, "scale": cfg.embedding_scale},
                           {"weight": "embed"}),
        layers=tuple(layers), schedule=default_schedule(len(layers)),
        # logits = (embed n(x)) * c = embed (n(x) * c): the constant is part of the last norm's gains
        final_norm=_norm(cfg, "final.norm", cfg.logit_scale),
        lm_head=PartSpec("linear", {"vocab_size": cfg.vocab_size, "hidden_size": H, "tied_to": None}, {"weight": "embed"}),
        tie_word_embeddings=True, eos_token_ids=cfg.eos_token_ids, max_position_embeddings=0,
        # the share of the first layer that mixes values is never used, and a layer without a feed-forward may still
        # carry its norm's gains
        ignorable_tensors=tuple(f"l{i}.mix.vmix" for i, layer in enumerate(cfg.layers) if layer["type"] == "attention") +
        tuple(f"l{i}.norm2" for i, layer in enumerate(cfg.layers) if layer.get("mlp") is None),
        family={"mixers": [layer["type"] for layer in cfg.layers], "norm_eps": cfg.norm_eps})
    fc.validate()
    return fc


register_architecture("Kefisun", KefisunConfig, kefisun_forward_config, aliases=("kefisun",))
