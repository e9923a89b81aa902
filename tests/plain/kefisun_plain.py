"""A plain, slow forward pass of the Kefisun design: whole sequences, no cache, no paging, one function per
mechanism, float64 torch on the CPU.  It shares no code with the engine: it reads a model folder with ``json`` and
the ``safetensors`` package and writes every sum as a loop or a dense matrix expression.

The design in short (x_t is the residual stream of token t, positions count from 0):

* x_t = embed[tok_t] * c_in; a layer: h = n1(x), h <- h + conv(h), x <- x + mixer(h); then, where the layer has a
  feed-forward, x <- x + ff(n2(x)); every n is x / sqrt(mean x^2 + eps) * (1 + g); conv is a causal convolution over
  time on each channel.
* mixer "attention": grouped-query softmax attention under a sliding window, without rotation.  q, k, v are
  projections of h that pass a short causal convolution per channel; q and k an RMS norm over the whole projection;
  a score is (q . k) scale - r1 ln(1 + r2 distance) with two numbers a head; from the second such layer on (of those
  that mix values) v <- (1 - a) v + a v_of_the_first_layer; the heads side by side are multiplied by sigmoid(W_g h).
* mixer "channel_delta": the delta rule with a decay per head and key channel, S <- g S, u = beta (v - S^T k),
  S <- S + k u^T, o = S^T q; q, k, v pass a short convolution and silu, q and k are unit vectors; the decay comes from
  a low-rank projection through softplus; each head's o is RMS-normed, times a gain, times a low-rank sigmoid gate.
* ff: g = min(W_gate h + b, limit), u = clamp(W_up h + b, +-limit), W_down (g sigmoid(1.702 g) (u + 1)) + b.
* logits = embed n_final(x) * c_out.
"""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional, Sequence

import torch

F = torch.float64


# --------------------------------------------------------------------------
# mechanisms
# --------------------------------------------------------------------------
def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def one_plus_norm(x: torch.Tensor, g: torch.Tensor, eps: float) -> torch.Tensor:
    return rms(x, eps) * (1.0 + g)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1.0 + torch.exp(-z))


def softplus(z: torch.Tensor) -> torch.Tensor:
    """ln(1 + e^z) = max(z, 0) + ln(1 + e^-|z|)."""
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def causal_convolution(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """u [T, C]; taps [C, K], the last column weighs the present token; zeros before the start."""
    T, K = u.shape[0], taps.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        for j in range(K):
            s = t - (K - 1) + j
            if s >= 0:
                out[t] = out[t] + taps[:, j] * u[s]
    return out


def input_convolution(h: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    return h + causal_convolution(h, taps)


def distance_biased_attention(q, k, v, scale: float, r1, r2, window: Optional[int]) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv]; head h reads key/value head h // (H / G); token t sees the last
    ``window`` tokens (itself among them; None: all); score = (q . k) scale - r1_h ln(1 + r2_h distance)."""
    T, H, _ = q.shape
    G, dv = k.shape[1], v.shape[2]
    out = torch.zeros((T, H, dv), dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for t in range(T):
            lo = 0 if window is None else max(0, t - window + 1)
            s = torch.zeros(t + 1 - lo, dtype=q.dtype)
            dist = torch.arange(t - lo, -1, -1, dtype=q.dtype)
            s = (k[lo:t + 1, g] @ q[t, h]) * scale - r1[h] * torch.log(1.0 + r2[h] * dist)
            p = torch.exp(s - s.max())
            out[t, h] = (p / p.sum()) @ v[lo:t + 1, g]
    return out


def mix_values(v: torch.Tensor, first: torch.Tensor, share: torch.Tensor) -> torch.Tensor:
    return (1.0 - share) * v + share * first


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def channel_decay(z: torch.Tensor, a_log: torch.Tensor, heads: int) -> torch.Tensor:
    """z [T, heads * dim] (the low-rank projection plus its bias) -> g [T, heads, dim] in (0, 1)."""
    T = z.shape[0]
    return torch.exp(-torch.exp(a_log).view(1, heads, 1) * softplus(z).view(T, heads, -1))


def channel_delta_rule(q, k, v, beta, g, state=None):
    """q, k [T, KH, d] (unit vectors, q also scaled); v [T, H, dv]; beta [T, H]; g [T, H, d].  Returns the read-outs
    [T, H, dv] and the final state [H, d, dv]."""
    T, H, dv = v.shape
    KH, d = k.shape[1], k.shape[2]
    S = torch.zeros((H, d, dv), dtype=v.dtype) if state is None else state.clone()
    out = torch.zeros((T, H, dv), dtype=v.dtype)
    for t in range(T):
        for h in range(H):
            kk, qq = k[t, h // (H // KH)], q[t, h // (H // KH)]
            S[h] = g[t, h].view(d, 1) * S[h]
            u = beta[t, h] * (v[t, h] - S[h].T @ kk)
            S[h] = S[h] + torch.outer(kk, u)
            out[t, h] = S[h].T @ qq
    return out, S


def clamped_glu(g: torch.Tensor, u: torch.Tensor, limit: float) -> torch.Tensor:
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


# --------------------------------------------------------------------------
# the model
# --------------------------------------------------------------------------
def load_folder(folder: str, dtype=F):
    from safetensors import safe_open
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    w: Dict[str, torch.Tensor] = {}
    with safe_open(os.path.join(folder, "model.safetensors"), "pt") as f:
        for name in f.keys():
            w[name] = f.get_tensor(name).to(dtype)
    return cfg, w


def attention_mixer(cfg, m, w, p: str, h: torch.Tensor, first_values: List[torch.Tensor]) -> torch.Tensor:
    """``first_values``: empty until the first layer that mixes values has run, then that layer's values."""
    T = h.shape[0]
    H, G, d, dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    eps = float(cfg["norm"]["eps"])
    q = causal_convolution(h @ w[p + "q"].T, w[p + "q.conv"])
    k = causal_convolution(h @ w[p + "k"].T, w[p + "k.conv"])
    v = causal_convolution(h @ w[p + "v"].T, w[p + "v.conv"])
    q = rms(q, eps) * w[p + "q.norm"]
    k = rms(k, eps) * w[p + "k.norm"]
    if m.get("v_mix"):
        if first_values:
            v = mix_values(v, first_values[0], w[p + "vmix"])
        else:
            first_values.append(v)
    mask = m.get("mask")
    o = distance_biased_attention(q.view(T, H, d), k.view(T, G, d), v.view(T, G, dv), float(m["scale"]), w[p + "r1"],
                                  w[p + "r2"], int(mask["size"]) if mask else None)
    return (o.reshape(T, H * dv) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def delta_mixer(cfg, m, w, p: str, h: torch.Tensor) -> torch.Tensor:
    T = h.shape[0]
    H, KH, d, dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    q, k, v = (silu(causal_convolution(h @ w[p + x].T, w[p + x + ".conv"])) for x in ("q", "k", "v"))
    q, k = unit(q.view(T, KH, d)) * d ** -0.5, unit(k.view(T, KH, d))
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = channel_decay((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"], w[p + "A_log"], H)
    o, _ = channel_delta_rule(q, k, v.view(T, H, dv), beta, g)
    o = rms(o, float(cfg["norm"]["eps"])) * w[p + "norm"]
    gate = torch.sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T)
    return (o.reshape(T, H * dv) * gate) @ w[p + "o"].T


def feed_forward(mlp, w, p: str, h: torch.Tensor) -> torch.Tensor:
    y = clamped_glu(h @ w[p + "gate"].T + w[p + "gate.b"], h @ w[p + "up"].T + w[p + "up.b"], float(mlp["limit"]))
    return y @ w[p + "down"].T + w[p + "down.b"]


def forward(cfg, w, tokens: Sequence[int], return_layers: bool = False):
    """Logits [T, vocab] of a whole sequence (and the residual stream after every layer)."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(list(tokens), dtype=torch.long)] * float(cfg["embedding"]["scale"])
    after, first_values = [], []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = input_convolution(one_plus_norm(x, w[p + "norm1"], eps), w[p + "canon1"])
        if layer["type"] == "attention":
            x = x + attention_mixer(cfg, layer["mixer"], w, p + "mix.", h, first_values)
        elif layer["type"] == "channel_delta":
            x = x + delta_mixer(cfg, layer["mixer"], w, p + "mix.", h)
        else:
            raise ValueError(f"layer {i}: unknown type {layer['type']!r}")
        if layer.get("mlp") is not None:
            x = x + feed_forward(layer["mlp"], w, p + "mlp.", one_plus_norm(x, w[p + "norm2"], eps))
        after.append(x.clone())
    y = one_plus_norm(x, w["final.norm"], eps) @ w["embed"].T * float(cfg["logit_scale"])
    return (y, torch.stack(after)) if return_layers else y


def greedy_generate(cfg, w, prompt: Sequence[int], new_tokens: int) -> List[int]:
    ids, out = list(prompt), []
    for _ in range(new_tokens):
        nxt = int(torch.argmax(forward(cfg, w, ids)[-1]))
        out.append(nxt)
        ids.append(nxt)
    return out
