"""A plain, slow forward pass of the Fovenex design: whole sequences, no cache, no paging, one function per
mechanism, float64 torch on the CPU.  It shares no code with the engine: it reads a model folder with ``json`` and
the ``safetensors`` package and writes every sum as a loop or a dense matrix expression.

The design in short (positions count from 0):

* s copies ("streams") X_1 .. X_s of every token's row, all embed[tok] at first.  A sublayer f (a mixer or a
  feed-forward) with vectors a, b [s], a matrix M [s, s], a norm and a gain l:  y = l * f(norm(sum_s a_s X_s)),
  X_t <- sum_s M[s, t] X_s + r b_t y, all t from the old rows; r is one constant of the model.  A layer is a mixer and,
  where it has one, a feed-forward.  logits = head norm(sum_s X_s).
* norm: (x - mean) / sqrt(var + eps) * g.
* mixer "attention": two softmax maps a head over the same values.  q and k are RMS-normed per head and map (one gain
  for all), the first rot.dims dims turn (dim i with i + dims/2; frequencies may be slowed along a ramp, with a
  magnitude on cos and sin), causal.  o = A1 v - lam A2 v with lam = e^(lq1 . lk1) - e^(lq2 . lk2) + diff; o is RMS-normed
  over the head's values (no gain), times (1 - diff), times sigmoid of one number a head and token.
* mixer "latent_attention": q = W_uq rms(W_dq h); (c | kr) = W_dkv h, c RMS-normed; a head's key is (W_uk c | kr
  turned), its value W_uv c, under a sliding window; sigmoid(W_g h) multiplies the heads side by side.  A layer may read
  another layer's c and kr.
* ff: W_down gelu(W_up h), gelu in its tanh form.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional, Sequence

import torch

F = torch.float64


# --------------------------------------------------------------------------
# mechanisms
# --------------------------------------------------------------------------
def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def layer_norm(x: torch.Tensor, g: torch.Tensor, eps: float) -> torch.Tensor:
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * g


def gelu(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def read_streams(X: torch.Tensor, a: torch.Tensor) -> torch.Tensor:
    """X [s, T, W] -> the row a sublayer's norm reads."""
    u = torch.zeros_like(X[0])
    for s in range(X.shape[0]):
        u = u + a[s] * X[s]
    return u


def write_streams(X: torch.Tensor, M: torch.Tensor, b: torch.Tensor, y: torch.Tensor, r: float) -> torch.Tensor:
    """M is indexed [from, to]."""
    n = X.shape[0]
    out = torch.zeros_like(X)
    for t in range(n):
        for s in range(n):
            out[t] = out[t] + M[s, t] * X[s]
        out[t] = out[t] + r * b[t] * y
    return out


def pair_frequencies(dims: int, base: float, scaling=None):
    """(frequency of pair i, magnitude of cos and sin)."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return f, 1.0
    factor, orig = float(scaling["factor"]), float(scaling["original"])

    def place(turns):      # the dim at which a pair makes that many turns within the original length
        return dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(place(float(scaling["fast"]))), 0)
    hi = min(math.ceil(place(float(scaling["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def turn(x: torch.Tensor, freqs: Sequence[float], mag: float = 1.0) -> torch.Tensor:
    """x [T, heads, d], row t at position t; pair i is (i, i + len(freqs)); the dims beyond the pairs pass."""
    n = len(freqs)
    pos = torch.arange(x.shape[0], dtype=x.dtype).view(-1, 1, 1)
    ang = pos * torch.tensor(list(freqs), dtype=x.dtype).view(1, 1, -1)
    c, s = torch.cos(ang) * mag, torch.sin(ang) * mag
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], dim=-1)


def softmax_map(scores: torch.Tensor, window: Optional[int]) -> torch.Tensor:
    """scores [T, T] (query, key) -> weights; a query sees itself and what lies before it, at most ``window`` of these."""
    T = scores.shape[0]
    i, j = torch.arange(T).view(-1, 1), torch.arange(T).view(1, -1)
    seen = j <= i
    if window is not None:
        seen = seen & (i - j < window)
    e = torch.where(seen, scores, torch.full_like(scores, float("-inf")))
    e = torch.exp(e - e.max(dim=1, keepdim=True).values)
    return e / e.sum(dim=1, keepdim=True)


def mixing_weight(lq1, lk1, lq2, lk2, diff: float) -> float:
    return math.exp(float((lq1 * lk1).sum())) - math.exp(float((lq2 * lk2).sum())) + diff


def difference_of_maps(q, k, v, scale: float, lam: float, diff: float, eps: float) -> torch.Tensor:
    """q [T, H, 2, d], k [T, G, 2, d], v [T, G, dv] -> [T, H, dv]."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        a = [softmax_map(q[:, h, m] @ k[:, g, m].T * scale, None) @ v[:, g] for m in range(2)]
        out[:, h] = rms(a[0] - lam * a[1], eps) * (1.0 - diff)
    return out


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


def difference_mixer(m, w, p: str, h: torch.Tensor, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    q = rms((h @ w[p + "q"].T).reshape(T, H * 2, d), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T).reshape(T, G * 2, d), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).reshape(T, G, dv)
    rot = m.get("rot")
    if rot:
        freqs, mag = pair_frequencies(int(rot["dims"]), float(rot["base"]), rot.get("scaling"))
        q, k = turn(q, freqs, mag), turn(k, freqs, mag)
    lam = mixing_weight(w[p + "lq1"], w[p + "lk1"], w[p + "lq2"], w[p + "lk2"], float(m["diff"]))
    o = difference_of_maps(q.reshape(T, H, 2, d), k.reshape(T, G, 2, d), v, float(m["scale"]), lam, float(m["diff"]), eps)
    o = o * torch.sigmoid(h @ w[p + "g"].T).unsqueeze(2)
    return o.reshape(T, H * dv) @ w[p + "o"].T


def latent_mixer(m, w, p: str, h: torch.Tensor, eps: float, kept: Dict[int, tuple], i: int) -> torch.Tensor:
    """``kept``: layer -> (its latents, its turned key parts), filled by the layers that have projections for them."""
    T = h.shape[0]
    H, d, r, dv, rank = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    freqs, _ = pair_frequencies(int(m["rot"]["dims"]), float(m["rot"]["base"]))
    q = ((rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T).reshape(T, H, d + r)
    if m.get("kv_from") is None:
        z = h @ w[p + "dkv"].T
        kept[i] = (rms(z[:, :rank], eps) * w[p + "dkv.norm"], turn(z[:, rank:].reshape(T, 1, r), freqs)[:, 0])
        c, kr = kept[i]
    else:
        c, kr = kept[int(m["kv_from"])]
    q_turned = turn(q[..., d:], freqs)
    key, val = (c @ w[p + "uk"].T).reshape(T, H, d), (c @ w[p + "uv"].T).reshape(T, H, dv)
    mask = m.get("mask")
    o = torch.zeros((T, H, dv), dtype=h.dtype)
    for a in range(H):
        s = (q[:, a, :d] @ key[:, a].T + q_turned[:, a] @ kr.T) * float(m["scale"])
        o[:, a] = softmax_map(s, int(mask["size"]) if mask else None) @ val[:, a]
    return (o.reshape(T, H * dv) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def feed_forward(w, p: str, h: torch.Tensor) -> torch.Tensor:
    return gelu(h @ w[p + "up"].T) @ w[p + "down"].T


def forward(cfg, w, tokens: Sequence[int], return_layers: bool = False):
    """Logits [T, vocab] of a whole sequence (and the sum of the streams after every layer)."""
    eps, r, n = float(cfg["norm"]["eps"]), float(cfg["residual_mult"]), int(cfg["streams"])
    row = w["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    X = torch.stack([row] * n)
    after, kept = [], {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = layer_norm(read_streams(X, w[p + "hc1.in"]), w[p + "norm1"], eps)
        if layer["type"] == "attention":
            y = difference_mixer(layer["mixer"], w, p + "mix.", h, eps)
        elif layer["type"] == "latent_attention":
            y = latent_mixer(layer["mixer"], w, p + "mix.", h, eps, kept, i)
        else:
            raise ValueError(f"layer {i}: unknown type {layer['type']!r}")
        X = write_streams(X, w[p + "hc1.mix"], w[p + "hc1.out"], y * w[p + "ls1"], r)
        if layer.get("mlp") is not None:
            h = layer_norm(read_streams(X, w[p + "hc2.in"]), w[p + "norm2"], eps)
            X = write_streams(X, w[p + "hc2.mix"], w[p + "hc2.out"], feed_forward(w, p + "mlp.", h) * w[p + "ls2"], r)
        after.append(X.sum(dim=0))
    y = layer_norm(X.sum(dim=0), w["final.norm"], eps) @ w["head"].T
    return (y, torch.stack(after)) if return_layers else y


def greedy_generate(cfg, w, prompt: Sequence[int], new_tokens: int) -> List[int]:
    ids, out = list(prompt), []
    for _ in range(new_tokens):
        nxt = int(torch.argmax(forward(cfg, w, ids)[-1]))
        out.append(nxt)
        ids.append(nxt)
    return out
