"""Small Fovenex configurations of the tests and their random weights.

The sizes differ from layer to layer and between the configurations in everything the format lets differ: heads against
key/value heads (equal, 2, 3 and 10 to 1), dim against vdim (2 dim below, equal to and above vdim; odd halves), streams
(1 to 6), rotated dims (none of the head to all of it), slowed frequencies and plain ones, windows of one token and
wider and none, layers that read an earlier layer's latents through a wider and a narrower window than its own, query
latents wider and narrower than the key/value ones, layers of either kind with and without a feed-forward, widths that are no
multiple of 4 or 8, diff from 0 up, a residual constant away from 1.

Weights are drawn here (not by the engine's random-weights mode): mixing matrices away from the identity and not symmetric,
gains away from 1, query and key gains that make scores spread, maps that weigh against each other."""
import json
import os

import torch

RAMP = dict(factor=4.0, original=64, fast=8.0, slow=1.0)


def _rot(dims, base=10000.0, scaling=None):
    r = dict(base=base, dims=dims)
    if scaling:
        r["scaling"] = dict(scaling)
    return r


def _attn(heads, kv, dim, vdim, scale, diff, rot=None):
    m = dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale, diff=diff)
    if rot:
        m["rot"] = rot
    return m


def _latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, window, base=10000.0, kv_from=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale, rot=_rot(rot_dim, base))
    if window:
        m["mask"] = dict(size=window)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def _layer(kind, mixer, ff=None):
    return dict(type=kind, mixer=mixer, mlp=dict(kind="dense", ff=ff) if ff else None)


MAIN = dict(
    architecture="Fovenex", width=96, vocab=310, norm=dict(eps=3e-6), streams=3, residual_mult=0.7,
    layers=[
        _layer("attention", _attn(4, 2, 32, 64, 0.2, 0.35, _rot(32, 500.0, RAMP)), 136),
        _layer("latent_attention", _latent(3, 24, 8, 40, 48, 56, 0.2, 33), 72),
        _layer("attention", _attn(3, 1, 24, 16, 0.25, 0.1, _rot(8))),
        _layer("latent_attention", _latent(5, 16, 8, 24, 48, 40, 0.25, 9, kv_from=1), 40),
        _layer("latent_attention", _latent(2, 40, 16, 16, 64, 24, 0.15, 20, base=700.0)),
        _layer("attention", _attn(2, 2, 64, 128, 0.12, 0.6, _rot(64, 10000.0, dict(RAMP, factor=9.0, original=300))), 64),
        _layer("latent_attention", _latent(2, 24, 8, 32, 48, 64, 0.2, 50, kv_from=1), 48),
    ])

# a width that is no multiple of 4, more streams than the unrolled kernels have, sizes no matrix-core kernel takes
ODD = dict(
    architecture="Fovenex", width=83, vocab=150, norm=dict(eps=1e-5), streams=6, residual_mult=1.3,
    layers=[
        _layer("latent_attention", _latent(3, 10, 6, 14, 27, 19, 0.3, 12), 36),
        _layer("attention", _attn(5, 5, 11, 30, 0.35, 0.0, _rot(4))),
        _layer("latent_attention", _latent(1, 12, 6, 18, 27, 33, 0.3, 1, kv_from=0), 60),
        _layer("attention", _attn(4, 2, 18, 20, 0.3, 0.8), 20),
    ])

# heads of 128 and beyond any matrix-core kernel, more maps a key/value head than the decode kernel takes, one stream, no window
WIDE = dict(
    architecture="Fovenex", width=128, vocab=200, norm=dict(eps=1e-6), streams=1, residual_mult=1.0,
    layers=[
        _layer("attention", _attn(4, 1, 64, 96, 0.13, 0.3, _rot(32, 10000.0, RAMP)), 64),
        _layer("latent_attention", _latent(4, 32, 16, 32, 128, 96, 0.15, None), 96),
        _layer("attention", _attn(10, 1, 16, 32, 0.25, 0.2, _rot(16))),
        _layer("attention", _attn(2, 1, 72, 40, 0.1, 0.45, _rot(48)), 32),
        _layer("latent_attention", _latent(3, 48, 32, 24, 64, 128, 0.12, 18, base=2000.0)),
    ])

CONFIGS = {"main": MAIN, "odd": ODD, "wide": WIDE}


def tensor_shapes(cfg):
    """name -> shape of every tensor a model of ``cfg`` needs."""
    W, V, s, out = cfg["width"], cfg["vocab"], cfg["streams"], {}
    out["embed"], out["head"], out["final.norm"] = (V, W), (V, W), (W,)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        for q in (1, 2) if layer.get("mlp") else (1,):
            out.update({f"{p}norm{q}": (W,), f"{p}ls{q}": (W,), f"{p}hc{q}.in": (s,), f"{p}hc{q}.out": (s,), f"{p}hc{q}.mix": (s, s)})
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "attention":
            G = m["kv_heads"]
            out.update({p + "mix.q": (H * 2 * d, W), p + "mix.k": (G * 2 * d, W), p + "mix.v": (G * dv, W), p + "mix.q.norm": (d,),
                        p + "mix.k.norm": (d,), p + "mix.g": (H, W)})
            out.update({p + "mix." + x: (d,) for x in ("lq1", "lk1", "lq2", "lk2")})
        else:
            r, rank, qr = m["rot_dim"], m["kv_rank"], m["q_rank"]
            out.update({p + "mix.dq": (qr, W), p + "mix.dq.norm": (qr,), p + "mix.uq": (H * (d + r), qr), p + "mix.uk": (H * d, rank),
                        p + "mix.uv": (H * dv, rank), p + "mix.g": (H * dv, W)})
            if m.get("kv_from") is None:
                out.update({p + "mix.dkv": (rank + r, W), p + "mix.dkv.norm": (rank,)})
        out[p + "mix.o"] = (W, H * dv)
        if layer.get("mlp"):
            out.update({p + "mlp.up": (layer["mlp"]["ff"], W), p + "mlp.down": (W, layer["mlp"]["ff"])})
    return out


def make_weights(cfg, seed, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    w, s = {}, cfg["streams"]
    for name, shape in tensor_shapes(cfg).items():
        last = name.split(".")[-1]
        rand = lambda: torch.randn(shape, generator=g)      # noqa: E731
        if name.endswith("q.norm") or name.endswith("k.norm"):
            t = 1.3 + 0.5 * rand()
        elif last.startswith("norm") or last.startswith("ls"):
            t = 1.0 + 0.25 * rand()
        elif last == "in":
            t = (1.0 + 0.5 * rand()) / s
        elif last == "out":
            t = 1.0 + 0.5 * rand()
        elif last == "mix" and ".hc" in name:
            t = torch.eye(s) + 0.3 * rand()
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.3 * rand()
        elif name == "embed":
            t = rand()
        else:
            t = rand() * (1.0 / shape[-1] ** 0.5)
        w[name] = t.to(dtype)
    return w


def write_config(folder, cfg, weights):
    from zedinfer_amd.weights.safetensors_io import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    write_safetensors(os.path.join(folder, "model.safetensors"), weights, metadata={"format": "pt"})
    return folder


def write_model(folder, name, seed=0, dtype=torch.float32):
    """config.json and model.safetensors of configuration ``name``; returns the folder."""
    return write_config(folder, CONFIGS[name], make_weights(CONFIGS[name], seed, dtype))


def random_config(seed):
    """A configuration drawn at random: sizes, head counts, the order of layers, streams, windows, which layers read
    another's latents, scales, diff, eps."""
    import random
    rng = random.Random(seed)
    cfg = dict(architecture="Fovenex", width=rng.choice([48, 64, 70, 72, 96, 128, 160]), vocab=rng.choice([97, 256, 411]),
               norm=dict(eps=rng.choice([1e-6, 1e-5, 3e-6])), streams=rng.choice([1, 2, 2, 3, 4, 5, 7]),
               residual_mult=rng.choice([1.0, 0.5, 0.3, 1.4]), layers=[])
    owners = []
    for i in range(rng.randint(2, 6)):
        ff = None if rng.random() < 0.3 else rng.choice([24, 40, 96])
        if rng.random() < 0.5:
            G = rng.choice([1, 2, 3, 4])
            dim, vdim = rng.choice([6, 8, 16, 24, 32, 48, 64, 80]), rng.choice([8, 12, 16, 32, 48, 64, 96, 128])
            rot = None
            if rng.random() < 0.85:
                rot = _rot(rng.choice([d for d in (2, 4, 8, 16, 24, 32, 64) if d <= dim]), rng.choice([100.0, 10000.0, 250000.0]),
                           rng.choice([None, RAMP, dict(factor=2.0, original=2048, fast=32.0, slow=1.0), dict(factor=40.0, original=20, fast=1.0, slow=1.0)]))
            cfg["layers"].append(_layer("attention", _attn(G * rng.choice([1, 2, 4]), G, dim, vdim,
                                                           rng.choice([0.1, 0.2, 0.3]) * (16.0 / dim) ** 0.5, rng.choice([0.0, 0.2, 0.5, 0.85]), rot), ff))
        else:
            window = rng.choice([None, 1, 5, 16, 17, 40, 200])
            src = rng.choice(owners) if owners and rng.random() < 0.5 else None
            if src is None:
                rank, r, base = rng.choice([16, 20, 32, 64, 96, 136]), rng.choice([4, 8, 16, 32]), rng.choice([100.0, 10000.0])
                owners.append(i)
            else:
                o = cfg["layers"][src]["mixer"]
                rank, r, base = o["kv_rank"], o["rot_dim"], o["rot"]["base"]
            dim = rng.choice([8, 12, 16, 32, 48])
            cfg["layers"].append(_layer("latent_attention", _latent(rng.choice([1, 2, 3, 4, 6]), dim, r, rng.choice([8, 10, 16, 32, 40]), rank,
                                                                    rng.choice([12, 16, 40, 72]), rng.choice([0.1, 0.2, 0.3]), window, base, src), ff))
    return cfg
