"""Small Kefisun configurations of the tests and their random weights.

The sizes differ from layer to layer and between the configurations in everything the format lets differ: heads
against key/value heads (equal, 2, 3 and 20 to 1), dim against vdim (smaller, larger, equal), taps of the input
convolution (1, 3, 6) and of the projections' (1 to 5), windows and none, layers that mix values and layers that do
not (the first layer is not always one that does), ranks of the low-rank gates, limits, scales, widths that are no
multiple of 4 or 8, layers of either kind with and without a feed-forward.

Weights are drawn here (not by the engine's random-weights mode): gains and biases away from their neutral values,
shares of the mixed values between and beyond 0 and 1, decays from slow to fast, wide convolution taps.  The two
optional ranks in the configurations name the tensors' own."""
import json
import os

import torch


def _attn(heads, kv, dim, vdim, conv, scale, window=None, mix=False):
    m = dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv, scale=scale, v_mix=mix)
    if window:
        m["mask"] = dict(size=window)
    return m


def _delta(heads, kv, dim, vdim, conv, ra, rg):
    return dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv, decay_rank=ra, gate_rank=rg)


def _dense(ff, limit):
    return dict(kind="dense", ff=ff, limit=limit)


def _layer(kind, mixer, mlp):
    return dict(type=kind, mixer=mixer, mlp=mlp)


MAIN = dict(
    architecture="Kefisun", width=96, vocab=310, norm=dict(eps=3e-6), canon=dict(taps=3), embedding=dict(scale=5.5),
    logit_scale=1.7,
    layers=[
        _layer("attention", _attn(3, 3, 24, 40, 1, 0.2, window=33), _dense(136, 1.5)),
        _layer("attention", _attn(6, 2, 32, 16, 4, 0.15, window=20, mix=True), _dense(72, 0.6)),
        _layer("channel_delta", _delta(4, 2, 16, 24, 2, 10, 7), _dense(40, 3.0)),
        _layer("attention", _attn(2, 1, 16, 32, 2, 0.25, window=9, mix=True), None),
        _layer("channel_delta", _delta(3, 3, 40, 8, 4, 32, 5), None),
        _layer("attention", _attn(4, 4, 64, 8, 3, 0.1, window=20, mix=True), _dense(64, 1.0)),
    ])

# a width that is no multiple of 4, more taps than the unrolled kernels have, heads that no matrix-core kernel takes
ODD = dict(
    architecture="Kefisun", width=83, vocab=150, norm=dict(eps=1e-5), canon=dict(taps=6), embedding=dict(scale=0.75),
    logit_scale=0.4,
    layers=[
        _layer("channel_delta", _delta(2, 1, 18, 10, 3, 3, 9), _dense(36, 2.0)),
        _layer("attention", _attn(5, 5, 20, 12, 5, 0.3, window=7, mix=True), _dense(60, 0.8)),
        _layer("attention", _attn(4, 2, 8, 30, 2, 0.4, window=12, mix=True), None),
    ])

# heads of 128 and beyond any matrix-core kernel, many query heads a key/value head, no input convolution to speak of
# (one tap), no windows; key channels that need the largest registers of the recurrence
WIDE = dict(
    architecture="Kefisun", width=128, vocab=200, norm=dict(eps=1e-6), canon=dict(taps=1), embedding=dict(scale=3.0),
    logit_scale=1.0,
    layers=[
        _layer("attention", _attn(2, 1, 128, 96, 3, 0.09, window=18), _dense(64, 4.0)),
        _layer("channel_delta", _delta(2, 2, 130, 72, 4, 33, 40), _dense(32, 1.2)),
        _layer("attention", _attn(20, 1, 16, 16, 2, 0.25), None),
        _layer("attention", _attn(1, 1, 144, 40, 2, 0.08, window=30, mix=True), _dense(32, 1.0)),
        _layer("channel_delta", _delta(2, 1, 64, 64, 1, 8, 8), None),
    ])

CONFIGS = {"main": MAIN, "odd": ODD, "wide": WIDE}


def tensor_shapes(cfg):
    """name -> shape of every tensor a model of ``cfg`` needs."""
    W, V, out = cfg["width"], cfg["vocab"], {}
    out["embed"] = (V, W)
    mixes = False
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"], out[p + "canon1"] = (W,), (W, cfg["canon"]["taps"])
        if layer["type"] == "attention":
            Qd, Kd, Vd = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
            out.update({p + "mix.q.norm": (Qd,), p + "mix.k.norm": (Kd,), p + "mix.r1": (m["heads"],), p + "mix.r2": (m["heads"],),
                        p + "mix.g": (m["heads"] * m["vdim"], W), p + "mix.o": (W, m["heads"] * m["vdim"])})
            if m.get("v_mix"):
                if mixes:
                    out[p + "mix.vmix"] = ()
                mixes = True
        else:
            Qd, Kd, Vd = m["kv_heads"] * m["dim"], m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            C = m["heads"] * m["dim"]
            out.update({p + "mix.b": (m["heads"], W), p + "mix.A_log": (m["heads"],), p + "mix.norm": (m["vdim"],),
                        p + "mix.a1": (m["decay_rank"], W), p + "mix.a2": (C, m["decay_rank"]), p + "mix.dt_bias": (C,),
                        p + "mix.g1": (m["gate_rank"], W), p + "mix.g2": (Vd, m["gate_rank"]), p + "mix.o": (W, Vd)})
        for x, rows in (("q", Qd), ("k", Kd), ("v", Vd)):
            out.update({f"{p}mix.{x}": (rows, W), f"{p}mix.{x}.conv": (rows, m["conv"])})
        mlp = layer.get("mlp")
        if mlp is None:
            continue
        out[p + "norm2"] = (W,)
        out.update({p + "mlp.gate": (mlp["ff"], W), p + "mlp.up": (mlp["ff"], W), p + "mlp.down": (W, mlp["ff"]),
                    p + "mlp.gate.b": (mlp["ff"],), p + "mlp.up.b": (mlp["ff"],), p + "mlp.down.b": (W,)})
    out["final.norm"] = (W,)
    return out


def make_weights(cfg, seed, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.split(".")[-1]
        rand = lambda: torch.randn(shape, generator=g)      # noqa: E731
        if last in ("norm1", "norm2") or name == "final.norm":
            t = 0.3 * rand()                                                 # the stored gain is the distance from one
        elif last == "norm":
            t = 1.0 + 0.2 * rand()
        elif last == "A_log":
            t = torch.log(0.2 + 3.0 * torch.rand(shape, generator=g))        # decays from slow to fast
        elif last == "dt_bias":
            t = rand() - 1.0
        elif last in ("conv", "canon1"):
            t = 0.5 * rand()
        elif last == "vmix":
            t = 0.4 + 0.5 * rand()
        elif last == "r1":
            t = 1.5 * torch.rand(shape, generator=g)
        elif last == "r2":
            t = 2.0 * torch.rand(shape, generator=g)
        elif name.endswith(".b") and ".mlp." in name:
            t = 0.3 * rand()
        elif name == "embed":
            t = rand() / cfg["embedding"]["scale"]
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
    """A configuration drawn at random: sizes, head counts, the order of layers, taps, windows, which layers mix
    values, ranks, limits, scales, eps."""
    import random
    rng = random.Random(seed)
    cfg = dict(architecture="Kefisun", width=rng.choice([48, 64, 70, 72, 96, 128, 160]), vocab=rng.choice([97, 256, 411]),
               norm=dict(eps=rng.choice([1e-6, 1e-5, 3e-6])), canon=dict(taps=rng.choice([1, 2, 3, 4, 5])),
               embedding=dict(scale=rng.choice([1.0, 0.3, 9.0])), logit_scale=rng.choice([1.0, 0.25, 3.0]), layers=[])
    shared = None      # the number of values a token in the layers that mix
    for i in range(rng.randint(2, 6)):
        mlp = None if rng.random() < 0.3 else _dense(rng.choice([24, 40, 96]), rng.choice([0.5, 1.0, 2.0, 7.0]))
        if rng.random() < 0.55:
            kvh, vdim = rng.choice([1, 2, 3, 4]), rng.choice([8, 16, 24, 40, 64])
            mix = rng.random() < 0.6
            if mix and shared is not None:
                kvh = rng.choice([k for k in (1, 2, 3, 4) if shared % k == 0])
                vdim = shared // kvh
            elif mix:
                shared = kvh * vdim
            dim = rng.choice([8, 16, 24, 32, 48, 64, 96, 128])
            mixer = _attn(kvh * rng.choice([1, 2, 4]), kvh, dim, vdim, rng.choice([1, 2, 3, 4, 6]),
                          rng.choice([0.05, 0.1, 0.2]) * (32.0 / dim) ** 0.5, window=rng.choice([None, 1, 5, 16, 17, 40, 200]), mix=mix)
            cfg["layers"].append(_layer("attention", mixer, mlp))
        else:
            kvh = rng.choice([1, 2, 3])
            mixer = _delta(kvh * rng.choice([1, 2, 3]), kvh, rng.choice([6, 8, 16, 24, 40, 64, 72]), rng.choice([4, 8, 20, 31, 64]),
                           rng.choice([1, 2, 3, 4]), rng.choice([1, 4, 16, 40]), rng.choice([1, 6, 32, 36]))
            cfg["layers"].append(_layer("channel_delta", mixer, mlp))
    return cfg
