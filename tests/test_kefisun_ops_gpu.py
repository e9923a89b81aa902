"""Every new mechanism of the Kefisun design alone, on the GPU, against the plain functions of
``tests/plain/kefisun_plain.py``: the convolution of a mixer's input (behind the norm, for portions and in one launch
for single tokens), low-rank gates, the delta rule with a decay per channel (whole, cut, single tokens, used slots),
values mixed with an earlier layer's, attention with a logarithm of the distance through every kernel, biases in the
clamped activation and in partial sums, a gate from partial sums, scaled embeddings and gains.  Sizes are the tests'
own."""
import pytest
import torch

from plain import kefisun_plain as plain
from zedinfer_amd import ops

pytestmark = pytest.mark.gpu
DEV = "cuda"
F64 = torch.float64
BF = torch.bfloat16


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


def _close(got, want, tol, what=""):
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    err = float((got - want).abs().max())
    assert err <= tol * max(1.0, float(want.abs().max())), (what, err, float(want.abs().max()))


def _entries(lens, slots):
    start, seq = [0], []
    for i, n in enumerate(lens):
        seq += [i] * n
        start.append(start[-1] + n)
    return dict(tok_seq=_i32(seq), entry_start=_i32(start[:-1]), entry_len=_i32(lens), entry_slot=_i32(slots))


# ---- the convolution in front of a mixer ------------------------------------------------------------------------------
STEPS = ([("a", 17)], [("a", 1), ("b", 2)], [("b", 1), ("a", 1)], [("b", 30), ("a", 2)], [("a", 1)], [("c", 1), ("a", 3)], [("c", 2)],
         [("c", 1)], [("c", 5)])
LENS = {"a": 25, "b": 33, "c": 9}
SLOT = {"a": 2, "b": 0, "c": 1}


@pytest.mark.parametrize("H, taps, dtype, add_one", [(96, 3, BF, True), (84, 4, torch.float32, True), (130, 1, BF, False),
                                                    (83, 2, torch.float32, True), (52, 6, BF, True), (1536, 4, BF, True), (4100, 2, torch.float32, False)])
def test_the_input_convolution_behind_the_norm_carries_its_rows_from_step_to_step(H, taps, dtype, add_one):
    g = torch.Generator().manual_seed(H)
    eps = 1e-5
    x = {r: 2 * torch.randn(n, H, generator=g) for r, n in LENS.items()}          # the stream, half of it still pending
    d = {r: torch.randn(n, H, generator=g) for r, n in LENS.items()}
    gain = (0.3 if add_one else 1.0) * torch.randn(H, generator=g)
    gain = gain.to(dtype).float()
    w = torch.randn(H, taps, generator=g)
    want = {r: plain.input_convolution(plain.rms((x[r] + d[r]).double(), eps) * (gain.double() + (1 if add_one else 0)), w.double())
            for r in LENS}
    tail = (taps - 1) * H
    state = torch.full((4, tail + 8), 5.0, device=DEV)          # a column slice of a wider row; slot 3 is nobody's
    for r, s in SLOT.items():
        state[s, 4:4 + tail] = 0.0
    view = state[:, 4:4 + tail] if taps > 1 else None
    cw = w.t().contiguous().to(DEV)
    fed = {r: 0 for r in LENS}
    got = {r: [] for r in LENS}
    for si, step in enumerate(STEPS):
        lens = [n for _, n in step]
        en = _entries(lens, [SLOT[r] for r, _ in step])
        rows = torch.cat([x[r][fed[r]:fed[r] + n] for r, n in step]).to(DEV)
        pend = torch.cat([d[r][fed[r]:fed[r] + n] for r, n in step]).to(DEV)
        N = rows.shape[0]
        S = 1 + si % 3
        delta = torch.stack([pend * 0.25] * S)                   # a stack of terms (or one) that sums to the pending half
        delta[-1] += pend - delta.sum(0)
        delta = delta.contiguous() if S > 1 else delta[0].contiguous()
        out = torch.zeros(N, H, dtype=dtype, device=DEV)
        gw = gain.to(DEV).to(dtype)
        single = all(n == 1 for n in lens)
        if single and ops.norm_input_conv_supported(H, taps, delta):
            ops.norm_input_conv(rows, delta, gw, 1.0 if add_one else 0.0, eps, cw, view, en["tok_seq"], en["entry_slot"], out=out)
        else:
            sc = ops.stream_scale(rows, delta, eps, out=torch.empty(N, device=DEV))
            ops.input_conv(rows, cw, view, **en, out=out, scale=sc, gain=gw, gain_add=1.0 if add_one else 0.0)
        at = 0
        for r, n in step:
            _close(rows[at:at + n], (x[r] + d[r])[fed[r]:fed[r] + n], 1e-6, "the stream takes the addition")
            got[r].append(out[at:at + n].cpu())
            at += n
            fed[r] += n
    for r in LENS:
        _close(torch.cat(got[r]), want[r], 1e-5 if dtype == torch.float32 else 1e-2, r)
    assert float(state[3].min()) == 5.0 == float(state[3].max()) and float(state[:, :4].min()) == 5.0 == float(state[:, 4 + tail:].max())


@pytest.mark.parametrize("taps", [2, 4, 6])
@pytest.mark.parametrize("n", [5, 300, 700, 2100])
def test_the_input_convolution_of_long_steps_and_of_rows_without_a_norm(n, taps):
    """Workgroups of several rows (their number grows with the step), entries that begin anywhere in them, rows read as
    they are, padding behind an entry's own tokens and an entry that has none of its own."""
    g = torch.Generator().manual_seed(n + taps)
    H = 64
    lens = [1, 2, 3]
    while sum(lens) < n:
        lens.append(min(1 + (len(lens) * 37) % 97, n - sum(lens)))
    slots_of = list(range(len(lens)))
    x = torch.randn(sum(lens), H, generator=g)
    w = torch.randn(H, taps, generator=g)
    old = torch.randn(len(lens) + 1, (taps - 1) * H, generator=g)
    state = old.clone().to(DEV)
    en = _entries(lens, slots_of)
    place = torch.arange(sum(lens), dtype=torch.int32)
    real = list(lens)
    real[1] = 1                              # the second entry brings one token and one of padding
    real[3 if len(lens) > 3 else 2] = 0       # one has none of its own
    at = 0
    for a, b in zip(lens, real):
        place[at + b:at + a] = -1
        at += a
    out = torch.zeros(sum(lens), H, device=DEV)
    ops.input_conv(x.to(DEV), w.t().contiguous().to(DEV), state, **en, out=out, slots=place.to(DEV))
    at = 0
    for e, (n_e, r_e) in enumerate(zip(lens, real)):
        before = old[e].view(taps - 1, H).double()
        seq = torch.cat([before, x[at:at + n_e].double()])
        want = plain.input_convolution(seq, w.double())[taps - 1:]
        _close(out[at:at + n_e], want, 1e-5, (e, n_e))
        tail = old[e].double() if r_e == 0 else torch.cat([before, x[at:at + r_e].double()])[-(taps - 1):].reshape(-1)
        _close(state[e], tail, 1e-6, ("tail", e, n_e, r_e))
        at += n_e
    assert torch.equal(state[-1].cpu(), old[-1])


# ---- low-rank gates -----------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("n", [1, 7, 40, 150])
@pytest.mark.parametrize("heads, dim, vdim, ra, rg, dtype", [(3, 16, 40, 32, 64, BF), (2, 40, 24, 10, 7, BF), (4, 8, 8, 64, 32, torch.float32),
                                                            (5, 20, 12, 3, 9, torch.float32), (2, 130, 72, 64, 96, BF)])
def test_low_rank_gates_also_far_out(n, heads, dim, vdim, ra, rg, dtype):
    g = torch.Generator().manual_seed(dim)
    Ca, Cg = heads * dim, heads * vdim
    proj = torch.randn(n, 4 + ra + rg + 4, generator=g)
    proj[0, 4:4 + ra] *= 40                                # gates far out on both sides
    wa, wg = torch.randn(Ca, ra, generator=g).to(dtype), torch.randn(Cg, rg, generator=g).to(dtype)
    bias, a_log = torch.randn(Ca, generator=g) * 2, torch.log(0.05 + 3 * torch.rand(heads, generator=g))
    want_a = plain.channel_decay(proj.double()[:, 4:4 + ra] @ wa.double().T + bias.double(), a_log.double(), heads).reshape(n, Ca)
    want_g = proj.double()[:, 4 + ra:4 + ra + rg] @ wg.double().T
    p = proj.to(DEV)
    oa, og = torch.zeros(n, Ca, device=DEV), torch.zeros(n, Cg, device=DEV)
    ops.lowrank_gates(p[:, 4:4 + ra], wa.to(DEV), bias.to(DEV), a_log.to(DEV), p[:, 4 + ra:4 + ra + rg], wg.to(DEV), oa, og)
    _close(oa[1:], want_a[1:], 2e-4, "decay") if n > 1 else None
    _close(oa[:1], want_a[:1], 2e-3, "decay far out")      # (the projection's rounding times 40)
    _close(og, want_g, 2e-5, "gate")
    assert float(oa.min()) >= 0.0 and float(oa.max()) <= 1.0


# ---- the delta rule with a decay per channel ------------------------------------------------------------------------------
def _delta_inputs(n, heads, kvh, dim, vdim, seed):
    g = torch.Generator().manual_seed(seed)
    q, k = plain.unit(torch.randn(n, kvh, dim, generator=g)) * dim ** -0.5, plain.unit(torch.randn(n, kvh, dim, generator=g))
    v, beta = torch.randn(n, heads, vdim, generator=g), torch.rand(n, heads, generator=g)
    decay = 0.3 + 0.7 * torch.rand(n, heads, dim, generator=g)
    decay[::5] = 1.0
    decay[3::11] *= 1e-3                                      # some strong forgetting
    return q, k, v, beta, decay


@pytest.mark.parametrize("heads, kvh, dim, vdim", [(4, 2, 16, 24), (3, 3, 40, 8), (2, 1, 18, 10), (2, 2, 130, 72), (1, 1, 256, 20), (6, 2, 64, 64),
                                                   (2, 1, 128, 130), (5, 5, 5, 3), (2, 2, 128, 4)])
def test_the_channel_delta_rule_in_portions_single_tokens_and_used_slots(heads, kvh, dim, vdim):
    lens_of = {"a": 71, "b": 19, "c": 6}
    data = {r: _delta_inputs(n, heads, kvh, dim, vdim, seed=n + dim) for r, n in lens_of.items()}
    want = {r: plain.channel_delta_rule(*[t.double() for t in data[r]]) for r in lens_of}
    floats = heads * dim * vdim
    pad = 4
    state = torch.full((3, pad + -(-floats // 4) * 4 + 4), 5.0, device=DEV)
    slot = {"a": 2, "b": 0, "c": 2}                             # c runs in a's slot after a has ended
    view = state[:, pad:pad + floats]
    view[2] = 0.0
    view[0] = 0.0
    got, fed = {r: [] for r in lens_of}, {r: 0 for r in lens_of}
    steps = ([("a", 17)], [("a", 1), ("b", 2)], [("b", 16), ("a", 32)], [("a", 1)], [("a", 1), ("b", 1)], [("a", 19)], [("c", 2)], [("c", 1)], [("c", 3)])
    for step in steps:
        if step[0][0] == "c" and fed["c"] == 0:
            end_a = view[2].clone()
            view[2] = 0.0
        lens = [n for _, n in step]
        en = _entries(lens, [slot[r] for r, _ in step])
        cat = lambda i: torch.cat([data[r][i][fed[r]:fed[r] + n] for r, n in step]).to(DEV)      # noqa: E731
        q, k, v, beta, decay = (cat(i) for i in range(5))
        N = q.shape[0]
        qk = torch.cat([q.reshape(N, -1), k.reshape(N, -1)], dim=1).contiguous()
        bg = torch.full((N, 2, heads), 77.0, device=DEV)
        bg[:, 0] = beta
        out = torch.full((N, heads * vdim), 9.0, device=DEV)
        ops.delta_channel(qk, v.reshape(N, -1).contiguous(), bg, decay.reshape(N, -1).contiguous(), view, en["entry_start"],
                          en["entry_len"], en["entry_slot"], heads, kvh, dim, vdim, out=out, single_tokens=all(n == 1 for n in lens))
        at = 0
        for r, n in step:
            got[r].append(out[at:at + n].cpu())
            at += n
            fed[r] += n
    for r in lens_of:
        _close(torch.cat(got[r]), want[r][0].reshape(lens_of[r], -1), 3e-5, r)
    for r, s in (("a", end_a), ("b", view[0]), ("c", view[2])):
        _close(s, want[r][1].reshape(-1), 3e-5, ("state", r))
    assert float(state[:, :pad].min()) == 5.0 == float(state[:, pad + floats:].max())      # nothing beside the state is touched
    assert float(state[1].min()) == 5.0 == float(state[1].max())                            # nor a slot of no entry


def test_a_cut_of_the_prompt_changes_no_bit_of_the_channel_delta_rule():
    heads, kvh, dim, vdim, n = 2, 2, 48, 20, 50
    q, k, v, beta, decay = (t.to(DEV) for t in _delta_inputs(n, heads, kvh, dim, vdim, seed=4))
    qk = torch.cat([q.reshape(n, -1), k.reshape(n, -1)], dim=1).contiguous()
    bg = torch.stack([beta, beta], dim=1).contiguous()
    outs = []
    for cuts in ([50], [1] * 50, [3, 16, 1, 17, 13], [8, 8, 16, 18], [7, 9, 2, 32]):
        state = torch.zeros(1, heads * dim * vdim, device=DEV)
        out, at = torch.empty(n, heads * vdim, device=DEV), 0
        for c in cuts:
            en = _entries([c], [0])
            ops.delta_channel(qk[at:at + c], v.reshape(n, -1)[at:at + c], bg[at:at + c], decay.reshape(n, -1)[at:at + c], state,
                              en["entry_start"], en["entry_len"], en["entry_slot"], heads, kvh, dim, vdim, out=out[at:at + c])
            at += c
        outs.append((out.clone(), state.clone()))
    for o, s in outs[1:]:
        assert torch.equal(o, outs[0][0]) and torch.equal(s, outs[0][1])


# ---- values mixed with an earlier layer's -----------------------------------------------------------------------------------
@pytest.mark.parametrize("splits", [1, 3])
@pytest.mark.parametrize("taps", [1, 3, 5])
def test_values_are_kept_after_the_convolution_and_mixed_before_they_are_cached(taps, splits):
    g = torch.Generator().manual_seed(taps)
    nh, nkv, dim, vdim, T, ps, d = 4, 2, 16, 24, 21, 8, 24
    Qd, Kd, Vd = nh * dim, nkv * dim, nkv * vdim
    C = Qd + Kd + Vd
    proj, w = torch.randn(T, C, generator=g), torch.randn(C, taps, generator=g)
    other, mix = torch.randn(T, Vd, generator=g), 0.3
    wide = torch.randn(splits, T, C + 8, generator=g)      # columns of a wider product, as partial sums
    wide[:, :, :C] = proj / splits
    stack = wide.to(DEV)[:, :, :C]
    rows = stack if splits > 1 else stack[0]
    conv = plain.causal_convolution(proj.double(), w.double())
    v = conv[:, Qd + Kd:]
    state = torch.zeros(2, max(1, (taps - 1) * C), device=DEV)
    en = _entries([T], [1])
    slots = _i32(list(range(T)))
    kept = torch.zeros(T, Vd, device=DEV)
    ones = torch.ones(max(Qd, Kd), device=DEV)
    for mixes in (False, True):
        kc, vc = torch.zeros(3, nkv, ps, d, device=DEV), torch.zeros(3, nkv, d, ps, device=DEV)
        q_out = torch.zeros(T, nh * d, device=DEV)
        ops.conv_qkv(rows, None, w.to(DEV), state, ones[:Qd], ones[:Kd], 1e-5, None, en["tok_seq"], en["entry_start"], en["entry_slot"],
                     slots, kc, vc, nh, nkv, dim, vdim, d, taps, q_out,
                     **(dict(mix_values=other.to(DEV), mix=mix) if mixes else dict(values_out=kept)))
        got = vc.permute(0, 3, 1, 2).reshape(24, nkv, d)[:T, :, :vdim].reshape(T, Vd)
        _close(got, plain.mix_values(v, other.double(), torch.tensor(mix, dtype=F64)) if mixes else v, 1e-5, ("cached", mixes))
        _close(q_out.view(T, nh, d)[:, :, :dim].reshape(T, Qd), plain.rms(conv[:, :Qd], 1e-5), 1e-5, "queries")
    _close(kept, v, 1e-5, "kept")


# ---- attention with a logarithm of the distance -------------------------------------------------------------------------------
def _paged(n_tokens, ps, seed, spare=3):
    pages = -(-n_tokens // ps)
    table = torch.randperm(pages + spare, generator=torch.Generator().manual_seed(seed))[:pages].to(torch.int32)
    pos = torch.arange(n_tokens)
    return table.view(1, -1), (table[pos // ps].long() * ps + pos % ps), pages + spare


def _dense(q, k, v, scale, r1, r2, window):
    """The plain mechanism as one matrix expression (held against it on a prefix): long sequences stay quick."""
    T, H, _ = q.shape
    G = k.shape[1]
    dist = (torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)).double()
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        s = (q[:, h] @ k[:, h // (H // G)].T) * scale - r1[h] * torch.log(1.0 + r2[h] * dist.clamp(min=0))
        s = s.masked_fill((dist < 0) | ((dist >= window) if window else torch.zeros_like(dist, dtype=torch.bool)), float("-inf"))
        out[:, h] = torch.softmax(s, dim=1) @ v[:, h // (H // G)]
    n = min(T, 40)
    assert float((out[:n] - plain.distance_biased_attention(q[:n], k[:n], v[:n], scale, r1, r2, window or None)).abs().max()) < 1e-9
    return out


CASES = [
    # T, heads, kv_heads, head size, page, window
    (300, 4, 2, 32, 8, 20), (450, 2, 1, 128, 16, 200), (333, 3, 3, 48, 16, 0), (260, 5, 5, 20, 4, 9), (700, 8, 4, 64, 16, 130),
    (2500, 2, 2, 64, 16, 2300), (200, 20, 1, 16, 8, 33), (2300, 2, 1, 128, 32, 0), (150, 1, 1, 144, 16, 64), (140, 2, 1, 64, 64, 1),
]


@pytest.mark.parametrize("case", CASES)
@pytest.mark.parametrize("dtype", [BF, torch.float32])
def test_attention_with_a_logarithm_of_the_distance_through_every_kernel(case, dtype):
    T, H, G, d, ps, window = case
    if dtype == torch.float32 and T > 1000:
        T = T // 4
    g = torch.Generator().manual_seed(T + d)
    q, k = torch.randn(T, H, d, generator=g).to(dtype).float(), torch.randn(T, G, d, generator=g).to(dtype).float()
    v = (2 * torch.randn(T, G, d, generator=g)).to(dtype).float()
    r1, r2 = 0.2 + 1.5 * torch.rand(H, generator=g), 0.1 + 2 * torch.rand(H, generator=g)
    # queries near the end ask for one key each with a score that stands out: the window's last place, the first one
    # outside it, and the places next to them; a key far back where there is no window
    W = window or T - 8
    for qi, gap in ((T - 1, W - 1), (T - 2, W), (T - 3, W + 1), (T - 4, max(W - 2, 0)), (T - 5, 0)):
        kj = max(qi - gap, 0)
        for a in range(H):
            q[qi, a] = 9.0 * k[kj, a // (H // G)] / k[kj, a // (H // G)].norm()
    q = q.to(dtype).float()
    scale = 1.3 / d ** 0.5
    want = _dense(q.double(), k.double(), v.double(), scale, r1.double(), r2.double(), window).reshape(T, H * d)
    table, slots, pages = _paged(T, ps, seed=T)
    kc = torch.full((pages, G, ps, d), 7.0, dtype=dtype, device=DEV)
    vc = torch.full((pages, G, d, ps), 7.0, dtype=dtype, device=DEV)
    kc[slots // ps, :, slots % ps] = k.to(DEV).to(dtype)
    vc[slots // ps, :, :, slots % ps] = v.to(DEV).to(dtype)
    qd = q.reshape(T, H * d).to(DEV).to(dtype).contiguous()
    tol = 3e-5 if dtype == torch.float32 else 2.5e-2
    pos, seq0, tab = torch.arange(T, dtype=torch.int32, device=DEV), torch.zeros(T, dtype=torch.int32, device=DEV), table.to(DEV)
    extras = dict(log_distance=(r1.to(DEV), r2.to(DEV)))
    att = torch.zeros(T, H * d, dtype=dtype, device=DEV)
    ops.attention_biased(qd, kc, vc, seq0, pos, tab, H, G, d, scale, window, out=att, **extras)
    _close(att, want, tol, "plain kernel")
    if ops.attention_decode_supported(dtype, H, G, d, ps):
        att = torch.zeros(T, H * d, dtype=dtype, device=DEV)
        ops.attention_decode(qd, kc, vc, seq0, pos, tab, H, G, d, scale, T, window, out=att, **extras)
        _close(att, want, tol, "single tokens")
        some = _i32([T - 1, T - 3, 5, T - 2])
        att2 = torch.zeros(T, H * d, dtype=dtype, device=DEV)
        ops.attention_decode(qd, kc, vc, seq0, pos, tab, H, G, d, scale, T, window, out=att2, tok_index=some, **extras)
        assert torch.equal(att2[some.long()], att[some.long()]) and float(att2[6].abs().max()) == 0.0
        # the same behind a gate: chunks left, merged and gated by a kernel, or by the output projection for few tokens
        head = d - 3                                       # (heads padded in the cache: only their first values count)
        rows = torch.cat([torch.arange(T - 9, T), torch.tensor([0, 5, W - 1, T // 2])]).clamp(0, T - 1)
        n, ws = rows.numel(), torch.full((ops.attention_decode_workspace(rows.numel(), H, d),), float("nan"), device=DEV)
        gate = 2 * torch.randn(3, n, H * head + 6, generator=g)
        args = (qd[rows.to(DEV)].contiguous(), kc, vc, seq0[:n], pos[rows.to(DEV)].contiguous(), tab, H, G, d, scale, T, window)
        sinks = torch.randn(H, generator=g).to(DEV) if G > 1 else None
        merged = want[rows].view(n, H, d)
        if sinks is not None:                              # (a sink rescales a head: the sums of its softmax, from the scores)
            merged = torch.zeros_like(merged)
            for i, t in enumerate(rows.tolist()):
                lo = max(0, t - window + 1) if window else 0
                for h in range(H):
                    dist = torch.arange(t - lo, -1, -1).double()
                    sc = k[lo:t + 1, h // (H // G)].double() @ q[t, h].double() * scale - r1[h].double() * torch.log(1 + r2[h].double() * dist)
                    wgt = torch.softmax(torch.cat([sc, sinks[h:h + 1].cpu().double()]), dim=0)[:-1]
                    merged[i, h] = wgt @ v[lo:t + 1, h // (H // G)].double()
        ops.attention_decode(*args, workspace=ws, sinks=sinks, leave_chunks=True, **extras)
        y = torch.zeros(n, H * head, dtype=BF, device=DEV)
        ops.attention_decode_merge_gated(ws, args[4], H, d, head, T, gate.to(DEV)[:, :, 6:], y, window=window, sinks=sinks)
        _close(y, (merged[:, :, :head].reshape(n, -1) * torch.sigmoid(gate[:, :, 6:].double().sum(0))), 2.5e-2, "merged and gated")
        wo = (torch.randn(40, H * d, generator=g) / (H * d) ** 0.5).to(BF)
        gate = 2 * torch.randn(6, n, H * d + 4, generator=g)
        for gt in (gate[:, :, 4:], gate[0, :, 4:]):
            if not ops.attention_decode_project_supported(wo.to(DEV), n, H, d):
                continue
            sums = ops.attention_decode_project(ws, wo.to(DEV), args[4], H, d, T, window, sinks=sinks, gate=gt.to(DEV))
            gated = merged.reshape(n, -1) * torch.sigmoid(gt.double().sum(0) if gt.dim() == 3 else gt.double())
            _close(sums.sum(0), gated @ wo.double().T, 2.5e-2, "projected behind the gate")
    if not ops.attention_prefill_supported(dtype, H, G, d, ps):
        return
    least, most = ops.attention_prefill_tile_min(), ops.attention_prefill_tile(dtype, d)
    for past in (0, T - 120, T - 70):
        n = T - past
        for tile, alone in [(least, False)] + ([(most, False), (least, True), (most, True)] if most > least else []):
            offs = list(range(0, n, tile))
            att = torch.zeros(n, H * d, dtype=dtype, device=DEV)
            ops.attention_prefill(qd[past:], kc, vc, _i32([0] * len(offs)), _i32(offs), _i32([0]), _i32([n]), _i32([past]), tab,
                                  H, G, d, scale, window, out=att, max_keys=T, tile=tile, alone=alone, **extras)
            _close(att, want[past:], tol, ("tiles", past, tile, alone))


# ---- the smaller pieces ---------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("inter, n, dtype", [(64, 5, BF), (62, 130, torch.float32), (300, 70, BF), (296, 70, BF), (1500, 64, BF), (37, 9, BF)])
def test_the_clamped_feed_forward_with_biases(inter, n, dtype):
    from zedinfer_amd.config import PartSpec
    from zedinfer_amd.parts import FEED_FORWARDS, Runtime
    g = torch.Generator().manual_seed(inter)
    H, limit = 96, 0.9
    w = {"gate": torch.randn(inter, H, generator=g) / H ** 0.5, "up": torch.randn(inter, H, generator=g) / H ** 0.5,
         "down": torch.randn(H, inter, generator=g) / inter ** 0.5, "gate_bias": torch.randn(inter, generator=g),
         "up_bias": torch.randn(inter, generator=g), "down_bias": torch.randn(H, generator=g)}
    w = {k: t.to(dtype) for k, t in w.items()}
    x = torch.randn(n, H, generator=g).to(dtype)
    p = {("f." + k.replace("_bias", ".b")): t.double() for k, t in w.items()}
    want = plain.feed_forward(dict(limit=limit), p, "f.", x.double())
    spec = PartSpec("clamped_mlp", {"hidden_size": H, "intermediate_size": inter, "limit": limit, "bias": True}, {k: k for k in w})
    part = FEED_FORWARDS.get("clamped_mlp")(spec, {k: t.to(DEV) for k, t in w.items()}, Runtime(DEV, dtype))
    y = part.forward(x.to(DEV))
    y = y.float().sum(0) if y.dim() == 3 else y
    _close(y, want, 1e-5 if dtype == torch.float32 else 2e-2, "clamped_mlp")
    # without biases it is the same form
    spec0 = PartSpec("clamped_mlp", {"hidden_size": H, "intermediate_size": inter, "limit": limit}, {k: k for k in ("gate", "up", "down")})
    part = FEED_FORWARDS.get("clamped_mlp")(spec0, {k: w[k].to(DEV) for k in ("gate", "up", "down")}, Runtime(DEV, dtype))
    y = part.forward(x.to(DEV))
    want = plain.clamped_glu(x.double() @ p["f.gate"].T, x.double() @ p["f.up"].T, limit) @ p["f.down"].T
    _close(y.float().sum(0) if y.dim() == 3 else y, want, 1e-5 if dtype == torch.float32 else 2e-2, "no biases")


@pytest.mark.parametrize("M, I, K", [(1, 88, 64), (17, 1504, 320), (64, 8192, 1024), (33, 6400, 264), (250, 24, 8)])
@pytest.mark.parametrize("biased", [True, False])
def test_the_clamped_activation_over_rows_that_alternate_in_blocks(M, I, K, biased):
    g = torch.Generator().manual_seed(I)
    x, w = torch.randn(M, K, generator=g).to(BF), (2 * torch.randn(2 * I, K, generator=g) / K ** 0.5).to(BF)
    b = torch.randn(2 * I, generator=g).to(BF) if biased else None
    full = x.double() @ w.double().T + (b.double() if biased else 0.0)
    blocks = full.view(M, I // 8, 2, 8)
    want = plain.clamped_glu(blocks[:, :, 0].reshape(M, I), blocks[:, :, 1].reshape(M, I), 1.1)
    rows = full.to(BF).to(DEV)
    wide = torch.zeros(M, I + 16, dtype=BF, device=DEV)
    _close(ops.clamped_glu_il8(rows, 1.1, out=wide[:, 8:8 + I]), want, 2e-2, "rows")
    assert float(wide[:, :8].abs().max()) == 0.0 and float(wide[:, 8 + I:].abs().max()) == 0.0
    xd, wd, bd = x.to(DEV), w.to(DEV), (b.to(DEV) if biased else None)
    if M <= ops.FEW_ROWS and ops.linear_swiglu_supported(xd, wd):
        _close(ops.linear_clamped_glu(xd, wd, bd, 1.1), want, 1e-2, "epilogue")
    else:
        with pytest.raises(ValueError):
            ops.linear_clamped_glu(xd, wd, bd, 1.1)


@pytest.mark.parametrize("M, N, K", [(1, 96, 512), (7, 1536, 1536), (70, 260, 768), (128, 90, 256), (200, 4096, 8192)])
def test_the_first_partial_sum_holds_the_bias(M, N, K):
    g = torch.Generator().manual_seed(N)
    x, w = torch.randn(M, K, generator=g).to(BF).to(DEV), torch.randn(N, K, generator=g).to(BF).to(DEV)
    b = (30 * torch.randn(N, generator=g)).to(BF).to(DEV)
    if not ops.linear_sums_supported(x, w):
        pytest.skip("not a product of few rows")
    with_b, without = ops.linear_sums(x, w, bias=b), ops.linear_sums(x, w)
    assert torch.equal(with_b[1:], without[1:])
    _close(with_b[0], without[0] + b.float(), 1e-6)


def test_a_gate_from_partial_sums_and_scaled_rows():
    g = torch.Generator().manual_seed(9)
    n, heads, head, x_head = 6, 3, 10, 16
    x, gate = torch.randn(n, heads * x_head, generator=g), torch.randn(4, n, heads * head + 5, generator=g)
    want = x.view(n, heads, x_head)[:, :, :head].reshape(n, -1).double() * torch.sigmoid(gate.double().sum(0)[:, 5:])
    out = torch.zeros(n, heads * head, device=DEV)
    ops.gate_heads(x.to(DEV), gate.to(DEV)[:, :, 5:], head, x_head, "sigmoid", out=out)
    _close(out, want, 1e-6)
    table = torch.randn(11, 20, generator=g).to(BF)
    out = torch.zeros(4, 20, device=DEV)
    ops.embedding(_i32([3, 0, 10, 3]), table.to(DEV), out=out, scale=2.7)
    _close(out, table[[3, 0, 10, 3]].double() * 2.7, 1e-6)
    from zedinfer_amd.config import PartSpec
    from zedinfer_amd.parts import NORMS, Runtime
    gain, rows = (0.3 * torch.randn(20, generator=g)).to(BF), torch.randn(5, 20, generator=g)
    part = NORMS.get("rmsnorm")(PartSpec("rmsnorm", {"dim": 20, "eps": 1e-5, "add_one": True, "gain_scale": 0.37}), {"weight": gain.to(DEV)},
                                Runtime(DEV, torch.float32))
    _close(part.forward(rows.to(DEV)), plain.one_plus_norm(rows.double(), gain.double(), 1e-5) * 0.37, 1e-6)
