"""Every new mechanism of the Fovenex design alone, on the GPU, against the plain functions of
``tests/plain/fovenex_plain.py``: residual streams written, read and normed in one launch; queries and keys normed, turned
and stored for softmax maps that share values; the difference of the maps from attention rows and from the chunks of decoded
tokens, through every attention kernel, with keys that carry the weight placed at borders; query latents, latents and key parts
from one product; a gate where the values are made; the activation alone.  Sizes are the tests' own."""
import pytest
import torch

from plain import fovenex_plain as plain
from zedinfer_amd import ops

pytestmark = pytest.mark.gpu
DEV = "cuda"
F32, F64, BF = torch.float32, torch.float64, torch.bfloat16


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


def _close(got, want, tol, what=""):
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    err = float((got - want).abs().max())
    assert err <= tol * max(1.0, float(want.abs().max())), (what, err, float(want.abs().max()))


def _tol(dtype):
    return 1e-5 if dtype == F32 else 1e-2


# ---- the streams --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("H, s, n", [(96, 2, 5), (83, 3, 4), (192, 1, 7), (1536, 2, 33), (1540, 4, 3), (4100, 3, 2), (8200, 2, 2), (64, 6, 5),
                                     (90, 16, 3), (3584, 2, 300)])
@pytest.mark.parametrize("dtype", [F32, BF])
def test_streams_are_written_read_and_normed_in_one_launch(H, s, n, dtype):
    g = torch.Generator().manual_seed(H + s)
    X = torch.randn((s, n, H), generator=g)
    M, b, a = torch.randn((s, s), generator=g), torch.randn(s, generator=g), torch.randn(s, generator=g)
    scale, gain = 1 + 0.3 * torch.randn(H, generator=g), 1 + 0.3 * torch.randn(H, generator=g)
    write = torch.cat([M.reshape(-1), b]).to(DEV)
    dev = lambda t: t.contiguous().to(DEV)      # noqa: E731
    for S in (0, 1, 2, 4, 7):
        if S == 0:
            y, y_dev = None, None
        else:
            terms = torch.randn((S, n, H), generator=g)
            if S == 1:
                y_dev = dev(terms[0].to(dtype))
                y = y_dev.float().cpu().double()
            else:
                y_dev, y = dev(terms), terms.double().sum(0)
        for equal in (False, True):
            base = X[:1].expand(s, n, H) if equal else X
            new = base.double() if y is None else plain.write_streams(base.double(), M.double(), b.double(), y * scale.double(), 1.0)
            u = plain.read_streams(new, a.double())
            for centered in (True, False):
                want = plain.layer_norm(u, gain.double(), 1e-5) if centered else plain.rms(u, 1e-5) * gain.double()
                streams = dev(X[0] if equal else X)
                keep = None if y is None else (streams if not equal else torch.empty((s, n, H), device=DEV))
                kw = {} if y is None else dict(y=y_dev, write=write, scale=dev(scale), keep=keep)
                out = ops.stream_mix(streams, dev(a), dev(gain), 1e-5, centered, out=torch.empty((n, H), dtype=dtype, device=DEV), **kw)
                _close(out, want, _tol(dtype), (S, equal, centered))
                if keep is not None:
                    _close(keep, new, 1e-5, ("kept", S, equal))
        # the end of a model: the sum of the streams, some rows of it, nothing kept
        if y is not None:
            rows = [n - 1, 0, n // 2]
            new = plain.write_streams(X.double(), M.double(), b.double(), y * scale.double(), 1.0)
            want = plain.layer_norm(new.sum(0), gain.double(), 1e-6)[rows]
            streams = dev(X)
            out = ops.stream_mix(streams, torch.ones(s, device=DEV), dev(gain), 1e-6, True, out=torch.empty((3, H), dtype=dtype, device=DEV),
                                 y=y_dev, write=write, scale=dev(scale), rows=_i32(rows))
            _close(out, want, _tol(dtype), ("rows", S))
            assert torch.equal(streams.cpu(), X)


def test_a_row_of_the_streams_does_not_depend_on_the_others():
    g = torch.Generator().manual_seed(1)
    X, y = torch.randn((2, 40, 1536), generator=g).to(DEV), torch.randn((40, 1536), generator=g).to(DEV)
    write, read, gain = torch.randn(6, generator=g).to(DEV), torch.randn(2, generator=g).to(DEV), torch.ones(1536, device=DEV)
    kw = lambda a, b: dict(y=y[a:b].contiguous(), write=write, keep=torch.empty((2, b - a, 1536), device=DEV))      # noqa: E731
    whole = ops.stream_mix(X, read, gain, 1e-6, True, out=torch.empty((40, 1536), device=DEV), **kw(0, 40))
    for a, b in ((0, 1), (7, 9), (3, 40)):
        part = ops.stream_mix(X[:, a:b].contiguous(), read, gain, 1e-6, True, out=torch.empty((b - a, 1536), device=DEV), **kw(a, b))
        assert torch.equal(part, whole[a:b])


def test_streams_that_do_not_fit_together_are_refused():
    X, a, gain, out = torch.zeros((2, 3, 8), device=DEV), torch.ones(2, device=DEV), torch.ones(8, device=DEV), torch.empty((3, 8), device=DEV)
    with pytest.raises(ValueError):
        ops.stream_mix(X, torch.ones(3, device=DEV), gain, 1e-6, True, out=out)
    with pytest.raises(ValueError):
        ops.stream_mix(X, a, gain, 1e-6, True, out=out, y=torch.zeros((3, 8), device=DEV), write=torch.zeros(5, device=DEV))
    with pytest.raises(ValueError):      # nothing to keep without a result
        ops.stream_mix(X, a, gain, 1e-6, True, out=out, keep=X)
    with pytest.raises(ValueError):
        ops.stream_mix(X, a, gain, 1e-6, True, out=torch.empty((2, 8), device=DEV))


# ---- softmax maps that share values: into the cache -----------------------------------------------------------------------
def _table(n, freqs, mag, positions):
    f = torch.tensor(freqs, dtype=F32, device=DEV)
    return ops.rope_table_scaled(_i32(positions), f, mag, out=torch.empty((n, len(freqs), 2), device=DEV))


def _turned(x, freqs, mag, positions):
    """Rows at the given positions: the plain turn of a sequence, picked."""
    T = max(positions) + 1
    full = torch.zeros((T,) + tuple(x.shape[1:]), dtype=F64)
    for i, p in enumerate(positions):
        full[p] = x[i]
    return plain.turn(full, freqs, mag)[positions]


@pytest.mark.parametrize("n", [5, 300])
@pytest.mark.parametrize("H, G, dim, vdim, d, rot, page", [(4, 2, 64, 128, 128, 64, 16), (3, 1, 32, 64, 64, 16, 8), (2, 2, 24, 40, 48, 8, 4),
                                                           (5, 1, 16, 64, 64, 0, 16), (2, 1, 64, 96, 128, 32, 32), (1, 1, 128, 64, 256, 128, 8)])
@pytest.mark.parametrize("dtype", [F32, BF])
def test_queries_and_keys_are_normed_turned_and_stored(n, H, G, dim, vdim, d, rot, page, dtype):
    tol = 1e-4 if dtype == F32 else 1e-2      # (an angle of 300 is good to 2e-5 in float32)
    g = torch.Generator().manual_seed(dim + n)
    width = (H + G) * 2 * dim + G * vdim
    proj = torch.randn((n, width), generator=g).to(dtype)
    qg, kg = 1 + 0.3 * torch.randn(dim, generator=g), 1 + 0.3 * torch.randn(dim, generator=g)
    positions = [3 + i for i in range(n)]
    freqs, mag = plain.pair_frequencies(rot, 50.0, dict(factor=4.0, original=64, fast=8.0, slow=1.0)) if rot else ([], 1.0)
    p64 = proj.double()
    q = plain.rms(p64[:, :H * 2 * dim].reshape(n, H * 2, dim), 1e-5) * qg.double()
    k = plain.rms(p64[:, H * 2 * dim:(H + G) * 2 * dim].reshape(n, G * 2, dim), 1e-5) * kg.double()
    v = p64[:, (H + G) * 2 * dim:].reshape(n, G, vdim)
    if rot:
        q, k = _turned(q, freqs, mag, positions), _turned(k, freqs, mag, positions)
    table = _table(n, freqs, mag, positions) if rot else None
    pages = n // page + 3
    order = torch.randperm(pages * page, generator=g)
    for scattered in (False, True):
        slots = (order[:n] if scattered else torch.arange(page, page + n)).tolist()
        slots[1] = -1                                  # a token without a place
        part = d // 2
        for terms in ((1, 3) if n == 5 else (1,)):
            src = proj.to(DEV)
            if terms > 1:
                src = torch.stack([proj.float() * 0.25] * terms)
                src[-1] += proj.float() - src.sum(0)
                src = src.to(DEV)
            for pad in (True, False):
                qo = torch.full((n, H * 2 * d), 7.0, dtype=dtype, device=DEV)
                kc = torch.full((pages, G, page, d), 9.0, dtype=dtype, device=DEV)
                vc = torch.full((pages, G, d, page), 9.0, dtype=dtype, device=DEV)
                ops.head_norm_store(src, qg.to(DEV), kg.to(DEV), 1e-5, table, _i32(slots), kc, vc, H, G, 2, dim, vdim, d, q_out=qo, pad=pad)
                got = qo.cpu().double().view(n, H, 2, d)
                want = q.reshape(n, H, 2, dim)
                for m in range(2):
                    _close(got[:, :, m, m * part:m * part + dim], want[:, :, m], tol, "queries")
                    rest = torch.ones(d, dtype=torch.bool)
                    rest[m * part:m * part + dim] = False
                    if pad:
                        assert float(got[:, :, m, rest].abs().max() if rest.any() else 0) == 0.0
                kcpu, vcpu = kc.cpu().double(), vc.cpu().double()
                touched = torch.zeros((pages, page), dtype=torch.bool)
                for t, sl in enumerate(slots):
                    if sl < 0:
                        continue
                    pg, off = sl // page, sl % page
                    touched[pg, off] = True
                    row = torch.zeros((G, d), dtype=F64)
                    for m in range(2):
                        row[:, m * part:m * part + dim] = k[t].view(G, 2, dim)[:, m]
                    assert float((kcpu[pg, :, off] - row).abs().max()) <= tol * max(1.0, float(row.abs().max())), ("keys", t)
                    assert float((vcpu[pg, :, :vdim, off] - v[t]).abs().max()) <= tol * max(1.0, float(v[t].abs().max()))
                    assert float(vcpu[pg, :, vdim:, off].abs().max() if vdim < d else 0) == 0.0
                assert bool((kcpu.permute(0, 2, 1, 3)[~touched] == 9.0).all()) and bool((vcpu.permute(0, 3, 1, 2)[~touched] == 9.0).all())


# ---- the difference of the maps ------------------------------------------------------------------------------------------
def _pool(seqs, G, dim, vdim, d, page, dtype, seed, spare=3):
    """Sequences (k [T, G, 2, dim], v [T, G, vdim]) in a paged cache, pages in a random order; (kc, vc, tables)."""
    g = torch.Generator().manual_seed(seed)
    need = [-(-k.shape[0] // page) for k, _ in seqs]
    pages = sum(need) + spare
    order = torch.randperm(pages, generator=g).tolist()
    kc = torch.full((pages, G, page, d), float("nan"), dtype=dtype)
    vc = torch.full((pages, G, d, page), float("nan"), dtype=dtype)
    tables = torch.full((len(seqs), max(need)), -1, dtype=torch.int32)
    part = d // 2
    for i, (k, v) in enumerate(seqs):
        for p in range(need[i]):
            tables[i, p] = order.pop()
        for t in range(k.shape[0]):
            pg, off = int(tables[i, t // page]), t % page
            row = torch.zeros((G, d))
            for m in range(2):
                row[:, m * part:m * part + dim] = k[t, :, m]
            kc[pg, :, off] = row.to(dtype)
            vc[pg, :, :, off] = 0
            vc[pg, :, :vdim, off] = v[t].to(dtype)
    return kc.to(DEV), vc.to(DEV), tables.to(DEV)


def _case(T, H, G, dim, vdim, seed, loud=(), spread=1.0):
    """Random q, k, v of a sequence; ``loud``: (query, key, map, head) whose score stands out."""
    g = torch.Generator().manual_seed(seed)
    q, k = spread * torch.randn((T, H, 2, dim), generator=g), torch.randn((T, G, 2, dim), generator=g)
    v = torch.randn((T, G, vdim), generator=g)
    for i, j, m, h in loud:
        k[j, h // (H // G), m] = q[i, h, m] * 4.0
    b = lambda t: t.to(BF).float()      # noqa: E731
    return b(q), b(k), b(v)


def _padded(q, d):
    n, H, _, dim = q.shape
    out = torch.zeros((n, H, 2, d))
    for m in range(2):
        out[:, :, m, m * (d // 2):m * (d // 2) + dim] = q[:, :, m]
    return out.reshape(n, H * 2 * d)


LAM, DIFF, EPS, SCALE = 0.4, 0.3, 1e-6, 0.2


def _reference(q, k, v, gate):
    o = plain.difference_of_maps(q.double(), k.double(), v.double(), SCALE, LAM, DIFF, EPS)
    return o * torch.sigmoid(gate.double()).unsqueeze(2)


@pytest.mark.parametrize("H, G, dim, vdim, d, page", [(4, 2, 64, 128, 128, 16), (3, 1, 32, 64, 64, 8), (4, 4, 24, 40, 48, 16), (8, 1, 48, 96, 96, 16),
                                                      (2, 1, 16, 96, 96, 32), (2, 2, 64, 100, 128, 64), (2, 1, 8, 16, 16, 8)])
def test_decoded_tokens_through_the_chunks(H, G, dim, vdim, d, page):
    """Single tokens at many positions (one chunk of keys and several), the loud key in a chunk's last and first place, at a
    page's border and far back."""
    lens = [1, 2, 9, page, page + 1, 255, 256, 257, 512, 513, 700]
    seqs, qs, want, gates = [], [], [], []
    g = torch.Generator().manual_seed(9)
    for i, T in enumerate(lens):
        loud = [(T - 1, j, m, h) for j, m, h in ((0, 0, 0), (max(T - 256, 0), 1, H - 1), (max(T - 257, 0), 0, H - 1)) if j < T - 1]
        q, k, v = _case(T, H, G, dim, vdim, 100 + i, loud)
        gate = torch.randn((T, H), generator=g)
        seqs.append((k, v))
        qs.append(q[-1:])
        gates.append(gate[-1:])
        want.append(_reference(q, k, v, gate)[-1])
    kc, vc, tables = _pool(seqs, G, dim, vdim, d, page, BF, 1)
    n = len(lens)
    q = _padded(torch.cat(qs), d).to(BF).to(DEV)
    pos, seq = _i32([T - 1 for T in lens]), _i32(list(range(n)))
    gate = torch.cat(gates).to(DEV)
    assert ops.attention_decode_supported(BF, 2 * H, G, d, page)
    ws = torch.empty(ops.attention_decode_workspace(n, 2 * H, d), device=DEV)
    ops.attention_decode(q, kc, vc, seq, pos, tables, 2 * H, G, d, SCALE, max(lens), 0, workspace=ws, leave_chunks=True)
    out = torch.empty((n, H * vdim), dtype=BF, device=DEV)
    terms = torch.stack([gate * 0.5, gate * 0.5])
    wide = torch.zeros((2, n, H + 5), device=DEV)
    wide[:, :, 2:2 + H] = terms
    for gt in (gate, gate.to(BF), wide[:, :, 2:2 + H]):
        ops.difference_merge(ws, pos, H, d, vdim, max(lens), LAM, 1.0 - DIFF, EPS, out=out, gate=gt)
        _close(out.view(n, H, vdim), torch.stack(want), 2e-2, "chunks")
    # the same from whole attention rows
    att = ops.attention_decode(q, kc, vc, seq, pos, tables, 2 * H, G, d, SCALE, max(lens), 0)
    two = ops.difference_heads(att, H, d, vdim, LAM, 1.0 - DIFF, EPS, out=torch.empty_like(out), gate=gate)
    _close(two.view(n, H, vdim), torch.stack(want), 2e-2, "rows")
    # a launch that covers fewer chunks than a token has shows it (256 keys: up to two chunks of 256, which begin at multiples of 8)
    ops.difference_merge(ws, pos, H, d, vdim, 256, LAM, 1.0 - DIFF, EPS, out=out, gate=gate)
    bad = out.view(n, -1).float().isnan().all(1).tolist()
    assert bad == [T > 512 for T in lens]


@pytest.mark.parametrize("H, G, dim, vdim, d", [(4, 2, 64, 128, 128), (3, 1, 32, 64, 64), (2, 1, 64, 90, 128), (2, 2, 24, 40, 48), (2, 1, 48, 96, 96)])
@pytest.mark.parametrize("page", [8, 16])
def test_portions_of_prompts(H, G, dim, vdim, d, page):
    """Several entries, some continuing a sequence, through the prompt kernel (the halves alone where it takes the size, every
    tile and both workgroups; the whole rows elsewhere), loud keys at block borders."""
    past, new = [0, 100, 130, 63, 1], [70, 5, 200, 65, 128]
    seqs, rows, want, gates = [], [], [], []
    g = torch.Generator().manual_seed(4)
    for i, (p, n) in enumerate(zip(past, new)):
        T = p + n
        loud = [(T - 1, 0, 0, 0), (T - 1, min(127, T - 2), 1, H - 1), (T - 2, min(128, T - 3), 0, H - 1), (p, max(p - 1, 0), 1, 0)]
        q, k, v = _case(T, H, G, dim, vdim, 50 + i, loud)
        gate = torch.randn((T, H), generator=g)
        seqs.append((k, v))
        rows.append(q[p:])
        gates.append(gate[p:])
        want.append(_reference(q, k, v, gate)[p:])
    kc, vc, tables = _pool(seqs, G, dim, vdim, d, page, BF, 2)
    N = sum(new)
    q = _padded(torch.cat(rows), d).to(BF).to(DEV)
    starts = [sum(new[:i]) for i in range(len(new))]
    ref = torch.cat(want)
    maps = 2 if ops.attention_prefill_maps_supported(BF, 2 * H, G, d, page, 2) else 1
    assert maps == (2 if d in (64, 128) else 1)
    if maps == 2:      # the rest of a query row is not read
        poisoned = q.clone().view(N, H, 2, d)
        poisoned[:, :, 0, d // 2:] = float("nan")
        poisoned[:, :, 1, :d // 2] = float("nan")
        q = poisoned.view(N, -1)
    for tile in sorted({64, ops.attention_prefill_tile(BF, d)}):
        for alone in ((False, True) if maps == 2 else (False,)):
            te = _i32([i for i, n in enumerate(new) for _ in range(0, n, tile)])
            to = _i32([o for n in new for o in range(0, n, tile)])
            att = ops.attention_prefill(q, kc, vc, te, to, _i32(starts), _i32(new), _i32(past), tables, 2 * H, G, d, SCALE, 0,
                                        max_keys=max(p + n for p, n in zip(past, new)), tile=tile, alone=alone, maps=maps)
            for gt in (torch.cat(gates).to(DEV), torch.cat(gates).to(DEV).to(BF)):
                out = ops.difference_heads(att, H, d, vdim, LAM, 1.0 - DIFF, EPS, out=torch.empty((N, H * vdim), dtype=BF, device=DEV), gate=gt)
                _close(out.view(N, H, vdim), ref, 3e-2, (tile, alone))


def test_a_long_prompt_whose_keys_are_cut_over_workgroups():
    H, G, dim, vdim, d, page, T = 2, 1, 64, 128, 128, 16, 4300
    loud = [(T - 1, 2047, 0, 0), (T - 1, 2048, 1, 1), (T - 2, 0, 1, 0), (T - 40, 4095, 0, 1)]
    q, k, v = _case(T, H, G, dim, vdim, 77, loud)
    kc, vc, tables = _pool([(k, v)], G, dim, vdim, d, page, BF, 3)
    n = 70
    rows = _padded(q[-n:], d).to(BF).to(DEV)
    ref = torch.zeros((n, H, vdim), dtype=F64)
    for h in range(H):
        a = []
        for m in range(2):
            s = (q[-n:, h, m].double() @ k[:, 0, m].double().T) * SCALE
            s = s.masked_fill(torch.arange(T).view(1, -1) > (T - n + torch.arange(n)).view(-1, 1), float("-inf"))
            a.append(torch.softmax(s, -1) @ v[:, 0].double())
        ref[:, h] = plain.rms(a[0] - LAM * a[1], EPS) * (1 - DIFF)
    for tile in (64, 128):
        te, to = _i32([0] * len(range(0, n, tile))), _i32(list(range(0, n, tile)))
        att = ops.attention_prefill(rows, kc, vc, te, to, _i32([0]), _i32([n]), _i32([T - n]), tables, 2 * H, G, d, SCALE, 0, max_keys=T,
                                    tile=tile, maps=2)
        out = ops.difference_heads(att, H, d, vdim, LAM, 1.0 - DIFF, EPS, out=torch.empty((n, H * vdim), dtype=BF, device=DEV))
        _close(out.view(n, H, vdim), ref, 3e-2, tile)


@pytest.mark.parametrize("H, d, vdim", [(3, 64, 64), (2, 128, 40), (5, 20, 18), (1, 512, 512), (2, 256, 256), (7, 16, 8)])
@pytest.mark.parametrize("dtype", [F32, BF])
def test_heads_from_attention_rows(H, d, vdim, dtype):
    g = torch.Generator().manual_seed(d)
    att = torch.randn((11, H * 2 * d), generator=g).to(dtype)
    gate = torch.randn((11, H + 3), generator=g)
    a = att.double().view(11, H, 2, d)[..., :vdim]
    want = plain.rms(a[:, :, 0] - 0.7 * a[:, :, 1], 1e-4) * 0.45
    out = torch.empty((11, H * vdim), dtype=dtype, device=DEV)
    ops.difference_heads(att.to(DEV), H, d, vdim, 0.7, 0.45, 1e-4, out=out)
    _close(out.view(11, H, vdim), want, _tol(dtype), "no gate")
    ops.difference_heads(att.to(DEV), H, d, vdim, 0.7, 0.45, 1e-4, out=out, gate=gate.to(DEV)[:, 1:1 + H])
    _close(out.view(11, H, vdim), want * torch.sigmoid(gate[:, 1:1 + H].double()).unsqueeze(2), _tol(dtype), "gate")


# ---- latents from one product, a gate where values are made --------------------------------------------------------------
@pytest.mark.parametrize("qr, rank, rot, page", [(80, 64, 16, 16), (19, 27, 6, 4), (768, 512, 64, 16), (8, 136, 0, 8)])
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("terms", [1, 2, 9])
def test_query_latents_latents_and_key_parts_from_one_product(qr, rank, rot, page, dtype, terms):
    g = torch.Generator().manual_seed(qr)
    n, at = 9, -(-qr // 8) * 8
    width = at + rank + rot + 5
    proj = 2 * torch.randn((n, width), generator=g)
    src = proj.to(DEV) if dtype == F32 or terms > 1 else proj.to(BF).to(DEV)
    ref = (proj if src.dtype == F32 else proj.to(BF)).double()
    if terms > 1:
        src = torch.stack([proj / terms] * terms)
        src[0] += proj - src.sum(0)
        src = src.to(DEV)
    qn, cn = (1 + 0.3 * torch.randn(qr, generator=g)).to(dtype), (1 + 0.3 * torch.randn(rank, generator=g)).to(dtype)
    positions = [5 + i for i in range(n)]
    freqs, _ = plain.pair_frequencies(rot, 100.0) if rot else ([], 1.0)
    table = _table(n, freqs, 1.0, positions) if rot else None
    pages = 4
    slots = torch.randperm(pages * page, generator=g)[:n].tolist()
    slots[3] = -1
    c, kr = torch.full((pages, page, rank), 9.0, dtype=dtype, device=DEV), torch.full((pages, page, rot), 9.0, dtype=dtype, device=DEV)
    cq = torch.empty((n, qr), dtype=dtype, device=DEV)
    ops.latent_inputs(src, qn.to(DEV), 1e-5, cq, at, cn.to(DEV), table, _i32(slots), c, kr, rank, rot)
    _close(cq, plain.rms(ref[:, :qr], 1e-5) * qn.double(), _tol(dtype), "query latents")
    lat = plain.rms(ref[:, at:at + rank], 1e-5) * cn.double()
    part = ref[:, at + rank:at + rank + rot]
    if rot:      # neighbours turn: the plain turn of halves, the dims reordered
        order = [j // 2 + (j % 2) * (rot // 2) for j in range(rot)]
        halves = torch.empty_like(part)
        halves[:, order] = part
        part = _turned(halves.view(n, 1, rot), freqs, 1.0, positions)[:, 0][:, order]
    used = torch.zeros(pages * page, dtype=torch.bool)
    for t, s in enumerate(slots):
        if s >= 0:
            used[s] = True
            _close(c.view(-1, rank)[s], lat[t], _tol(dtype), "latent")
            if rot:
                _close(kr.view(-1, rot)[s], part[t], _tol(dtype), "key part")
    assert bool((c.view(-1, rank).cpu()[~used].float() == 9.0).all())
    alone = torch.empty_like(cq)
    ops.latent_inputs(src, qn.to(DEV), 1e-5, alone)
    assert torch.equal(alone, cq)


@pytest.mark.parametrize("heads, dim, rot, rank, n", [(3, 24, 8, 64, 5), (12, 128, 64, 512, 40), (2, 16, 16, 72, 17), (4, 40, 0, 24, 1)])
def test_queries_carried_through_the_keys_projection_from_partial_sums(heads, dim, rot, rank, n):
    """The plain product of a query and any key (W_uk c | turned part) is that of the carried query and (c | turned part)."""
    g = torch.Generator().manual_seed(rank)
    q = torch.randn((n, heads * (dim + rot)), generator=g).to(BF).float()
    uk = (torch.randn((heads * dim, rank), generator=g) / dim ** 0.5).to(BF)
    uk_t = uk.view(heads, dim, rank).transpose(1, 2).contiguous()
    positions = [2 + 3 * i for i in range(n)]
    freqs, _ = plain.pair_frequencies(rot, 100.0) if rot else ([], 1.0)
    table = _table(n, freqs, 1.0, positions) if rot else None
    per = q.double().view(n, heads, dim + rot)
    want = torch.einsum("nhd,hdr->nhr", per[..., :dim], uk.double().view(heads, dim, rank))
    if rot:
        order = [j // 2 + (j % 2) * (rot // 2) for j in range(rot)]
        halves = torch.empty_like(per[..., dim:])
        halves[..., order] = per[..., dim:]
        want = torch.cat([want, _turned(halves, freqs, 1.0, positions)[..., order]], dim=-1)
    assert ops.latent_query_cores(uk_t.to(DEV), heads, dim, rot)
    for S in (1, 3, 8):
        stack = torch.randn((S, n, q.shape[1]), generator=g)
        stack[-1] += q - stack.sum(0)
        for dtype in (F32, BF):
            out = torch.full((n, heads, rank + rot), float("nan"), dtype=dtype, device=DEV)
            ops.latent_query(stack.to(DEV), uk.to(DEV), table, heads, dim, rank, rot, out=out, w_uk_t=uk_t.to(DEV))
            _close(out, want, 1e-2, (S, dtype))
    for dtype in (F32, BF):      # whole rows, few and many
        many = torch.cat([q] * 40)
        t2 = torch.cat([table] * 40) if rot else None
        out = torch.empty((40 * n, heads, rank + rot), dtype=BF, device=DEV)
        ops.latent_query(many.to(DEV).to(dtype), uk.to(DEV), t2, heads, dim, rank, rot, out=out, w_uk_t=uk_t.to(DEV))
        _close(out.view(40, n, heads, -1)[17], want, 1e-2, dtype)
    two = ops.latent_query(q.to(DEV), uk.to(DEV), table, heads, dim, rank, rot, out=torch.empty((n, heads, rank + rot), device=DEV), w_uk_t=uk_t.to(DEV))
    _close(two, want, 1e-2, "few")


@pytest.mark.parametrize("heads, vdim, rank, n", [(3, 40, 64, 5), (3, 72, 64, 300), (12, 128, 512, 40), (2, 18, 24, 17)])
def test_values_gated_where_they_are_made(heads, vdim, rank, n):
    g = torch.Generator().manual_seed(rank)
    o = torch.randn((n, heads, rank), generator=g).to(BF).float()
    uv = (torch.randn((heads * vdim, rank), generator=g) / rank ** 0.5).to(BF)
    gate = torch.randn((n, heads * vdim + 8), generator=g)
    want = torch.einsum("nhr,hvr->nhv", o.double(), uv.double().view(heads, vdim, rank)).reshape(n, -1) * torch.sigmoid(gate[:, :-8].double())
    assert ops.latent_value_gates(uv.to(DEV), heads, rank)
    full = gate.to(DEV)
    stack = torch.stack([full * 0.25, full * 0.75])
    for gt, tol in ((full[:, :-8], 1e-2), (full.to(BF)[:, :-8], 2e-2), (stack[..., :-8], 1e-2)):
        out = ops.latent_value(o.to(DEV), uv.to(DEV), vdim, out=torch.empty((n, heads * vdim), dtype=BF, device=DEV), gate=gt)
        _close(out, want, tol)
    with pytest.raises(ValueError):
        ops.latent_value(o[..., :rank - 4].contiguous().to(DEV), uv.float()[:, :rank - 4].contiguous().to(DEV), vdim,
                         out=torch.empty((n, heads * vdim), device=DEV), gate=full[:, :-8])


# ---- the activation alone -------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("I", [64, 83, 1028])
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("activation", sorted(ops.ACTIVATIONS))
def test_the_activation(I, dtype, activation):
    g = torch.Generator().manual_seed(I)
    z = 4 * torch.randn((7, I), generator=g)
    z[0, :4] = torch.tensor([-200.0, 200.0, 0.0, -9.0])
    fn = {"gelu_tanh": plain.gelu, "silu": lambda t: t * torch.sigmoid(t), "relu2": lambda t: torch.relu(t) ** 2,
          "gelu_erf": torch.nn.functional.gelu}[activation]
    for terms in (1, 3, 11, 18):
        src = z.to(DEV).to(dtype) if terms == 1 else torch.stack([z / terms] * terms).to(DEV)
        ref = src.double().cpu() if terms == 1 else src.double().cpu().sum(0)
        out = ops.activate(src, activation, out=torch.empty((7, I), dtype=dtype, device=DEV))
        _close(out, fn(ref), 1e-6 if dtype == F32 else 5e-3, (activation, terms))
        assert torch.isfinite(out).all()


@pytest.mark.parametrize("M,N,K,bias", [(1, 83, 64, True), (16, 256, 200, False), (33, 8960, 256, False), (64, 400, 1536, True)])
@pytest.mark.parametrize("activation", [a for a in sorted(ops.ACTIVATIONS) if a != "gelu_erf"])
def test_the_activation_in_the_products_epilogue(M, N, K, bias, activation):
    g = torch.Generator().manual_seed(M * N)
    x, w = torch.randn((M, K), generator=g).to(BF), (3 * torch.randn((N, K), generator=g) / K ** 0.5).to(BF)
    b = torch.randn(N, generator=g).to(BF) if bias else None
    z = x.double() @ w.double().T + (b.double() if bias else 0.0)
    fn = {"gelu_tanh": plain.gelu, "silu": lambda t: t * torch.sigmoid(t), "relu2": lambda t: torch.relu(t) ** 2}[activation]
    out = torch.full((M, N + 5), 9.0, dtype=BF, device=DEV)[:, :N]
    ops.linear_activated(x.to(DEV), w.to(DEV), activation, bias=None if b is None else b.to(DEV), out=out)
    _close(out, fn(z), 1e-2, (activation, M, N, K))
    assert (out.untyped_storage().nbytes() == M * (N + 5) * 2) and bool((torch.as_strided(out, (M, 5), (N + 5, 1), N) == 9.0).all())


def test_where_the_products_epilogue_pays():
    x = lambda M, K: torch.zeros((M, K), dtype=BF, device=DEV)
    w = lambda N, K: torch.zeros((N, K), dtype=BF, device=DEV)
    assert ops.linear_activated_supported(x(8, 1536), w(8960, 1536), "gelu_tanh")
    assert not ops.linear_activated_supported(x(65, 1536), w(8960, 1536), "gelu_tanh")       # more rows than it takes
    assert not ops.linear_activated_supported(x(8, 8192), w(512, 8192), "gelu_tanh")         # few weight rows, much k: better cut
    assert not ops.linear_activated_supported(x(8, 1536), w(8960, 1536), "gelu_erf")
    assert not ops.linear_activated_supported(x(8, 1536).float(), w(8960, 1536).float(), "gelu_tanh")
    with pytest.raises(ValueError):
        ops.linear_activated(x(65, 64), w(64, 64), "silu")
