"""Each Minerax mechanism alone (package op on CPU tensors or the gfx950 kernel) against the slow
oracle, with inputs made so that a key, a sink, a stream or a state missed or wrongly seen shows."""
import math

import pytest
import torch

from replisense_rfq_amd import ops

from . import oracle

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
BS = 32
D64 = torch.float64


def close(a, b, tol=2e-5):
    a, b = a.double().cpu(), b.double().cpu()
    assert a.shape == b.shape, (a.shape, b.shape)
    assert float((a - b).abs().max()) <= tol * max(1.0, float(b.abs().max())), \
        float((a - b).abs().max())


def i32(x, device):
    return torch.tensor(x, dtype=torch.int32, device=device)


def run_rows(cuts, slot):
    """(first row, rows, (row_state, row_back, row_fwd, positions)) of every portion of one
    sequence; the state half alternates as the scheduler alternates it."""
    at = 0
    for gen, n in enumerate(cuts):
        yield at, n, ([2 * slot + (gen & 1)] * n, list(range(n)), list(range(n - 1, -1, -1)),
                      list(range(at, at + n)))
        at += n


# ------------------------------------------------------------------ residual streams
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 8])
@pytest.mark.parametrize("d", [37, 44, 256, 2052])
def test_streams_update_weighted_sum_and_norm(device, S, d):
    """Every new stream is formed from the previous ones (row s of mix: what stream s gives); the
    next sublayer reads the layer norm of a weighted sum."""
    g = torch.Generator().manual_seed(1)
    T, eps = 5, 1e-3
    x = torch.randn(T, S, d, generator=g) * 3 + 1.5
    y = torch.randn(T, d + 3, generator=g)[:, :d] - 0.5
    mix, wo = torch.randn(S, S, generator=g), torch.randn(S, generator=g)
    wi, w = torch.randn(S, generator=g), torch.randn(d, generator=g)
    old = x.double().transpose(0, 1)
    new = oracle.streams_update(old, mix.double(), wo.double(), y.double())
    want = oracle.layer_norm(oracle.streams_in(new, wi.double()), w.double(), eps)
    dev = [t.to(device) for t in (mix, wo, wi, w)]
    for dtype, tol in ((torch.float32, 3e-5), (torch.bfloat16, 1e-2)):
        yy = y.to(dtype)
        ref_new = new if dtype == torch.float32 else \
            oracle.streams_update(old, mix.double(), wo.double(), yy.double())
        xd, out = x.clone().to(device), torch.empty(T, d, dtype=dtype, device=device)
        ops.streams_norm(xd, yy.to(device), *dev[:2], dev[2], dev[3], eps, out=out)
        close(xd.transpose(0, 1), ref_new, 1e-5)
        close(out, oracle.layer_norm(oracle.streams_in(ref_new, wi.double()), w.double(), eps), tol)
        # without keep the result is the same (the streams are not needed any more)
        out2 = torch.empty_like(out)
        ops.streams_norm(x.clone().to(device), yy.to(device), *dev[:2], dev[2], dev[3], eps, out=out2,
                         keep=False)
        close(out2, out, 0)
    if S > 1:                                            # the transposed matrix gives something else
        other = oracle.streams_update(old, mix.double().T, wo.double(), y.double())
        assert float((oracle.layer_norm(oracle.streams_in(other, wi.double()), w.double(), eps) - want).abs().max()) > 1e-2


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("centre", [True, False])
def test_streams_start_from_the_embedding(device, centre):
    g = torch.Generator().manual_seed(2)
    S, d, eps = 3, 50, 1e-4
    table = (torch.randn(21, d, generator=g) + 0.7).bfloat16()
    ids = [5, 0, 20, 5]
    wi, w = torch.randn(S, generator=g), torch.randn(d, generator=g)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        x = torch.full((4, S, d), 9.0, device=device)
        out = torch.empty(4, d, dtype=dtype, device=device)
        ops.streams_norm(x, w_in=wi.to(device), w=w.to(device), eps=eps, centre=centre, out=out,
                         ids=i32(ids, device), table=table.to(dtype).to(device))
        e = table.double()[ids]
        close(x, e[:, None].expand(4, S, d), 0)
        u = oracle.streams_in(e[None].expand(S, 4, d), wi.double())
        close(out, oracle.layer_norm(u, w.double(), eps) if centre else oracle.over_rms(u, eps) * w.double(), tol)


@pytest.mark.parametrize("device", DEVICES)
def test_layer_norm_of_rows_far_from_zero(device):
    """A mean a thousand times the deviation: the squares are those of the deviations."""
    g = torch.Generator().manual_seed(3)
    T, d = 3, 128
    x = (torch.randn(T, 1, d, generator=g) + 1000.0)
    one, w = torch.ones(1), torch.randn(d, generator=g)
    out = torch.empty(T, d, device=device)
    ops.streams_norm(x.to(device), w_in=one.to(device), w=w.to(device), eps=1e-5, out=out)
    close(out, oracle.layer_norm(x[:, 0].double(), w.double(), 1e-5), 2e-3)


# ------------------------------------------------------------------ feed-forward unit, gate
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("F", [5, 64, 3000])
def test_gated_tanh_gelu(device, F):
    g = torch.Generator().manual_seed(4)
    x = torch.randn(4, 2 * F + 8, generator=g) * 4
    x[0, 0], x[0, 1] = 30.0, -30.0
    for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 1e-2)):
        xd = x.to(dtype)
        got = ops.gelu_glu_rows(xd.to(device)[:, :2 * F])
        close(got, oracle.gelu_tanh(xd[:, :F].double()) * xd[:, F:2 * F].double(), tol)
    z = torch.linspace(-6, 6, 400)[None]
    got = ops.gelu_glu_rows(torch.cat([z, torch.ones_like(z)], 1).to(device))
    close(got, oracle.gelu_tanh(z.double()), 1e-6)
    erf = 0.5 * z.double() * (1.0 + torch.erf(z.double() / math.sqrt(2.0)))
    assert float((got.double().cpu() - erf).abs().max()) > 1e-4          # not the exact gelu


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,n", [(3, 7), (4, 16), (1, 1), (5, 8)])
def test_heads_side_by_side_times_the_gate(device, H, n):
    g = torch.Generator().manual_seed(5)
    T = 6
    x = torch.randn(H, T, n, generator=g)
    wide = torch.randn(T, H * n + 11, generator=g) * 2
    for lo in (8, 3):
        for dtype, tol in ((torch.float32, 1e-6), (torch.bfloat16, 1e-2)):
            xd, gd = x.to(dtype), wide.to(dtype)[:, lo:lo + H * n]
            got = ops.gate_heads(xd.to(device), wide.to(dtype).to(device)[:, lo:lo + H * n],
                                 torch.empty(T, H * n, dtype=dtype, device=device))
            want = xd.double().transpose(0, 1).reshape(T, H * n) * oracle.sigmoid(gd.double())
            close(got, want, tol)


# ------------------------------------------------------------------ frequencies
def test_scaled_frequencies_against_the_oracle():
    for dims, base, sc in ((20, 30000.0, dict(factor=6.0, original=512, fast=16.0, slow=1.0)),
                           (8, 300.0, dict(factor=3.0, original=40, fast=8.0, slow=1.0)),
                           (6, 50.0, dict(factor=2.0, original=1000, fast=0.5, slow=0.4)),   # lo = hi
                           (12, 10000.0, dict(factor=5.0, original=6, fast=64.0, slow=32.0)),  # lo at 0
                           (4, 1e6, dict(factor=1.0, original=4096, fast=32.0, slow=1.0)),
                           (10, 700.0, None)):
        scaling = () if sc is None else ("yarn", sc["factor"], float(sc["original"]), sc["fast"], sc["slow"])
        f, mult = ops.rotary_scaled_freq(dims, base, scaling)
        wf, wm = oracle.frequencies({"dims": dims, "base": base, "scaling": sc})
        close(f, wf, 1e-7)
        assert abs(mult - wm) < 1e-12


# ------------------------------------------------------------------ convolution, norms, rotation, pages
def _page_rows(cache, slots):
    return torch.stack([cache[s // BS, :, s % BS] for s in slots]).cpu()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,dim,vdim,rot", [(4, 2, 16, 8, 8), (3, 3, 10, 6, 4), (8, 2, 32, 40, 32), (2, 1, 6, 5, 0)])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6])
def test_convolved_rows_normed_and_rotated(device, H, G, dim, vdim, rot, taps):
    """q, k and v pass the convolution (no activation) before norm and rotation, in portions
    through a slot with another sequence's rest; v is convolved only.  The first tokens see
    zeros, portions shorter than the taps keep what lies further back."""
    g = torch.Generator().manual_seed(6)
    cuts = [2, 1, 1, 9, 1, 2, 40]
    T, eps, slots_n, slot = sum(cuts), 1e-4, 3, 2
    nq, nk = H * dim, G * dim
    W = nq + nk + G * vdim
    pad = 8 if dim % 8 == 0 and vdim % 8 == 0 else 5
    wide = torch.randn(T, W + pad, generator=g)
    w = torch.randn(W, taps, generator=g)
    qn, kn = torch.randn(nq, generator=g), torch.randn(nk, generator=g)
    rcfg = {"dims": rot, "base": 777.0, "scaling": dict(factor=3.0, original=40, fast=8.0, slow=1.0)}
    f, mult = ops.rotary_scaled_freq(rot, 777.0, ("yarn", 3.0, 40.0, 8.0, 1.0), device)
    kc = torch.full((4, G, BS, dim), 9.0, device=device)
    vc = torch.full((4, G, BS, vdim), 9.0, device=device)
    page = [3, 1]
    state = (torch.randn(2 * slots_n, taps - 1, W, generator=g) * 100).to(device)
    other = state.clone()
    wt = w.t().contiguous().to(device)
    qs, wheres = [], []
    for lo, n, rows in run_rows(cuts, slot):
        where = [page[p // BS] * BS + p % BS for p in rows[3]]
        wheres += where
        q = torch.empty(n, H, dim, device=device)
        r = [i32(x, device) for x in rows]
        ops.qk_norm_rotary_append(wide.to(device)[lo:lo + n], None, qn.to(device), kn.to(device), True, dim, eps,
                                  r[3], f, mult, 0, 0, i32(where, device), kc, vc, H, G, dim, dim, vdim, 0, q,
                                  conv=(wt, state, *r[:3]))
        qs.append(q.cpu())
    c = oracle.causal_conv(wide[:, :W].double(), w.double())
    pos = torch.arange(T)
    wf, wm = oracle.frequencies(rcfg)
    wq = oracle.rotate((oracle.over_rms(c[:, :nq], eps) * qn.double()).view(T, H, dim), pos, wf, wm, False)
    wk = oracle.rotate((oracle.over_rms(c[:, nq:nq + nk], eps) * kn.double()).view(T, G, dim), pos, wf, wm, False)
    close(torch.cat(qs), wq, 3e-5)
    close(_page_rows(kc, wheres), wk, 3e-5)
    close(_page_rows(vc, wheres), c[:, nq + nk:].view(T, G, vdim), 3e-5)
    keep = [i for i in range(2 * slots_n) if i % slots_n != slot]      # other slots are untouched
    assert torch.equal(state[keep].cpu(), other[keep].cpu())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,dim,rd,R", [(3, 12, 8, 24), (2, 6, 6, 14), (8, 32, 16, 64), (5, 7, 3, 9)])
def test_latent_row_and_neighbouring_pairs(device, H, dim, rd, R):
    """Only the trailing part of every query head is rotated, in neighbouring pairs (an odd last
    entry stays); it goes to a slice of wider rows.  The page row is [normed latent | rotated
    key part].  Half-split pairs give something else."""
    g = torch.Generator().manual_seed(7)
    pos = [0, 1, 2, 40, 41, 500]
    slots = [5 * BS, 5 * BS + 1, 2 * BS + 31, -1, 3 * BS + 7, BS + 2]
    T, eps = len(pos), 1e-4
    nq = H * (dim + rd)
    proj = torch.randn(T, nq + R + rd + 5, generator=g)
    nw = torch.randn(R, generator=g)
    rot = rd // 2 * 2
    rcfg = {"dims": rot, "base": 300.0, "scaling": dict(factor=3.0, original=40, fast=8.0, slow=1.0)}
    f, mult = ops.rotary_scaled_freq(rot, 300.0, ("yarn", 3.0, 40.0, 8.0, 1.0), device)
    x, p = proj.double(), torch.tensor(pos)
    wf, wm = oracle.frequencies(rcfg)
    heads = x[:, :nq].view(T, H, dim + rd)
    kv = x[:, nq:nq + R + rd]
    for full in (False, True):
        pool = torch.full((6, 1, BS, R + rd), 9.0, device=device)
        q = torch.full((T, H, R + rd), 7.0, device=device)
        out = torch.empty(T, H, dim + rd, device=device) if full else q[:, :, R:]
        ops.qk_norm_rotary_append(proj.to(device), None, None, nw.to(device), False, R, eps, i32(pos, device), f,
                                  mult, dim, R, i32(slots, device), pool, None, H, 1, dim + rd, R + rd, 0, 2, out,
                                  neighbours=True)
        want = oracle.rotate(heads[..., dim:], p, wf, wm, True)
        if full:
            close(out[..., :dim], heads[..., :dim], 0)
            close(out[..., dim:], want, 1e-5)
        else:
            close(q[..., R:], want, 1e-5)
            assert float((q[..., :R] - 7.0).abs().max()) == 0.0
        live = [i for i, s in enumerate(slots) if s >= 0]
        row = torch.cat([oracle.over_rms(kv[:, :R], eps) * nw.double(),
                         oracle.rotate(kv[:, None, R:], p, wf, wm, True)[:, 0]], -1)
        close(_page_rows(pool, [slots[i] for i in live])[:, 0], row[live], 1e-5)
        assert float(pool[0].min()) == 9.0
    if rot >= 4:
        assert float((oracle.rotate(heads[..., dim:], p, wf, wm, False) - want).abs().max()) > 0.1


@pytest.mark.parametrize("device", DEVICES)
def test_batched_product_into_a_slice(device):
    """The latent queries' product writes the leading columns of wider rows."""
    g = torch.Generator().manual_seed(8)
    T, H, dim, R, rd = 9, 3, 8, 24, 8
    pr, uk = torch.randn(T, H * 16, generator=g), torch.randn(H, dim, R, generator=g)
    for dtype in (torch.float32, torch.bfloat16):
        a, b = pr.to(dtype), uk.to(dtype)
        q = torch.full((T, H, R + rd), 7.0, device=device)
        ops.bmm_f32(a.to(device).unflatten(1, (H, 16))[:, :, :dim].transpose(0, 1), b.to(device),
                    out=q[:, :, :R].transpose(0, 1))
        for h in range(H):
            close(q[:, h, :R], a[:, 16 * h:16 * h + dim].double() @ b[h].double(), 1e-5)
        assert float((q[..., R:] - 7.0).abs().max()) == 0.0


# ------------------------------------------------------------------ attention
ORDER = [4, 0, 9, 2, 7, 1, 8, 3, 6, 5, 10, 11, 12, 13, 14]


def _attend(device, q, k, v, vdim, sections, scale, window=0, sink=None, softcap=0.0, out_mult=1.0,
            dtype=torch.float32, mfma=None, short=False):
    """sections: [(first row, rows)] of ONE sequence, each its own launch with everything before it
    cached in pages that lie in odd order; v None: the values are the keys' leading entries."""
    L, H = q.shape[:2]
    G, nb = k.shape[1], (L + BS - 1) // BS
    order = ORDER[:nb]
    blocks = max(order) + 2
    kc = torch.full((blocks, G, BS, k.shape[2]), 7.0, dtype=dtype)
    vc = kc if v is None else torch.full((blocks, G, BS, vdim), 7.0, dtype=dtype)
    for j in range(L):
        kc[order[j // BS], :, j % BS] = k[j].to(dtype)
        if v is not None:
            vc[order[j // BS], :, j % BS] = v[j].to(dtype)
    kc = kc.to(device)
    vc = kc if v is None else vc.to(device)
    bt = i32([order + [blocks - 1] * 3], device)
    out = torch.zeros(L, H * vdim + 8, dtype=dtype, device=device)[:, :H * vdim]     # a slice of wider rows
    sk = None if sink is None else sink.float().to(device)
    for lo, n in sections:
        nblk = (n + ops.KEEP_QBLK - 1) // ops.KEEP_QBLK
        ops.attn_keep_window(q[lo:lo + n].float().contiguous().to(device), kc, vc, vdim, bt,
                             i32([0], device), i32([n], device), i32([lo + n], device),
                             i32([0] * nblk, device), i32(list(range(nblk)), device), sk, None,
                             out[lo:lo + n], scale, window, short_rows=32 if (short and n <= 32) else 0,
                             mfma=mfma, softcap=softcap, out_mult=out_mult)
    return out


def _dense(q, k, v, scale, window=0, sink=None, softcap=0.0, out_mult=1.0):
    L, H = q.shape[:2]
    ok = oracle.visible(L, window)
    out = torch.zeros(L, H, v.shape[2], dtype=D64)
    for h in range(H):
        c = h // (H // k.shape[1])
        s = oracle.cap((q[:, h].double() @ k[:, c].double().T) * scale, softcap)
        out[:, h] = oracle.weights(s, ok, None if sink is None else sink[h].double()) @ v[:, c].double() * out_mult
    return out.reshape(L, -1)


SECTIONS = [(0, 70), (70, 3), (73, 45)] + [(118 + i, 1) for i in range(32)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 16, 8), (3, 3, 40, 24), (2, 1, 7, 9)])
@pytest.mark.parametrize("softcap", [0.5, 3.0, 50.0])
def test_capped_attention_in_sections(device, H, G, dim, vdim, softcap):
    """A prompt portion, a short extend and decoded rows (work-item kernel and grouped decode
    kernel); scores well beyond the cap; the cap comes after the scale and before the mask."""
    g = torch.Generator().manual_seed(9)
    L, scale = 150, 0.9
    q, k = torch.randn(L, H, dim, generator=g), torch.randn(L, G, dim, generator=g)
    v = torch.randn(L, G, vdim, generator=g)
    want = _dense(q, k, v, scale, softcap=softcap, out_mult=0.6)
    for short in (False, True):
        close(_attend(device, q, k, v, vdim, SECTIONS, scale, softcap=softcap, out_mult=0.6, short=short), want, 5e-5)
    if softcap < 10:
        assert float((_dense(q, k, v, scale, out_mult=0.6) - want).abs().max()) > 0.05


@pytest.mark.parametrize("device", DEVICES)
def test_far_key_among_hundreds_under_the_cap(device):
    """One score stands out of hundreds; the cap takes it down to a known share."""
    g = torch.Generator().manual_seed(10)
    L, H, G, dim, vdim, cap = 450, 2, 2, 8, 8, 8.0
    q, k = torch.randn(L, H, dim, generator=g) * 0.1, torch.randn(L, G, dim, generator=g) * 0.1
    v = torch.zeros(L, G, vdim)
    q[L - 1, 1, 1] = k[3, 1, 1] = 5.0
    v[3, 1] = 50.0
    want = _dense(q, k, v, 1.0, softcap=cap)
    for sections, short in (([(0, L)], False), ([(0, L - 1), (L - 1, 1)], True), ([(0, L - 1), (L - 1, 1)], False)):
        got = _attend(device, q, k, v, vdim, sections, 1.0, softcap=cap, short=short)
        close(got, want, 5e-5)
        assert 40.0 < float(got[L - 1, vdim]) < 46.0               # exp(8 tanh(25 / 8)) beside 449 keys near 1
    assert float(_dense(q, k, v, 1.0)[L - 1, vdim]) > 49.9


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("R,rd,H", [(24, 8, 3), (15, 10, 5), (64, 32, 8)])
@pytest.mark.parametrize("window", [1, 5, 32, 33, 100])
def test_windowed_latent_attention_with_sinks(device, R, rd, H, window):
    g = torch.Generator().manual_seed(11)
    L = 150
    q, k = torch.randn(L, H, R + rd, generator=g), torch.randn(L, 1, R + rd, generator=g)
    sink = torch.randn(H, generator=g)
    want = _dense(q, k, k[..., :R], 0.3, window, sink)
    for short in (False, True):
        close(_attend(device, q, k, None, R, SECTIONS, 0.3, window, sink, short=short), want, 5e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 65, 97])
@pytest.mark.parametrize("decoded", [False, True])
def test_a_latent_at_the_window_edge_stands_out(device, window, decoded):
    """One cached row matches the last query and carries a value far from the others: on the
    window's last position it shows in the output, one position further out it must not.  The
    sink takes its share once."""
    g = torch.Generator().manual_seed(12)
    L, H, R, rd = 140, 2, 8, 8
    sink = torch.tensor([0.0, 9.0])
    for inside in (True, False):
        q, k = torch.randn(L, H, R + rd, generator=g) * 0.1, torch.randn(L, 1, R + rd, generator=g) * 0.1
        j = L - 1 - (window - 1) - (0 if inside else 1)
        q[L - 1, :, R] = k[j, 0, R] = 3.0
        k[j, 0, 0] = 100.0
        q[:, :, 0] = 0.0
        want = _dense(q, k, k[..., :R], 1.0, window, sink)
        got = _attend(device, q, k, None, R, [(0, L - 1), (L - 1, 1)] if decoded else [(0, L)], 1.0, window, sink,
                      short=decoded)
        close(got, want, 5e-5)
        assert (float(got[L - 1, 0]) > 50.0) == inside, (window, inside)
        if inside:
            assert 40.0 < float(got[L - 1, R]) < 60.0              # a sink as large as the score: half


# ------------------------------------------------------------------ MFMA tiles
@pytest.mark.gpu
@pytest.mark.parametrize("H,G,E,vdim,shared", [(4, 2, 32, 32, False), (6, 2, 64, 64, False), (3, 3, 128, 128, False),
                                               (4, 1, 96, 64, True), (16, 1, 96, 64, True), (5, 1, 128, 96, True),
                                               (32, 1, 128, 96, True), (4, 1, 128, 64, True),
                                               (2, 1, 320, 256, True)])
@pytest.mark.parametrize("softcap", [0.0, 2.0, 30.0])
@pytest.mark.parametrize("window", [0, 1, 33, 70])
def test_attention_on_mfma_tiles(H, G, E, vdim, shared, softcap, window):
    """bf16 pages with sizes of the MFMA tiles: prompt portions cut inside pages and query blocks
    and decoded rows against the dense computation on the same (rounded) keys and values."""
    assert ops.keep_mfma_ok(E, vdim, shared=shared)
    g = torch.Generator().manual_seed(13)
    L, scale = 150, E ** -0.5 * 3
    q = torch.randn(L, H, E, generator=g)
    k = torch.randn(L, G, E, generator=g).bfloat16().float()
    v = None if shared else torch.randn(L, G, vdim, generator=g).bfloat16().float()
    sink = torch.randn(H, generator=g) if shared else None
    want = _dense(q, k, k[..., :vdim] if shared else v, scale, window, sink, softcap, 0.7)
    for short in (False, True):
        got = _attend("cuda", q, k, v, vdim, SECTIONS, scale, window, sink, softcap, 0.7, torch.bfloat16, short=short)
        close(got, want, 6e-3)


# ------------------------------------------------------------------ delta rule into a slice of wider rows
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,dim,vdim", [(2, 2, 32, 64), (4, 2, 64, 32), (3, 1, 7, 5), (2, 1, 128, 40), (4, 4, 16, 16),
                                          (2, 2, 96, 48), (1, 1, 48, 130)])
@pytest.mark.parametrize("cuts", [[40], [2, 1, 33, 4], [150, 3, 1]])
def test_delta_rule_in_portions(device, H, G, dim, vdim, cuts):
    """The recurrence through a state slot with stale contents, results in a column slice of a
    wider matrix whose other columns stay; the state left behind is the oracle's."""
    g = torch.Generator().manual_seed(14)
    T, S, slot, eps = sum(cuts), 2, 1, 1e-4
    q, v = torch.randn(T, G, dim, generator=g), torch.randn(T, H, vdim, generator=g)
    q = oracle.unit_vectors(q.double()).float()
    k = oracle.unit_vectors(torch.randn(T, G, dim, generator=g).double()).float()
    z, gate = torch.randn(T, H * dim, generator=g) * 2, torch.randn(T, H * vdim, generator=g)
    beta = torch.randn(T, H, generator=g)
    zb, nw = torch.randn(H * dim, generator=g), torch.randn(vdim, generator=g)
    a_log = torch.randn(H, generator=g) * 0.5 - 0.5
    dec = oracle.channel_decay((z.double() + zb.double()).view(T, H, dim), a_log.double())
    o, last = torch.zeros(T, H, vdim, dtype=D64), []
    for h in range(H):
        c = h // (H // G)
        o[:, h], s = oracle.delta_scan(q[:, c].double() * dim ** -0.5, k[:, c].double(), v[:, h].double(), dec[:, h],
                                       oracle.sigmoid(beta[:, h].double()))
        last.append(s)
    want = (oracle.over_rms(o, eps) * nw.double()).reshape(T, -1) * oracle.sigmoid(gate.double())
    state = (torch.randn(2 * S, H, dim, vdim, generator=g) * 50).to(device)
    other = state.clone()
    y = torch.full((T, H * vdim + 24), 5.0, device=device)
    dev = [x.to(device) for x in (q, k, v, z, torch.exp(a_log.double()).float(), zb, beta, gate, nw)]
    for lo, n, rows in run_rows(cuts, slot):
        hi = lo + n
        ops.gated_linear_recurrence(dev[0][lo:hi], dev[1][lo:hi], dev[2][lo:hi], dev[3][lo:hi].clone(), dev[4], dev[5],
                                    1.0, dev[6][lo:hi], dev[7][lo:hi], True, dev[8], eps, dim ** -0.5, state,
                                    *(i32(x, device) for x in rows), y[lo:hi, 16:16 + H * vdim],
                                    i32([0], device) if device != "cpu" else None)
    close(y[:, 16:16 + H * vdim], want, 1e-4)
    assert float((y[:, :16] - 5.0).abs().max()) == 0.0 == float((y[:, 16 + H * vdim:] - 5.0).abs().max())
    half = 1 - ((len(cuts) - 1) & 1)
    close(state[half * S + slot], torch.stack(last), 1e-4)
    close(state[0], other[0], 0)
    close(state[S], other[S], 0)
