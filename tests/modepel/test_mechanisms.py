"""Each Modepel mechanism alone (package op on CPU tensors or the gfx950 kernel) against the slow
oracle, with inputs made so that a key, the added one, a blend or a state missed or wrongly seen
shows."""
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
    assert float((a - b).abs().max()) <= tol * max(1.0, float(b.abs().max())), \
        float((a - b).abs().max())


def i32(x, device):
    return torch.tensor(x, dtype=torch.int32, device=device)


# ------------------------------------------------------------------ stream and norms
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("d", [37, 44, 256, 1028, 1030, 2052, 4100, 8196])
def test_gain_sandwich(device, d):
    """x += g_post rms(y + sigmoid(s) y2 + w h) ; out = g_pre rms(x), each part optional, mixed
    types, strided inputs, out in the place of h."""
    g = torch.Generator().manual_seed(1)
    T, eps, gp, gn = 5, 1e-2, 0.7, 1.3
    x = torch.randn(T, d, generator=g) * 3
    y = torch.randn(T, d, generator=g)
    y2 = (torch.randn(T, d, generator=g) * 2).bfloat16()
    wide = torch.randn(T, d + 4, generator=g)
    h = wide[:, :d]
    z = torch.randn(T, 3, generator=g)
    w = torch.rand(T, generator=g)
    for use in ("y", "y2", "h", "y y2 h", "y h", ""):
        p, want = {}, torch.zeros(T, d, dtype=D64)
        if "y" in use.split():
            p["y"] = y.to(device)
            want = want + y.double()
        if "y2" in use:
            p.update(y2=y2.to(device), y2_logit=z.to(device)[:, 1])
            want = want + y2.double() * oracle.sigmoid(z[:, 1:2].double())
        if "h" in use:
            p.update(h_in=wide.to(device)[:, :d], h_weight=w.to(device))
            want = want + h.double() * w.double()[:, None]
        ref = x.double() + (oracle.gain_norm(want, gp, eps) if use else 0.0)
        for dt in (torch.float32, torch.bfloat16):
            xd, out = x.clone().to(device), torch.empty(T, d, dtype=dt, device=device)
            ops.gain_sandwich(xd, g_post=gp, g_pre=gn, eps=eps, out=out, **p)
            close(xd, ref)
            close(out, oracle.gain_norm(ref, gn, eps), 2e-5 if dt == torch.float32 else 6e-3)
    xd, hh = x.clone().to(device), h.contiguous().to(device)
    ops.gain_sandwich(xd, y.to(device), gp, gn, eps, hh, h_in=hh, h_weight=w.to(device))   # in place
    ref = x.double() + oracle.gain_norm(y.double() + h.double() * w.double()[:, None], gp, eps)
    close(hh, oracle.gain_norm(ref, gn, eps))
    xd = x.clone().to(device)
    ops.gain_sandwich(xd, y.to(device), gp, eps=eps)                                       # no next norm
    close(xd, x.double() + oracle.gain_norm(y.double(), gp, eps))


@pytest.mark.parametrize("device", DEVICES)
def test_norm_eps_lies_inside_the_root(device):
    x = torch.full((2, 64), 1e-3)
    out = torch.empty(2, 64, device=device)
    ops.gain_sandwich(x.clone().to(device), g_pre=1.0, eps=1e-6, out=out)
    close(out, torch.full((2, 64), 1.0 / math.sqrt(2.0)), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("F", [7, 40, 384, 2056, 4104, 10240, 16392])
def test_poly_norm(device, F):
    g = torch.Generator().manual_seed(2)
    z = torch.randn(4, F, generator=g) * torch.tensor([0.01, 1.0, 3.0, 30.0])[:, None]
    for coef in ((0.4, -0.3, 0.6, 0.2), (1.0, 0.0, 0.0, 0.0), (0.0, 1.0, 0.0, 0.0), (0.0, 0.0, 1.0, 0.0),
                 (0.0, 0.0, 0.0, 1.0)):
        want = oracle.poly_norm(z.double(), coef, 1e-4)
        close(ops.poly_norm_rows(z.to(device), coef, 1e-4), want, 1e-5)
        zb = z.bfloat16()
        got = ops.poly_norm_rows(zb.to(device), coef, 1e-4)
        close(got, oracle.poly_norm(zb.double(), coef, 1e-4), 6e-3)
        zd = z.to(device)
        ops.poly_norm_rows(zd, coef, 1e-4, zd)                       # in place
        close(zd, want, 1e-5)


# ------------------------------------------------------------------ rotation, biases, blended values
SLOTS = [3, 70, 31, 32, -1, 100, 5]
POS = [0, 1, 17, 400, 9, 900, 2]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,dim,vdim,rot", [(4, 2, 16, 8, 8), (3, 3, 10, 6, 4), (6, 2, 64, 32, 32),
                                              (2, 1, 8, 24, 0), (1, 1, 6, 5, 6)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_rotation_biases_and_blended_values(device, H, G, dim, vdim, rot, dtype):
    g = torch.Generator().manual_seed(3)
    T, base, lam = len(POS), 700.0, 0.35
    n = (H + G) * dim + G * vdim
    pr = torch.randn(T, n + 8 * ((H * vdim + 7) // 8), generator=g).to(dtype)     # gate columns follow
    b = torch.randn(n, generator=g)
    first = torch.randn(T, G * vdim, generator=g)
    inv, _ = ops.rotary_scaled_freq(rot, base, (), device)
    x = pr.double()[:, :n] + b.double()
    pos = torch.tensor(POS)
    wq = oracle.rotate_half(x[:, :H * dim].view(T, H, dim), pos, rot, base)
    wk = oracle.rotate_half(x[:, H * dim:(H + G) * dim].view(T, G, dim), pos, rot, base)
    v0 = x[:, (H + G) * dim:].view(T, G, vdim)
    tol = 2e-4 if dtype == torch.float32 else 8e-3
    for v_in, take, hand_on in ((None, 0.9, False), (None, 0.9, True), (first, lam, False), (first, 1.0, True)):
        kc = torch.full((5, G, BS, dim), 9.0, dtype=dtype, device=device)
        vc = torch.full((5, G, BS, vdim), 9.0, dtype=dtype, device=device)
        q = torch.empty(T, H, dim, device=device)
        vo = torch.empty(T, G * vdim, device=device) if hand_on else None
        ops.qk_norm_rotary_append(pr.to(device), b.to(device), None, None, False, 0, 1e-6, i32(POS, device),
                                  inv, 1.0, 0, 0, i32(SLOTS, device), kc, vc, H, G, dim, dim, vdim, 0, q,
                                  None if v_in is None else v_in.to(device), take, vo)
        close(q, wq, 2e-4)
        wv = v0 if v_in is None else oracle.mixed_values(v0, v_in.double().view(T, G, vdim), take)
        hold = torch.zeros(5, BS, dtype=torch.bool)
        for t, s in enumerate(SLOTS):
            if s >= 0:
                close(kc[s // BS, :, s % BS], wk[t], tol)
                close(vc[s // BS, :, s % BS], wv[t], tol)
                hold[s // BS, s % BS] = True
        assert bool((kc.cpu().permute(0, 2, 1, 3)[~hold] == 9.0).all())       # nothing else written
        assert bool((vc.cpu().permute(0, 2, 1, 3)[~hold] == 9.0).all())
        if hand_on:
            close(vo, v0.reshape(T, -1), 1e-5)


# ------------------------------------------------------------------ attention
def _dense(q, k, v, scale, gate):
    L, H = q.shape[:2]
    G = k.shape[1]
    pos = torch.arange(L)
    ok = pos[None, :] <= pos[:, None]
    out = torch.zeros(L, H, v.shape[2], dtype=D64)
    for h in range(H):
        c = h // (H // G)
        out[:, h] = oracle.softmax_plus_one((q[:, h].double() @ k[:, c].double().T) * scale, ok) @ v[:, c].double()
    return out.reshape(L, -1) * oracle.sigmoid(gate.double())


def _attend(device, q, k, v, gate, sections, scale, dtype=torch.float32, short=True, mfma=None):
    """sections: [(first row, rows)] of one sequence, each its own launch with everything before it
    cached in pages that lie in odd order."""
    L, H = q.shape[:2]
    G, vdim = v.shape[1:]
    order = [4, 0, 9, 2, 7, 1, 8, 3, 6, 5, 10, 11, 12, 13, 14][: (L + BS - 1) // BS]
    blocks = max(order) + 2
    kc = torch.full((blocks, G, BS, k.shape[2]), 7.0, dtype=dtype)
    vc = torch.full((blocks, G, BS, vdim), 7.0, dtype=dtype)
    for j in range(L):
        kc[order[j // BS], :, j % BS] = k[j].to(dtype)
        vc[order[j // BS], :, j % BS] = v[j].to(dtype)
    kc, vc = kc.to(device), vc.to(device)
    bt = i32([order + [blocks - 1] * 3], device)
    out = torch.zeros(L, H * vdim, dtype=dtype, device=device)
    zero = torch.zeros(H, device=device)
    gd = gate.to(dtype).to(device)
    for lo, n in sections:
        nblk = (n + ops.KEEP_QBLK - 1) // ops.KEEP_QBLK
        ops.attn_keep_window(q[lo:lo + n].float().contiguous().to(device), kc, vc, vdim, bt, i32([0], device),
                             i32([n], device), i32([lo + n], device), i32([0] * nblk, device),
                             i32(list(range(nblk)), device), zero, gd[lo:lo + n], out[lo:lo + n], scale,
                             short_rows=32 if (short and n <= 32) else 0, mfma=mfma)
    return out


SECTIONS = [(0, 70), (70, 3), (73, 40)] + [(113 + i, 1) for i in range(17)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 16, 8), (3, 3, 40, 24), (2, 1, 8, 72), (6, 3, 64, 32), (2, 2, 6, 1)])
def test_attention_with_added_one_and_gate_per_output(device, H, G, dim, vdim):
    g = torch.Generator().manual_seed(4)
    L, scale = 130, 0.4
    q, k = torch.randn(L, H, dim, generator=g), torch.randn(L, G, dim, generator=g)
    v, gate = torch.randn(L, G, vdim, generator=g), torch.randn(L, H * vdim, generator=g)
    want = _dense(q, k, v, scale, gate)
    for short in (False, True):
        close(_attend(device, q, k, v, gate, SECTIONS, scale, short=short), want, 5e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 32, 32), (6, 3, 64, 32), (3, 1, 64, 64), (4, 1, 128, 128),
                                          (16, 1, 32, 32), (2, 2, 96, 64)])
def test_attention_on_mfma_tiles(H, G, dim, vdim):
    """bf16 pages: prompt rows (and decoded rows of wide groups) on the tiles, a gate per output
    with strided rows."""
    g = torch.Generator().manual_seed(5)
    L, scale = 130, dim ** -0.5
    q, k = torch.randn(L, H, dim, generator=g), torch.randn(L, G, dim, generator=g).bfloat16().float()
    v, gate = torch.randn(L, G, vdim, generator=g).bfloat16().float(), torch.randn(L, H * vdim + 8, generator=g)
    gate = gate.bfloat16().float()[:, :H * vdim]
    want = _dense(q, k, v, scale, gate)
    assert ops.keep_mfma_ok(dim, vdim)
    close(_attend("cuda", q, k, v, gate, SECTIONS, scale, torch.bfloat16, mfma=True), want, 8e-3)
    close(_attend("cuda", q, k, v, gate, SECTIONS, scale, torch.bfloat16, mfma=False), want, 8e-3)


@pytest.mark.parametrize("device", DEVICES)
def test_far_key_among_hundreds_and_the_added_one(device):
    """A key 440 tokens back takes a row's weight over; where every score is strongly negative the
    added one leaves almost nothing; a single token's output is halved at score 0."""
    g = torch.Generator().manual_seed(6)
    L, H, G, dim, vdim = 450, 2, 1, 8, 16
    q, k = torch.randn(L, H, dim, generator=g) * 0.1, torch.randn(L, G, dim, generator=g) * 0.1
    v = torch.randn(L, G, vdim, generator=g)
    q[:, :, 0], k[:, :, 0] = 0.0, 0.0
    q[L - 1, 1, 0], k[9, 0, 0] = 4.0, 4.0
    v[9] = 50.0
    q[L - 1, 0, 1], k[:, 0, 1] = 5.0, -5.0
    gate = torch.full((L, H * vdim), 20.0)
    want = _dense(q, k, v, 1.0, gate)
    assert float((want[L - 1, vdim:] - 50.0).abs().max()) < 1.0 and float(want[L - 1, :vdim].abs().max()) < 1e-6
    for sections in ([(0, L)], [(0, L - 1), (L - 1, 1)], [(0, L - 5), (L - 5, 5)]):
        close(_attend(device, q, k, v, gate, sections, 1.0), want, 5e-5)
    one = _attend(device, torch.zeros(1, H, dim), k[:1], v[:1], gate[:1], [(0, 1)], 1.0)
    close(one, v[:1].repeat(1, H, 1).reshape(1, -1) / 2, 1e-5)


# ------------------------------------------------------------------ matrix memory
def run_rows(cuts, slot, gen=0):
    """row_state / row_back / row_fwd / positions of a sequence's portions, one launch each."""
    at = 0
    for n in cuts:
        yield at, n, ([slot * 2 + (gen & 1)] * n, list(range(n)), list(range(n - 1, -1, -1)),
                      list(range(at, at + n)))
        at += n
        gen += 1


def _memory_inputs(g, T, H, dim, vdim, zi=(0.0, 2.0), zf=(2.0, 2.0)):
    """A projection's columns (q | k | v | gate, other columns around them) and gate logits."""
    wide = torch.randn(T, 2 * H * dim + 2 * H * vdim + 8, generator=g)
    z = torch.cat([torch.randn(T, H, generator=g) * zi[1] + zi[0], torch.randn(T, H, generator=g) * zf[1] + zf[0]], 1)
    return wide, z, torch.randn(2 * H, generator=g), torch.rand(H * vdim, generator=g) + 0.5


def _memory_want(wide, z, zb, nw, H, dim, vdim, cap, eps):
    T = wide.shape[0]
    a, b, c = H * dim, 2 * H * dim, 2 * H * dim + H * vdim
    x = wide.double()
    q, k = x[:, :a].view(T, H, dim) * dim ** -0.5, x[:, a:b].view(T, H, dim)
    v = x[:, b:c].view(T, H, vdim)
    zz = z.double() + zb.double()
    li, lf = oracle.memory_gates(zz[:, :H], zz[:, H:], cap)
    res = [oracle.matrix_memory(q[:, h], k[:, h], v[:, h], li[:, h], lf[:, h]) for h in range(H)]
    o = torch.stack([r[0] for r in res], 1)
    y = oracle.rms_unit(o, eps).reshape(T, -1) * nw.double()
    return y * oracle.sigmoid(x[:, c:c + H * vdim]), [r[1] for r in res]


def _memory_run(device, wide, z, zb, nw, H, dim, vdim, cap, eps, portions, slots=3, dtype=torch.float32,
                chunked=None, stale=50.0):
    """portions: iterable of (rows lo .. lo + n, state arrays, run starts).  The pools start out
    with another sequence's rest."""
    g = torch.Generator().manual_seed(99)
    a, b, c = H * dim, 2 * H * dim, 2 * H * dim + H * vdim
    S = (torch.randn(2 * slots, H, dim, vdim, generator=g) * stale).to(device)
    n = (torch.randn(2 * slots, H, dim, generator=g) * stale).to(device)
    m = (torch.randn(2 * slots, H, generator=g) * stale).to(device)
    wd, zd = wide.to(dtype).to(device), z.to(device)
    outs = []
    for lo, rows, st in portions:
        out = torch.empty(rows, H * vdim, dtype=dtype, device=device)
        w, zz = wd[lo:lo + rows], zd[lo:lo + rows]
        runs = i32([i for i, x in enumerate(st[1]) if x == 0] + [-1], device) if device != "cpu" else None
        ops.mlstm_recurrence(w[:, :a], w[:, a:b], w[:, b:c], zz, zb.to(device), cap, dim ** -0.5,
                             w[:, c:c + H * vdim], nw.to(device), eps, S, n, m,
                             *(i32(x, device) for x in st), out, runs, chunked)
        outs.append(out.cpu())
    return torch.cat(outs), (S.cpu(), n.cpu(), m.cpu())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,dim,vdim", [(2, 16, 24), (3, 10, 7), (1, 1, 1), (2, 64, 48), (1, 130, 66), (2, 32, 260)])
@pytest.mark.parametrize("cuts", [[45], [1] * 45, [2, 1, 3, 39], [7, 2, 2, 33, 1]])
def test_matrix_memory_in_portions(device, H, dim, vdim, cuts):
    """Whole, token by token and in portions through a slot with stale contents: zero state and a
    zero maximum at position 0, whatever the slot holds; the final state is the oracle's."""
    g = torch.Generator().manual_seed(7)
    T, cap, eps = sum(cuts), 6.0, 1e-5
    wide, z, zb, nw = _memory_inputs(g, T, H, dim, vdim)
    want, states = _memory_want(wide, z, zb, nw, H, dim, vdim, cap, eps)
    got, (S, n, m) = _memory_run(device, wide, z, zb, nw, H, dim, vdim, cap, eps, run_rows(cuts, 2))
    close(got, want, 2e-4)
    at = 2 + 3 * (len(cuts) & 1)
    for h in range(H):
        close(S[at, h], states[h][0], 1e-4)
        close(n[at, h], states[h][1], 1e-4)
        close(m[at, h], torch.tensor(states[h][2]), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("zi,zf,what", [(-20.0, 20.0, "never forgets, the floor of the denominator"),
                                        (20.0, -20.0, "forgets at once"), (20.0, 20.0, "keeps everything"),
                                        (-20.0, -20.0, "the maximum sinks below zero")])
def test_matrix_memory_extremes(device, zi, zf, what):
    """Gate logits beyond the cap on either side: the cap, the running maximum that starts at 0
    and the exp(-m) floor decide the output."""
    g = torch.Generator().manual_seed(8)
    H, dim, vdim, T, cap = 2, 16, 16, 140, 5.0
    wide, z, zb, nw = _memory_inputs(g, T, H, dim, vdim, (zi, 3.0), (zf, 3.0))
    # an eps that does not vanish beside small read-outs: their size shows in the output
    want, _ = _memory_want(wide, z, zb, nw, H, dim, vdim, cap, 1e-2)
    for cuts in ([T], [100] + [1] * 40):
        got, _ = _memory_run(device, wide, z, zb, nw, H, dim, vdim, cap, 1e-2, run_rows(cuts, 0))
        close(got, want, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_matrix_memory_remembers_a_far_token(device):
    """Almost no forgetting: a token 300 positions back whose input gate is wide open owns the
    read-out of a query that matches its key, in a prompt and decoded."""
    g = torch.Generator().manual_seed(9)
    H, dim, vdim, T, cap = 1, 8, 8, 310, 15.0
    wide, z, zb, nw = _memory_inputs(g, T, H, dim, vdim, (-2.0, 0.1), (12.0, 0.1))
    zb.zero_()
    z[7, 0] = 8.0
    wide[7, dim:2 * dim] = 0.0
    wide[7, dim] = 3.0
    wide[T - 1, :dim] = 0.0
    wide[T - 1, 0] = 3.0
    want, _ = _memory_want(wide, z, zb, nw, H, dim, vdim, cap, 1e-5)
    v = wide[7, 2 * dim:2 * dim + vdim].double()
    lone = oracle.rms_unit(v, 0.0) * nw.double() * oracle.sigmoid(wide[T - 1, 2 * dim + vdim:2 * dim + 2 * vdim].double())
    assert float((want[T - 1] - lone).abs().max()) < 0.1
    for cuts in ([T], [T - 1, 1], [5, 200, 104, 1]):
        got, _ = _memory_run(device, wide, z, zb, nw, H, dim, vdim, cap, 1e-5, run_rows(cuts, 1))
        close(got, want, 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_matrix_memory_two_runs_in_one_launch(device):
    g = torch.Generator().manual_seed(10)
    H, dim, vdim, cap, eps = 2, 12, 20, 8.0, 1e-5
    a, za, zb, nw = _memory_inputs(g, 33, H, dim, vdim)
    b, zz, _, _ = _memory_inputs(g, 5, H, dim, vdim)
    st = [[2] * 33 + [0] * 5, list(range(33)) + list(range(5)), list(range(32, -1, -1)) + list(range(4, -1, -1)),
          list(range(33)) + list(range(5))]
    got, _ = _memory_run(device, torch.cat([a, b]), torch.cat([za, zz]), zb, nw, H, dim, vdim, cap, eps,
                         [(0, 38, st)])
    close(got[:33], _memory_want(a, za, zb, nw, H, dim, vdim, cap, eps)[0], 2e-4)
    close(got[33:], _memory_want(b, zz, zb, nw, H, dim, vdim, cap, eps)[0], 2e-4)


@pytest.mark.gpu
@pytest.mark.parametrize("H,dim,vdim", [(3, 32, 80), (1, 64, 128), (2, 96, 16), (1, 128, 80), (1, 256, 64)])
@pytest.mark.parametrize("zi,zf", [((0.0, 2.0), (2.0, 2.0)), ((8.0, 6.0), (-20.0, 10.0)), ((-6.0, 1.0), (9.0, 1.0))])
def test_matrix_memory_chunks_on_mfma_tiles(H, dim, vdim, zi, zf):
    """Chunked bf16 form: portions that end inside, at and just past a chunk, then decoded rows,
    against the oracle on the same bf16 operands; strong and almost no forgetting."""
    g = torch.Generator().manual_seed(11)
    T, cap, eps = 210, 9.0, 1e-5
    wide, z, zb, nw = _memory_inputs(g, T, H, dim, vdim, zi, zf)
    wide = wide.bfloat16().float()
    want, states = _memory_want(wide, z, zb, nw, H, dim, vdim, cap, eps)
    for cuts in ([T], [64, 65, 2, 63, 16], [1, 128, 81], [130, 1, 1, 1, 77]):
        got, (S, n, m) = _memory_run("cuda", wide, z, zb, nw, H, dim, vdim, cap, eps, run_rows(cuts, 2),
                                     dtype=torch.bfloat16, chunked=True)
        e = (got.double() - want).abs()
        assert float(e.max()) <= 8e-3 * float(want.abs().max()) + 0.0, (cuts, float(e.max()))
        at = 2 + 3 * (len(cuts) & 1)
        for h in range(H):
            close(S[at, h], states[h][0], 2e-4)
            close(n[at, h], states[h][1], 2e-4)
            close(m[at, h], torch.tensor(states[h][2]), 1e-4)


@pytest.mark.gpu
def test_matrix_memory_chunked_runs_of_unequal_length_in_one_launch():
    g = torch.Generator().manual_seed(12)
    H, dim, vdim, cap, eps = 2, 32, 32, 9.0, 1e-5
    lens = [150, 1, 64, 3]
    parts = [_memory_inputs(g, n, H, dim, vdim) for n in lens]
    zb, nw = parts[0][2], parts[0][3]
    wide = torch.cat([p[0] for p in parts]).bfloat16().float()
    z = torch.cat([p[1] for p in parts])
    st = [[], [], [], []]
    for s, n in enumerate(lens):
        st[0] += [2 * s] * n
        st[1] += list(range(n))
        st[2] += list(range(n - 1, -1, -1))
        st[3] += list(range(n))
    got, _ = _memory_run("cuda", wide, z, zb, nw, H, dim, vdim, cap, eps, [(0, sum(lens), st)], slots=4,
                         dtype=torch.bfloat16, chunked=True)
    at = 0
    for n in lens:
        want, _ = _memory_want(wide[at:at + n], z[at:at + n], zb, nw, H, dim, vdim, cap, eps)
        close(got[at:at + n], want, 8e-3)
        at += n


# ------------------------------------------------------------------ routing and experts
def _route(device, z, corr, real, top, groups, keep, scale):
    T = z.shape[0]
    ids = torch.empty(T, top, dtype=torch.int32, device=device)
    wts = torch.empty(T, top, device=device)
    ident = torch.empty(T, device=device)
    ops.moe_route_softmax(z.to(device), corr.to(device), real, top, groups, keep, scale, ids, wts, ident)
    return ids.cpu(), wts.cpu(), ident.cpu()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("real,same,top,groups,keep", [(9, 3, 5, 4, 2), (6, 0, 2, 3, 1), (5, 3, 8, 0, 0), (1, 1, 1, 2, 1),
                                                       (90, 6, 5, 12, 4), (3, 9, 3, 4, 2), (7, 1, 8, 1, 1)])
def test_routing(device, real, same, top, groups, keep):
    """Corrections move the choice but not the weights, all choice scores may be negative, groups
    rank by their best choice score, identity experts count in softmax, groups and top."""
    g = torch.Generator().manual_seed(13)
    T, n, scale = 70, real + same, 1.7
    z = torch.randn(T, n + 1, generator=g) * 2                    # a further column that is no logit
    for mean in (0.0, -3.0):
        corr = torch.randn(n, generator=g) * 0.3 + mean
        r = {"top": top, "scale": scale}
        if groups:
            r["groups"] = {"count": groups, "keep": keep}
        want_ids, want_w = oracle.route(z[:, :n].double(), corr.double(), r)
        ids, wts, ident = _route(device, z, corr, real, top, groups, keep, scale)
        is_same = want_ids >= real
        assert torch.equal(ids.long(), torch.where(is_same, torch.full_like(want_ids, real), want_ids))
        close(wts, torch.where(is_same, torch.zeros_like(want_w), want_w), 1e-5)
        close(ident, (want_w * is_same).sum(-1), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_routing_ties_go_to_the_lower_index(device):
    ids, wts, ident = _route(device, torch.zeros(2, 8), torch.full((8,), -1.0), 6, 3, 4, 2, 2.0)
    assert ids.tolist() == [[0, 1, 2]] * 2
    close(wts, torch.full((2, 3), 0.25))
    close(ident, torch.zeros(2))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("d,ff", [(24, 10), (96, 64)])
def test_experts_skip_identity_pairs(device, d, ff):
    g = torch.Generator().manual_seed(14)
    T, E, same, top = 19, 4, 2, 3
    h = torch.randn(T, d, generator=g)
    w = {"router": torch.randn(E + same, d, generator=g), "correction": torch.randn(E + same, generator=g) * 0.2}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"] = (torch.randn(ff, d, generator=g) * d ** -0.5 for _ in range(2))
        w[f"e{e}.down"] = torch.randn(d, ff, generator=g) * ff ** -0.5
    w64 = {k: v.double() for k, v in w.items()}
    f = {"router": {"experts": E, "identity": same, "top": top, "scale": 1.2}}
    want = oracle.mixture(f, w64, "", h.double())
    z = h @ w["router"].T
    ids, wts, ident = _route(device, z, w["correction"], E, top, 0, 0, 1.2)
    assert int((ids == E).sum()) > 0
    w13 = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(E)]).to(device)
    w2 = torch.stack([w[f"e{e}.down"] for e in range(E)]).to(device)
    y = torch.empty(T, d, device=device)
    ops.moe_experts(h.to(device), ids.to(device), wts.to(device), w13, w2, None, y)
    close(y.cpu().double() + ident.double()[:, None] * h.double(), want, 5e-5)
