"""The HIP kernels behind the Dusupel decoder, one mechanism at a time, against plain fp64 torch statements of the same op (the oracle's
functions where one exists): the layer-norm pair (embedding, tail, gathered rows), the low-rank product with decays and gates as
epilogue, the output norm's gates / repeated weights / row strides, the delta rule's inputs and its scan over state slots in portions
(decay per head and per key channel, shared q / k heads, head sizes around the padding), and the convolved rotary store + windowed
attention that keeps the first tokens (scalar fp32 / bf16 and MFMA forms; prompt portions beside decoded rows; scattered pages)."""
import math

import pytest
import torch

from oracle import dusupel as F

pytestmark = pytest.mark.gpu
DEV = "cuda"
F64 = torch.float64


def H():
    from ssd_amd.hip import ops
    return ops


def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def elem(f32):
    return torch.float32 if f32 else torch.bfloat16


def tol(f32):
    return dict(rtol=2e-5, atol=2e-5) if f32 else dict(rtol=2e-2, atol=2e-2)


d = lambda t: t.to(DEV).contiguous()


@pytest.mark.parametrize("f32", [True, False])
# one row per workgroup of 256 or 1024 threads; the last case is too wide for the registers that keep a row
@pytest.mark.parametrize("W,T", [(40, 9), (328, 70), (2304, 5), (4352, 70)])
def test_layer_norm_pair_embedding_tail_and_gathered_rows(f32, W, T):
    V, eps, el = 23, 1e-5, elem(f32)
    table = (rnd(V, W, seed=1) + 0.5).to(el)
    ids = torch.randint(0, V, (T,), generator=torch.Generator().manual_seed(2))
    w = [(1 + 0.3 * rnd(W, seed=10 + i)).to(el) for i in range(3)]
    b = [(0.5 * rnd(W, seed=20 + i)).to(el) for i in range(3)]
    x = torch.full((T, W), float("nan"), device=DEV)
    o1, o2 = torch.zeros(T, W, dtype=el, device=DEV), torch.zeros(T, W, dtype=el, device=DEV)
    H().lnorm_embed(d(ids), d(table), x, eps, T, W, f32, norm1=(d(w[0]), d(b[0]), o1), norm2=(d(w[1]), d(b[1]), o2))
    ref = table.double()[ids]
    assert torch.equal(x.cpu().double(), ref)
    for o, i in ((o1, 0), (o2, 1)):
        assert torch.allclose(o.cpu().double(), F.layer_norm(ref, w[i], b[i], eps), **tol(f32))
    y = rnd(T, W, seed=3, scale=2.0) + 40.0            # a mean far from zero: the variance needs the squared DEVIATIONS
    H().lnorm_tail(x, d(y), 0.37, eps, T, W, f32, norm1=(d(w[2]), d(b[2]), o1))
    ref = ref + 0.37 * y.double()
    assert torch.allclose(x.cpu().double(), ref, rtol=1e-6, atol=1e-6)
    near = dict(rtol=2e-5, atol=1e-4) if f32 else tol(False)
    assert torch.allclose(o1.cpu().double(), F.layer_norm(ref, w[2], b[2], eps), **near)
    H().lnorm_tail(x, d(y), -0.37, eps, T, W, f32)      # the last layer: no norm follows
    ref = ref - 0.37 * y.double()
    assert torch.allclose(x.cpu().double(), ref, rtol=1e-4, atol=1e-5)
    pick = torch.tensor([T - 1, 0, 2], dtype=torch.int32)
    out = torch.zeros(3, W, dtype=el, device=DEV)
    before = x.clone()
    H().lnorm_rows(x, d(w[1]), d(b[1]), out, eps, 3, W, f32, gather=d(pick))
    assert torch.allclose(out.cpu().double(), F.layer_norm(x.cpu().double()[pick.long()], w[1], b[1], eps), **tol(f32)) and torch.equal(x, before)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("M,N,K,nd", [(1, 100, 16, 64), (5, 37, 24, 0), (70, 132, 40, 132), (33, 68, 13, 31)])
def test_low_rank_product_with_decays_and_gates(f32, M, N, K, nd):
    el = elem(f32)
    x, w = rnd(M, K, seed=1).to(el), rnd(N, K, seed=2).to(el)
    rate, bias = rnd(max(nd, 1), seed=3).exp(), rnd(max(nd, 1), seed=4, scale=3.0)
    y = torch.zeros(M, N, device=DEV)
    H().gemm_rows_decay_gate(d(x), d(w), y, M, N, K, d(rate), d(bias), nd, f32)
    z = x.double() @ w.double().T
    ref = torch.sigmoid(z)
    if nd:
        ref[:, :nd] = torch.exp(-rate.double()[:nd] * F.softplus(z[:, :nd] + bias.double()[:nd]))
    assert torch.allclose(y.cpu().double(), ref, rtol=1e-4, atol=1e-5)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("act", [0, 1, 2])
def test_output_norm_gates_repeated_weights_and_row_stride(f32, act):
    T, groups, per, ldo, ldg = 6, 5, 20, 120, 130
    N, el = groups * per, elem(f32)
    o, gate, w = rnd(T, N, seed=1), rnd(T, ldg, seed=2), (1 + 0.3 * rnd(per, seed=3)).to(el)
    out = torch.full((T, ldo), 7.0, dtype=el, device=DEV)
    H().group_gate_norm(d(o), d(gate), ldg, d(w), 1e-5, out, T, N, groups, False, f32, gate_act=act, w_period=per, out_scale=1.3, ldo=ldo)
    g = {0: F.silu, 1: torch.sigmoid, 2: lambda t: t}[act](gate[:, :N].double())
    ref = (F.rms(o.double().view(T, groups, per), 1e-5) * w.double()).reshape(T, N) * g * 1.3
    assert torch.allclose(out[:, :N].cpu().double(), ref, **tol(f32)) and bool((out[:, N:] == 7.0).all())


DELTA_CASES = [
    # H, G, D, Dv, taps, channel decay
    (2, 2, 8, 8, 3, True), (4, 2, 24, 20, 4, False), (3, 1, 32, 33, 2, True), (6, 3, 40, 16, 1, False), (2, 1, 64, 40, 4, True),
    (1, 1, 96, 64, 3, True), (4, 4, 128, 17, 4, False), (2, 1, 130, 8, 6, True), (1, 1, 300, 24, 4, True), (2, 2, 512, 4, 3, False),
]


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("case", DELTA_CASES)
def test_delta_rule_inputs_and_scan_in_portions_over_slots(f32, case):
    """Two sequences in slots 2 and 0 of a pool that holds NaN; the first arrives in portions of 1, 2, 18 and 23 rows (one of them beside
    the second one's rows, one longer than a staged batch); every row of the inputs and of the read-out equals the whole-sequence
    statement, the rows of the portions equal those of one whole portion bit by bit, and the saved convolution inputs are the last ones."""
    Hh, G, D, Dv, taps, ch = case
    el, R, c0, col_off = elem(f32), 11, 5, 3           # other channels share the convolution state, other columns the projection rows
    DP = 32 if D <= 32 else -(-D // 64) * 64
    n_ch = 2 * G * D + Hh * Dv
    C, NP = c0 + n_ch + 2, col_off + n_ch + 2 * Hh + R + 1
    b_off, a_off, lr_off = col_off + n_ch, col_off + n_ch + Hh, col_off + n_ch + 2 * Hh
    cw = rnd(n_ch, taps, seed=1).to(el)
    rate, bias = rnd(Hh, seed=2, scale=0.5).exp(), rnd(Hh, seed=3) - 2.0
    nA, nB = 44, 17
    pA, pB = rnd(nA, NP, seed=4), rnd(nB, NP, seed=5)
    dA, dB = ((-rnd(n, Hh * DP, seed=s).exp() * 0.2).exp() for n, s in ((nA, 6), (nB, 7)))

    def reference(proj, dec):
        n = proj.shape[0]
        u = F.silu(F.short_conv(proj[:, col_off:col_off + n_ch].double(), cw))
        q = F.unit(u[:, :G * D].view(n, G, D)) * D ** -0.5
        k = F.unit(u[:, G * D:2 * G * D].view(n, G, D))
        v = u[:, 2 * G * D:].view(n, Hh, Dv)
        beta = torch.sigmoid(proj[:, b_off:b_off + Hh].double())
        gh = torch.exp(-rate.double() * F.softplus(proj[:, a_off:a_off + Hh].double() + bias.double()))
        rep = lambda t: t.repeat_interleave(Hh // G, dim=1)
        decay = dec.double().view(n, Hh, DP)[:, :, :D] if ch else gh.unsqueeze(-1)
        return q, k, v, beta, gh, F.delta_rule(rep(q), rep(k), v, beta, decay)

    state = torch.full((3, Hh, Dv, DP), float("nan"), device=DEV)
    # the saved rows of channels that nobody convolves hold numbers, all else NaN
    conv = torch.full((3, max(taps - 1, 1), C), float("nan"), device=DEV)

    def run(parts, slots):
        """parts: [(proj rows, decay rows, first position)] -> (qk, v, scalars, low-rank rows, out)"""
        rows, dec = torch.cat([p[0] for p in parts]), torch.cat([p[1] for p in parts])
        T = rows.shape[0]
        cu = torch.tensor([0] + [p[0].shape[0] for p in parts]).cumsum(0).to(torch.int32)
        pos = torch.cat([torch.arange(p[2], p[2] + p[0].shape[0]) for p in parts])
        z = lambda *s, dt=torch.float32: torch.full(s, float("nan"), dtype=dt, device=DEV)
        qk, v, sc, lr, o = z(T, G, 2, DP), z(T, Hh, Dv), z(T, Hh, 4), z(T, 16, dt=el), z(T, Hh, Dv)
        proj, sl, cud, posd = d(rows), d(torch.tensor(slots, dtype=torch.int32)), d(cu), d(pos)
        H().delta_prep(proj, NP, col_off, d(cw), taps, conv, C, c0, sl, posd, len(parts), b_off, qk, v, sc, T, Hh, G, D, Dv, DP, f32,
                       a_off=-1 if ch else a_off, rate=d(rate), bias=d(bias), lr_off=lr_off, lr_n=R, lr_out=lr, ld_lr=16, cu_q=cud)
        # the state covers channels c0 .. of C: save through a projection whose columns start c0 earlier
        wide = d(torch.cat([torch.zeros(T, C), rows], dim=1))
        H().delta_scan(qk, v, sc, posd, sl, state, o, len(parts), Hh, G, D, Dv, DP, wide, C + NP, C + col_off - c0, n_ch + c0 + 2, conv, taps,
                       decay=d(dec) if ch else None, ldd=Hh * DP, cu_q=cud)
        return [t.cpu() for t in (qk, v, sc, lr, o)]

    outs, at = [], 0
    for i, n in enumerate((1, 2, 18, 23)):
        parts, slots = [(pA[at:at + n], dA[at:at + n], at)], [2]
        if i == 1:
            parts.append((pB, dB, 0))
            slots.append(0)
        r = run(parts, slots)
        outs.append([t[:n] for t in r])
        if i == 1:
            rest = [t[n:] for t in r]
        at += n
    assert at == nA
    for got, proj, dec in ((([torch.cat(t) for t in zip(*outs)]), pA, dA), (rest, pB, dB)):
        q, k, v, beta, gh, o = reference(proj, dec)
        near = dict(rtol=1e-4, atol=2e-5)
        assert torch.allclose(got[0][:, :, 0, :D].double(), q, **near) and torch.allclose(got[0][:, :, 1, :D].double(), k, **near)
        assert float(got[0][..., D:].abs().max() if D < DP else 0.0) == 0.0
        assert torch.allclose(got[1].double(), v, **near)
        assert torch.allclose(got[2][..., 0].double(), beta, **near)
        assert torch.allclose(got[2][..., 1].double(), torch.ones_like(gh) if ch else gh, **near)
        assert torch.allclose(got[2][..., 2].double(), (q * k).sum(-1).repeat_interleave(Hh // G, dim=1), **near)
        assert torch.allclose(got[3][:, :R].double(), proj[:, lr_off:lr_off + R].to(el).double()) and float(got[3][:, R:].float().abs().max()) == 0
        err = (got[4].double() - o).abs().max() / o.abs().max()
        assert float(err) < 2e-5, float(err)
    if taps > 1:
        assert torch.equal(conv[2, :, c0:c0 + n_ch].cpu(), pA[nA - taps + 1:, col_off:col_off + n_ch])
        assert torch.equal(conv[0, :, c0:c0 + n_ch].cpu(), pB[nB - taps + 1:, col_off:col_off + n_ch])
    assert bool(torch.isnan(state[1]).all())
    kept = state[2].clone()
    whole = run([(pA, dA, 0)], [2])
    assert torch.equal(whole[4], torch.cat([t[4] for t in outs])) and torch.equal(state[2], kept)


ATT_CASES = [
    # f32, H, G, D, Dv, window, keep, rot, taps, bs, mfma
    (True, 4, 2, 24, 20, 16, 3, 8, 3, 16, False), (True, 3, 1, 8, 6, 33, 0, 8, 4, 8, False), (True, 2, 2, 16, 8, 1, 1, 0, 2, 16, False),
    (True, 2, 1, 12, 12, 0, 5, 6, 1, 16, False), (True, 2, 2, 10, 9, 40, 70, 10, 6, 16, False), (False, 4, 2, 24, 20, 16, 3, 8, 3, 16, False),
    (False, 8, 2, 32, 64, 40, 20, 16, 3, 32, True), (False, 5, 1, 96, 80, 70, 33, 48, 4, 64, True), (False, 4, 4, 64, 32, 17, 64, 64, 4, 32, True),
    (False, 20, 1, 128, 48, 100, 7, 32, 2, 64, True), (False, 4, 2, 160, 160, 33, 12, 40, 3, 32, True), (False, 4, 2, 32, 32, 0, 9, 32, 3, 32, True),
]


@pytest.mark.parametrize("case", ATT_CASES)
def test_convolved_rotary_store_and_window_that_keeps_first_tokens(case):
    """Three sequences in one varlen batch -- a prompt portion that continues an earlier one, a whole short prompt, one decoded row --
    over pages handed out in scattered order that hold NaN; sharp scores, so one key more or fewer shows."""
    f32, Hh, G, D, Dv, window, keep, rot, taps, bs, mfma = case
    el, scale, base, oscale = elem(f32), 2.0 / math.sqrt(D), 1000.0, 0.8
    nq, nk, nv, no = Hh * D, G * D, G * Dv, Hh * Dv
    C = nq + nk + nv
    col_off, ldo = 2, -(-(no + 3) // 4) * 4
    NP = col_off + C + no
    cw = (rnd(C, taps, seed=1, scale=0.4) + torch.nn.functional.one_hot(torch.tensor(taps - 1), taps)).to(el)
    freqs = torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)] or [0.0], dtype=F64).float()
    lens, new = [150, 37, 121], [53, 37, 1]                 # context length after this step, rows this step brings
    nb = sum(-(-n // bs) for n in lens) + 3
    max_blocks = max(-(-n // bs) for n in lens)
    kc = torch.full((nb, G, bs, D), float("nan"), dtype=el, device=DEV)
    vc = torch.full((nb, G, Dv, bs), float("nan"), dtype=el, device=DEV)
    conv = torch.full((4, max(taps - 1, 1), C), float("nan"), device=DEV)
    pages = torch.randperm(nb, generator=torch.Generator().manual_seed(2)).tolist()
    bt = torch.zeros(len(lens), max_blocks, dtype=torch.int32)
    state_slots = torch.tensor([3, 0, 1], dtype=torch.int32)

    def store(rows, slots, pos, cu, sl):
        T = rows.shape[0]
        q = torch.zeros(T, nq, dtype=el, device=DEV)
        H().winattn_store_conv_rope(d(rows), NP, col_off, d(cw), taps, conv, C, d(sl), d(pos), len(cu) - 1, d(freqs), rot, d(slots), q, kc,
                                    vc, T, Hh, G, D, Dv, bs, f32, cu_q=d(torch.tensor(cu, dtype=torch.int32)))
        return q

    projs, refs, far, rows, pos, slots, cu = [], [], [], [], [], [], [0]
    for b, (n, k) in enumerate(zip(lens, new)):
        proj = rnd(n, NP, seed=10 + b)
        mine = [pages.pop() for _ in range(-(-n // bs))]
        bt[b, :len(mine)] = torch.tensor(mine, dtype=torch.int32)
        sl = torch.tensor([mine[p // bs] * bs + p % bs for p in range(n)], dtype=torch.int32)
        if n > k:        # the earlier portion: stored by a call of its own, then its last inputs saved as a scan does
            store(proj[:n - k], sl[:n - k], torch.arange(n - k), [0, n - k], state_slots[b:b + 1])
            if taps > 1:
                conv[int(state_slots[b])] = d(proj[n - k - taps + 1:n - k, col_off:col_off + C])
        u = F.short_conv(proj[:, col_off:col_off + C].double(), cw)
        qr = F.turn(u[:, :nq].view(n, Hh, D), torch.arange(n), rot, base)
        kr = F.turn(u[:, nq:nq + nk].view(n, G, D), torch.arange(n), rot, base)
        vr = u[:, nq + nk:].view(n, G, Dv)
        for store_to, win in ((refs, window), (far, window + 1)):
            see = F.visible(n, {"size": win, "keep_first": keep} if window else None)
            out = torch.zeros(n, Hh, Dv, dtype=F64)
            for h in range(Hh):
                s = (qr[:, h] @ kr[:, h // (Hh // G)].T) * scale
                out[:, h] = torch.softmax(torch.where(see, s, torch.full_like(s, -math.inf)), -1) @ vr[:, h // (Hh // G)]
            store_to.append((out.reshape(n, no) * torch.sigmoid(proj[:, col_off + C:].double()) * oscale)[n - k:])
        rows.append(proj[n - k:])
        pos.append(torch.arange(n - k, n))
        slots.append(sl[n - k:])
        cu.append(cu[-1] + k)
    T = cu[-1]
    rows, pos = torch.cat(rows), torch.cat(pos)
    q = store(rows, torch.cat(slots), pos, cu, state_slots)
    out = torch.full((T, ldo), 5.0, dtype=el, device=DEV)
    gate = d(rows).view(-1)[col_off + C:]
    H().winattn_paged(q, kc, vc, None, None, d(bt), max_blocks, d(pos), len(lens), T, Hh, G, D, Dv, bs, window, scale, 0.0, out, f32,
                      cu_q=d(torch.tensor(cu, dtype=torch.int32)), max_q=max(new) if mfma else 0, keep_first=keep, gate=gate, ldg=NP,
                      out_scale=oscale, ldo=ldo)
    ref, other = torch.cat(refs), torch.cat(far)
    got = out[:, :no].cpu().double()
    assert torch.isfinite(got).all() and bool((out[:, no:] == 5.0).all())
    if f32:
        assert torch.allclose(got, ref, rtol=1e-4, atol=2e-5), float((got - ref).abs().max())
    else:
        assert float((got - ref).abs().max()) < 0.06 * float(ref.abs().max()), float((got - ref).abs().max())
        assert float((got - ref).pow(2).mean().sqrt()) < 0.012 * float(ref.pow(2).mean().sqrt()) + 1e-3
    if window and keep < 37:        # the statement is sharp: one key more is far away
        assert float((other - ref).abs().max()) > (100 * float((got - ref).abs().max()) if f32 else 0.02)


def test_glu_rows_with_a_row_stride():
    T, Fd, ldo = 5, 24, 40
    ab = rnd(T, 2 * Fd, seed=1)
    out = torch.full((T, ldo), 3.0, device=DEV)
    H().glu_rows(d(ab), out, T, Fd, H().GLU_SILU, True, ldo=ldo)
    ref = F.silu(ab[:, :Fd].double()) * ab[:, Fd:].double()
    assert torch.allclose(out[:, :Fd].cpu().double(), ref, **tol(True)) and bool((out[:, Fd:] == 3.0).all())


def test_sizes_the_kernels_do_not_take_are_refused():
    from ssd_amd.hip.lib import SsdHipError
    z = lambda *s: torch.zeros(*s, device=DEV)
    i32, i64 = torch.zeros(1, dtype=torch.int32, device=DEV), torch.zeros(1, dtype=torch.int64, device=DEV)
    ok = dict(B=1, Hh=2, G=1, D=8, Dv=8, DP=32)

    def scan(B, Hh, G, D, Dv, DP):
        H().delta_scan(z(1, 4, 2, 1024), z(1, 4, 64), z(1, 4, 4), i64, i32, z(1, 4, 64, 1024), z(1, 4, 64), B, Hh, G, D, Dv, DP, z(1, 64), 64, 0,
                       32, z(1, 3, 32), 4, q_per_seq=1)

    scan(**ok)
    for bad in (dict(DP=64), dict(D=40), dict(G=3), dict(D=600, DP=640), dict(D=0)):
        with pytest.raises(SsdHipError):
            scan(**{**ok, **bad})
    with pytest.raises(SsdHipError):        # the epilogue's tables come through its own entry point only
        H().gemm_rows(z(1, 8), z(4, 8), z(1, 4), 1, 4, 8, True, 7)
