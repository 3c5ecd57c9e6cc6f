"""The HIP kernels behind the Tumudra decoder, one mechanism at a time, against plain fp64 torch statements of the same op (the oracle's
functions where one exists): scaled embedding rows, the output-norm tail (one row, or two normed sides), the norm without a bias, the biased
product, the output norm with a denominator per head, the outer-product memory over state slots in portions (exponential gates inside the
scan and ahead of it, fixed decays; head sizes around the padding), the per-head-norm rotary store and the attention over scattered pages
(scalar and MFMA forms; decode batches whose keys are cut over workgroups; more query heads than a tile has rows; queries alone)."""
import pytest
import torch

from oracle import tumudra as F

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
i32 = lambda x: torch.tensor(x, dtype=torch.int32)


@pytest.mark.parametrize("f32", [True, False])
# one row per workgroup of 256 or 1024 threads; the last two are too wide for the registers that keep a row
@pytest.mark.parametrize("W,T", [(40, 9), (328, 70), (2304, 5), (4352, 70), (16640, 2)])
def test_scaled_embedding_output_norm_tail_of_one_row_and_of_two_sides(f32, W, T):
    V, eps, el = 23, 1e-5, elem(f32)
    table = (rnd(V, W, seed=1) + 0.5).to(el)
    ids = torch.randint(0, V, (T,), generator=torch.Generator().manual_seed(2))
    x = torch.full((T, W), float("nan"), device=DEV)
    hn = torch.zeros(T, W, dtype=el, device=DEV)
    H().embed_hist(d(ids), d(table), x, T, W, f32, rows_out=hn, scale=7.3)
    ref = table.double()[ids] * 7.3
    assert torch.allclose(x.cpu().double(), ref, rtol=1e-6) and torch.allclose(hn.cpu().double(), ref, **tol(f32))
    w, w1, w2 = ((1 + 0.3 * rnd(W, seed=s)).to(el) for s in (10, 11, 12))
    y = rnd(T, W, seed=3, scale=2.0) + 40.0            # a mean far from zero: the variance needs the squared DEVIATIONS
    H().lnorm_post_tail(x, d(y), d(w), eps, T, W, f32, next_out=hn)
    ref = ref + F.layer_norm(y.double(), w, eps)
    near = dict(rtol=2e-5, atol=1e-4)
    assert torch.allclose(x.cpu().double(), ref, **near) and torch.allclose(hn.cpu().double(), ref, **(near if f32 else tol(False)))
    yl, yr = rnd(T, W, seed=4, scale=0.01), rnd(T, W, seed=5, scale=30.0) + 3.0         # sides of very unequal size
    pair = lambda s: s * (F.rms(yl.double(), eps) * w1.double() + F.rms(yr.double(), eps) * w2.double())
    H().lnorm_post_tail(x, d(yl), d(w), eps, T, W, f32, y2_rows=d(yr), w1=d(w1), w2=d(w2), pair_scale=0.5, next_out=hn)
    before, ref = ref, ref + F.layer_norm(pair(0.5), w, eps)
    assert torch.allclose(x.cpu().double(), ref, **near) and torch.allclose(hn.cpu().double(), ref, **(near if f32 else tol(False)))
    assert float((F.layer_norm(yl.double() + yr.double(), w, eps) - (ref - before)).abs().max()) > 0.1        # (the sides' own norms matter)
    H().lnorm_post_tail(x, d(yl), d(w), eps, T, W, f32, y2_rows=d(yr), w1=d(w1), w2=d(w2), pair_scale=1e-3)      # eps shows at this scale
    ref = ref + F.layer_norm(pair(1e-3), w, eps)
    assert torch.allclose(x.cpu().double(), ref, **near)
    pick = i32([T - 1, 0, T // 2])
    out = torch.zeros(3, W, dtype=el, device=DEV)
    H().lnorm_rows(x, d(w1), None, out, eps, 3, W, f32, gather=d(pick))
    assert torch.allclose(out.cpu().double(), F.layer_norm(x.cpu().double()[pick.long()], w1, eps), **tol(f32))


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("M,N,K", [(1, 100, 16), (5, 37, 24), (70, 132, 40), (33, 68, 13)])
def test_product_with_a_bias(f32, M, N, K):
    x, w, b = rnd(M, K, seed=1).to(elem(f32)), rnd(N, K, seed=2).to(elem(f32)), rnd(N, seed=3, scale=5.0)
    y = torch.zeros(M, N, device=DEV)
    H().gemm_rows_bias(d(x), d(w), y, M, N, K, d(b), f32)
    assert torch.allclose(y.cpu().double(), x.double() @ w.double().T + b.double(), rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("gate_first", [True, False])
def test_output_norm_with_a_denominator_per_head(f32, gate_first):
    T, groups, per = 6, 5, 20
    N, el = groups * per, elem(f32)
    o, gate, w, den = rnd(T, N, seed=1), rnd(T, N, seed=2), (1 + 0.3 * rnd(N, seed=3)).to(el), rnd(T, groups, seed=4).abs() * 50 + 0.2
    out = torch.zeros(T, N, dtype=el, device=DEV)
    H().group_gate_norm(d(o), d(gate), N, d(w), 1e-2, out, T, N, groups, gate_first, f32, gate_act=1, den=d(den))
    g = torch.sigmoid(gate.double()).view(T, groups, per)
    v = o.double().view(T, groups, per) / den.double().unsqueeze(-1)
    ref = (F.rms(v * g, 1e-2) if gate_first else F.rms(v, 1e-2) * g).reshape(T, N) * w.double()
    assert torch.allclose(out.cpu().double(), ref, **tol(f32))


MEMORY_CASES = [(2, 8, 8), (3, 24, 20), (1, 32, 33), (3, 33, 31), (2, 64, 64), (1, 96, 15), (2, 128, 16), (2, 130, 17), (1, 256, 40), (1, 300, 24), (1, 512, 5)]


@pytest.mark.parametrize("kind", ["gates", "decay"])
@pytest.mark.parametrize("Hh,D,Dv", MEMORY_CASES)
def test_outer_product_memory_in_portions_over_slots(Hh, D, Dv, kind):
    """Two sequences in slots 2 and 0 of a pool that holds NaN; the first arrives in portions of 1, 2, 37, 8 and 292 rows (one of them beside the
    second one's rows, one of several staged batches and gate chunks, two in the decoding form).  Read-out and denominator equal the whole-sequence statement; the rows
    of the portions equal those of one whole portion bit by bit; gates computed ahead of the scan equal those inside it bit by bit."""
    gates_on = kind == "gates"
    DP = 32 if D <= 32 else -(-D // 64) * 64
    q0, k0 = 3, 5 + Hh * D                     # column offsets with gaps between the parts
    v0 = k0 + Hh * D + 1
    i0, f0 = v0 + Hh * Dv, v0 + Hh * Dv + Hh + 2
    NP, cap, qs = f0 + Hh + 3, 5.0, D ** -0.5
    nA, nB = 340, 19
    pA, pB = rnd(nA, NP, seed=4), rnd(nB, NP, seed=5)
    bi, bf = rnd(Hh, seed=6), 2.0 + rnd(Hh, seed=7)
    decay = torch.tensor([1.0 - 2.0 ** -(1 + 3 * h) for h in range(Hh)])

    def reference(p):
        n, x = p.shape[0], p.double()
        q, k, v = x[:, q0:q0 + Hh * D].view(n, Hh, D) * qs, x[:, k0:k0 + Hh * D].view(n, Hh, D), x[:, v0:v0 + Hh * Dv].view(n, Hh, Dv)
        if not gates_on:
            return F.retention(q, k, v, decay.tolist())
        i = F.soft_cap(x[:, i0:i0 + Hh] + bi.double(), cap)
        f = F.log_sigmoid(F.soft_cap(x[:, f0:f0 + Hh] + bf.double(), cap))
        return F.matrix_memory(q, k, v, i, f)

    cols = Dv + gates_on
    state, running = torch.full((3, Hh, cols, DP), float("nan"), device=DEV), torch.full((3, Hh, Dv + 1), float("nan"), device=DEV)

    def run(parts, slots, ahead):
        """parts: [(rows, first position)] -> out / den (gates) or out"""
        p = torch.cat([x for x, _ in parts])
        pos = torch.cat([torch.arange(x.shape[0]) + at for x, at in parts])
        cu = i32([0] + torch.tensor([x.shape[0] for x, _ in parts]).cumsum(0).tolist())
        T = p.shape[0]
        out, den = (torch.full(s, float("nan"), device=DEV) for s in ((T, Hh * Dv), (T, Hh)))
        rows = dict(q_per_seq=T) if len(parts) == 1 and T <= 8 else dict(cu_q=d(cu))         # a fixed row count: the decoding form
        common = dict(i_off=i0, f_off=f0, bias_i=d(bi), bias_f=d(bf), cap=cap, m_state=running, **rows)
        g = None
        if gates_on and ahead:
            g = torch.full((T, Hh, 4), float("nan"), device=DEV)
            H().memory_gates(d(p), NP, positions=d(pos), state_slots=d(i32(slots)), gates=g, B=len(parts), H=Hh, Dv=Dv, **common)
        kw = dict(common, gates=g, den=den) if gates_on else dict(decay=d(decay), **rows)
        H().memory_scan(d(p), NP, q0, k0, v0, d(pos), d(i32(slots)), state, out, len(parts), Hh, D, Dv, DP, q_scale=qs, **kw)
        return (out.view(T, Hh, Dv) / den.unsqueeze(-1) if gates_on else out.view(T, Hh, Dv)).cpu()

    outs, rest, at = [], None, 0
    for j, n in enumerate((1, 2, 37, 8, 292)):
        parts, slots = [(pA[at:at + n], at)], [2]
        if j == 1:
            parts.append((pB, 0))
            slots.append(0)
        r = run(parts, slots, ahead=j % 2 == 1)
        outs.append(r[:n])
        if j == 1:
            rest = r[n:]
        at += n
    assert at == nA
    for got, p in ((torch.cat(outs), pA), (rest, pB)):
        ref = reference(p)
        err = (got.double() - ref).abs().max() / ref.abs().max()
        assert float(err) < 3e-5, float(err)
    assert bool(torch.isnan(state[1]).all())
    kept, kept_m = state[2].clone(), running[2].clone()
    for ahead in (False, True) if gates_on else (False,):
        assert torch.equal(run([(pA, 0)], [2], ahead), torch.cat(outs)) and torch.equal(state[2], kept)
        if gates_on:
            assert torch.equal(running[2, :, 0], kept_m[:, 0])


ATT_CASES = [
    # f32, H, G, D, Dv, window, rot, bs, mfma, workspace
    (True, 4, 2, 24, 20, 16, 8, 16, False, False), (True, 3, 1, 8, 6, 33, 8, 8, False, False), (True, 2, 2, 16, 8, 1, 0, 16, False, False),
    (True, 2, 1, 12, 12, 0, 6, 16, False, False), (True, 6, 3, 130, 9, 40, 128, 16, False, False), (False, 4, 2, 24, 20, 16, 8, 16, False, True),
    (False, 8, 2, 32, 64, 40, 16, 32, True, True), (False, 5, 1, 96, 80, 70, 48, 64, True, False), (False, 4, 4, 64, 32, 17, 64, 32, True, True),
    (False, 20, 1, 128, 48, 100, 32, 64, True, True), (False, 4, 2, 160, 160, 33, 40, 32, True, True), (False, 4, 2, 32, 32, 0, 32, 32, True, True),
]


def attention_reference(x, Hh, G, D, Dv, wq, wk, eps, rot, scale, window):
    n = x.shape[0]
    x, pos = x.double(), torch.arange(n)
    q, k, v = x[:, :Hh * D].view(n, Hh, D), x[:, Hh * D:(Hh + G) * D].view(n, G, D), x[:, (Hh + G) * D:].view(n, G, Dv)
    q, k = (F.turn(F.rms(t, eps) * w.double(), pos, rot, False) for t, w in ((q, wq), (k, wk)))
    return F.softmax_attention(q, k, v, scale, F.visible(n, window or None))


def store_and_attend(case, lens, new, seed=0, split=True, scale=None):
    """Sequences of lens tokens whose last `new` rows come as one varlen batch, the earlier ones stored before; scattered pages of a cache that
    holds NaN.  Returns (attention rows, reference, the same reference with a window one token longer, the arguments of a repeat)."""
    f32, Hh, G, D, Dv, window, dims, bs, mfma, ws = case
    el, eps, scale = elem(f32), 1e-5, D ** -0.5 if scale is None else scale
    NP = (Hh + G) * D + G * Dv
    max_blocks = max(-(-n // bs) for n in lens) + 1
    nb = sum(-(-n // bs) for n in lens) + 3
    kc, vc = torch.full((nb, G, bs, D), float("nan"), dtype=el, device=DEV), torch.full((nb, G, Dv, bs), float("nan"), dtype=el, device=DEV)
    pages = torch.randperm(nb, generator=torch.Generator().manual_seed(1)).tolist()
    bt = torch.zeros(len(lens), max_blocks, dtype=torch.int32)
    wq, wk = (1.5 + rnd(D, seed=3, scale=0.3)).to(el), (1.5 + rnd(D, seed=4, scale=0.3)).to(el)
    rot = {"base": 100.0, "dims": dims}
    qf = d((F.angular_frequencies(rot) if dims else torch.zeros(1)).float())
    refs, longer, rows, pos, slots, cu = [], [], [], [], [], [0]
    store = lambda x, p, sl, q: H().winattn_store_norm_rope(d(x), NP, d(wq), d(wk), eps, d(p), qf, dims, d(sl), q, kc, vc, x.shape[0], Hh, G, D, Dv, bs, f32)
    for b, (n, k) in enumerate(zip(lens, new)):
        proj = rnd(n, NP, seed=seed + 10 + b)
        mine = [pages.pop() for _ in range(-(-n // bs))]
        bt[b, :len(mine)] = i32(mine)
        sl = i32([mine[p // bs] * bs + p % bs for p in range(n)])
        if n > k:
            store(proj[:n - k], torch.arange(n - k), sl[:n - k], torch.zeros(n - k, Hh * D, dtype=el, device=DEV))
        refs.append(attention_reference(proj, Hh, G, D, Dv, wq, wk, eps, rot, scale, window)[n - k:])
        if window:
            longer.append(attention_reference(proj, Hh, G, D, Dv, wq, wk, eps, rot, scale, window + 1)[n - k:])
        rows.append(proj[n - k:])
        pos += list(range(n - k, n))
        slots.append(sl[n - k:])
        cu.append(cu[-1] + k)
    T, pos = cu[-1], torch.tensor(pos)
    q = torch.zeros(T, Hh * D, dtype=el, device=DEV)
    store(torch.cat(rows), pos, torch.cat(slots), q)
    q2 = torch.zeros_like(q)                          # queries alone: the same rows, and the pages stay as they are
    kc0, vc0 = kc.clone(), vc.clone()
    H().winattn_store_norm_rope(d(torch.cat(rows)), NP, d(wq), None, eps, d(pos), qf, dims, None, q2, None, None, T, Hh, 0, D, Dv, bs, f32)
    same = lambda a, b: torch.equal(torch.nan_to_num(a.float(), nan=7e7), torch.nan_to_num(b.float(), nan=7e7))
    assert torch.equal(q, q2) and same(kc, kc0) and same(vc, vc0)
    ldo = Hh * Dv + 12
    out = torch.full((T, ldo), 5.0, dtype=el, device=DEV)
    work = torch.full((1024 * 16 * (Dv + 2),), float("nan"), device=DEV) if ws and split else None
    H().winattn_paged(q, kc, vc, None, None, d(bt), max_blocks, d(pos), len(lens), T, Hh, G, D, Dv, bs, window, scale, 0.0, out, f32,
                      cu_q=d(i32(cu)), max_q=max(new) if mfma else 0, ldo=ldo, workspace=work)
    assert bool((out[:, Hh * Dv:] == 5.0).all())
    return out[:, :Hh * Dv].cpu().double(), torch.cat(refs), torch.cat(longer) if longer else None


def check(got, ref, longer, f32):
    assert torch.isfinite(got).all()
    if f32:
        assert torch.allclose(got, ref, rtol=1e-4, atol=2e-5), float((got - ref).abs().max())
    else:
        assert float((got - ref).abs().max()) < 0.06 * float(ref.abs().max()), float((got - ref).abs().max())
        assert float((got - ref).pow(2).mean().sqrt()) < 0.012 * float(ref.pow(2).mean().sqrt()) + 1e-3
    if longer is not None:        # the statement is sharp: one key more is far away
        assert float((longer - ref).abs().max()) > (100 * float((got - ref).abs().max()) if f32 else 0.02)


@pytest.mark.parametrize("case", ATT_CASES)
def test_head_norm_rotary_store_and_attention_over_scattered_pages(case):
    """A prompt portion that continues an earlier one, a whole short prompt and one decoded row in one batch."""
    check(*store_and_attend(case, [150, 37, 121], [40, 37, 1]), case[0])


@pytest.mark.parametrize("case", [c for c in ATT_CASES if c[8] and c[9]])
def test_decode_batches_with_keys_cut_over_workgroups(case):
    """One decoded row per sequence (and two): contexts of one key, of less than a slice, and of several slices, in one batch; the cut form
    against the statement and against the form without a workspace."""
    for new in ([1, 1, 1, 1], [2, 1, 2, 1]):
        lens = [1100, 257, 2, 31]
        got = store_and_attend(case, lens, new, seed=50)
        check(*got, case[0])
        plain = store_and_attend(case, lens, new, seed=50, split=False)[0]
        assert float((got[0] - plain).abs().max()) < 0.03 * float(plain.abs().max())


def test_one_far_key_in_another_slice_takes_the_softmax():
    """Scores scaled so that the best key takes the whole weight: each row copies the value of its best key, which lies in any slice."""
    case = (False, 4, 2, 32, 32, 0, 0, 32, True, True)
    got, ref, _ = store_and_attend(case, [1500, 900, 1301], [1, 1, 1], seed=80, scale=40.0)
    err = (got - ref).view(3, 4, 32).abs().amax(-1)
    assert float(err.median()) < 0.05 and float((err < 0.3).float().mean()) > 0.8      # (bf16 scores: two nearly equal best keys may mix)


def test_sizes_the_kernels_do_not_take_are_refused():
    from ssd_amd.hip.lib import SsdHipError
    z = lambda *s: torch.zeros(*s, device=DEV)
    si, li = torch.zeros(1, dtype=torch.int32, device=DEV), torch.zeros(1, dtype=torch.int64, device=DEV)

    def scan(D=8, Dv=8, DP=32, ld=256, Hh=2, cap=1.0, q_off=0, f_off=130):
        H().memory_scan(z(1, 4096), ld, q_off, 32, 64, li, si, z(1, 2, 16, 1024), z(1, 64), 1, Hh, D, Dv, DP, i_off=128, f_off=f_off, bias_i=z(2),
                        bias_f=z(2), cap=cap, m_state=z(1, 2, 16), den=z(1, 2), q_per_seq=1)

    scan()
    for bad in (dict(DP=64), dict(D=40), dict(D=600, DP=640), dict(ld=40), dict(cap=0.0), dict(f_off=255), dict(D=0), dict(Dv=0)):
        with pytest.raises(SsdHipError):
            scan(**bad)
    with pytest.raises(SsdHipError):        # the epilogue's bias comes through its own entry point only
        H().gemm_rows(z(1, 8), z(4, 8), z(1, 4), 1, 4, 8, True, 8)
    with pytest.raises(SsdHipError):        # two sides need both weights
        H().lnorm_post_tail(z(1, 8), z(1, 8), z(8), 1e-5, 1, 8, True, y2_rows=z(1, 8), w1=z(8))
    with pytest.raises(SsdHipError):        # an odd rotated part
        H().winattn_store_norm_rope(z(1, 16), 16, z(8), None, 1e-5, li, z(4), 3, None, z(1, 16), None, None, 1, 2, 0, 8, 8, 16, True)
