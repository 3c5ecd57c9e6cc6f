"""The Tumudra decoder through the engine (Config -> ModelRunner -> block manager with state slots -> HIP kernels) against the plain
whole-sequence oracle (oracle/tumudra.py, float64): small self-made configurations with random weights.  The fp32 element mode is the sharp
one: a key too many or too few at a window's edge, a wrong page, a lost or stale state, a running maximum that is not carried, keys of the
wrong layer or a bias that is left out is orders of magnitude above rounding there.  Attention norms are scaled so that single keys carry
the output, and the gates and decays so that some heads remember hundreds of tokens."""
import json
import os

import pytest
import torch

from oracle import tumudra as F

pytestmark = pytest.mark.gpu

TOL = {"float32": 1e-4, "bfloat16": 6e-2}


def write_model(path, cfg, w):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return str(path)


def row_err(got: torch.Tensor, ref: torch.Tensor) -> torch.Tensor:
    d = got.double().cpu() - ref.double()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / ref.double().std()


def rel_err(got, ref) -> float:
    return float(row_err(got, ref).max())


def floor16(cfg, w, toks, ref) -> torch.Tensor:
    """What bf16 rounding of every projection's input alone does to the float64 statement, per position."""
    return row_err(F.forward(cfg, w, toks, round_input=lambda t: t.bfloat16().double()), ref)


def close(got, ref, dtype, floor=None) -> bool:
    """fp32: every position within 1e-4 of the spread.  bf16: every position within 6 %, or eight times the largest effect that rounding of
    the projections' inputs alone has, when `floor` gives it."""
    e = row_err(got, ref)
    bound = TOL[dtype] if dtype == "float32" or floor is None else max(TOL[dtype], 8 * float(floor.max()))
    return bool(torch.isfinite(got).all() and (e < bound).all())


def configs():
    P, A, R, S, M, N, rot = (F.parallel_layer, F.attention_layer, F.retention_layer, F.attention_sizes, F.memory_sizes, F.dense_mlp, F.rotation)
    slow = {"factor": 6.0, "low": 1.0, "high": 3.0, "original": 40}
    return {
        # every layer kind, with and without a feed-forward, keys borrowed over a distance and twice; sizes chosen so that nothing the kernels
        # index by coincides; rotations over a part of a head, frequencies in all three ranges of the scaling
        "all_kinds": F.make_config([A(N(40), heads=6, kv_heads=3, dim=10, vdim=14, rot=rot(6, 300.0)),
                                    P(S(heads=4, kv_heads=2, dim=12, vdim=6, size=9, rot=rot(8, 60.0, slow)), M(heads=3, dim=8, vdim=20, gate_cap=4.0), N(24)),
                                    R(heads=3, dim=14, vdim=10, decay=[0.6, 0.95, 0.998], rot=rot(10, 200.0)),
                                    A(None, heads=3, kv_heads=3, dim=10, vdim=14, rot=rot(6, 300.0), scale=0.5, kv_from=0),
                                    P(S(heads=3, kv_heads=1, dim=16, vdim=8, scale=0.1, size=37, rot=rot(16, 500.0)), M(heads=2, dim=40, vdim=12, gate_cap=15.0)),
                                    A(N(28), heads=12, kv_heads=3, dim=10, vdim=14, rot=rot(6, 300.0), kv_from=0)], vocab=101, width=72, scale=6.0),
        # values that are 1 or equal: heads, kv heads, window, sizes, no rotation, a decay of 1, both sides' inner sizes equal
        "ones": F.make_config([P(S(heads=1, kv_heads=1, dim=8, vdim=8, size=1, rot=rot(0)), M(heads=1, dim=1, vdim=8, gate_cap=1.0), N(8)),
                               A(N(8), heads=1, kv_heads=1, dim=2, vdim=1, rot=rot(2)), R(heads=1, dim=8, vdim=1, decay=[1.0], rot=rot(0)),
                               P(S(heads=2, kv_heads=2, dim=2, vdim=4, size=2, rot=rot(2, 10.0, slow)), M(heads=2, dim=4, vdim=4))], vocab=33, width=40, scale=1.0),
        # no window on the side-by-side attention, sizes that are no multiple of 8
        "odd_sizes": F.make_config([P(S(heads=6, kv_heads=2, dim=12, vdim=10, rot=rot(4)), M(heads=5, dim=7, vdim=11), N(52)),
                                    A(N(20), heads=2, kv_heads=2, dim=20, vdim=36), R(heads=2, dim=33, vdim=5, rot=rot(6), mlp=N(28)),
                                    A(N(12), heads=4, kv_heads=2, dim=20, vdim=36, kv_from=1), R(heads=5, dim=9, vdim=13, rot=rot(8))], vocab=77, width=50),
        # sizes the MFMA attention takes (value tiles that fill and that do not fill the register array; more query heads per key head than a
        # tile has rows), a stacked output product, state rows of 32, 64 and 128 channels
        "fast_forms": F.make_config([P(S(heads=8, kv_heads=2, dim=32, vdim=64, size=70, rot=rot(16)), M(heads=16, dim=32, vdim=32), N(48)),
                                     A(N(64), heads=4, kv_heads=1, dim=64, vdim=48, rot=rot(48)), R(heads=2, dim=64, vdim=64, rot=rot(32)),
                                     A(N(32), heads=20, kv_heads=1, dim=64, vdim=48, rot=rot(48), kv_from=1),
                                     P(S(heads=4, kv_heads=4, dim=96, vdim=96, size=33, rot=rot(96, 1e4, slow)), M(heads=2, dim=128, vdim=32))], vocab=120, width=96),
        "only_attention": F.make_config([A(N(), heads=4, kv_heads=2), A(None, heads=2, kv_heads=2, kv_from=0), A(N(), heads=2, kv_heads=1, dim=16)], vocab=40, width=48),
        "only_recurrent": F.make_config([R(heads=2, dim=12, vdim=20, mlp=N()), R(heads=3, dim=8, vdim=8)], vocab=40, width=48),
    }


def make(name, seed=0):
    cfg = json.loads(json.dumps(configs()[name]))
    return cfg, F.random_model(cfg, seed)


def engine(tmp_path, cfg, w, dtype, max_tokens=512, block_size=16, **kw):
    from ssd_amd.engine.trace_engine import TraceEngine
    eng = TraceEngine(write_model(tmp_path / "m", cfg, w), dtype=dtype, max_tokens=max_tokens, block_size=block_size, **kw)
    m = eng.runner.model
    for t in m.kv + m.state:                    # a cache row or a state slot that is read before it is written shows as NaN
        for u in (t or ()):
            if u is not None:
                u.fill_(float("nan"))
    for u in (m.proj, m.y) + ((m.o, m.den, m.gates) if hasattr(m, "o") else ()):      # and so do rows that no kernel of the step has written
        u.fill_(float("nan"))
    return eng


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def _replay(eng, rid, toks, cuts):
    """Feed toks in portions ending at `cuts`; returns the logits of every position."""
    out, lo = [], 0
    for hi in cuts:
        out.append(eng.step([{"id": rid, "tokens": toks[lo:hi], "want": list(range(hi - lo))}], [rid] if hi == len(toks) else []))
        lo = hi
    return torch.cat(out)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(configs()))
def test_whole_prompt_and_every_layer_match_the_oracle(tmp_path, name, dtype):
    cfg, w = make(name)
    toks = tokens(83, cfg["vocab"], 1)
    res = []
    ref = F.forward(cfg, w, toks, res)
    floor = floor16(cfg, w, toks, ref)
    eng = engine(tmp_path, cfg, w, dtype)
    eng.runner.model.tap_residuals = []
    got = eng.step([{"id": "a", "tokens": toks, "want": list(range(len(toks)))}], ["a"])
    taps = eng.runner.model.tap_residuals
    assert len(taps) == len(res) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(taps, res)):
        assert close(a, b, dtype, floor), f"layer {i}: {rel_err(a, b)}"
    assert close(got, ref, dtype, floor), rel_err(got, ref)


@pytest.mark.parametrize("name", list(configs()))
def test_portions_and_token_by_token_decoding_equal_the_whole_prompt(tmp_path, name):
    cfg, w = make(name, seed=2)
    n = 70
    toks = tokens(n, cfg["vocab"], 3)
    ref = F.forward(cfg, w, toks)
    eng = engine(tmp_path, cfg, w, "float32", block_size=16)
    whole = _replay(eng, "w", toks, [n])
    assert close(whole, ref, "float32"), rel_err(whole, ref)
    schedules = {
        "token by token from the first": list(range(1, n + 1)),
        "prompt then decoding": [41] + list(range(42, n + 1)),
        "portions of two": list(range(2, n + 1, 2)),
        "portions of changing size, cut at and next to page borders": [15, 16, 17, 32, 35, 47, 48, 50, 64, 65, n],
        "three then single tokens over a page border": [3] + list(range(4, 20)) + [n],
    }
    for what, cuts in schedules.items():
        got = _replay(eng, what, toks, cuts)
        # every row is computed from its own inputs, the cache and the state in a fixed order: no dependence on the cut at all
        assert torch.equal(got, whole), what


def test_what_the_design_fixes_shows(tmp_path):
    """The model is sensitive to what the test is about: against an oracle whose window is one key longer or shorter, whose slowest decay,
    gate cap, biases, frequency scaling, embedding factor, score scale or borrowed layer differs a little, the engine is FAR from equal;
    against the right one it is equal -- in prompts, portions and decoding."""
    cfg, w = make("all_kinds", seed=5)
    n = 90
    toks = tokens(n, cfg["vocab"], 6)
    ref = F.forward(cfg, w, toks)
    eng = engine(tmp_path, cfg, w, "float32", block_size=16)
    got = _replay(eng, "a", toks, [40] + list(range(41, n + 1)))
    assert close(got, ref, "float32"), rel_err(got, ref)
    far = 10 * TOL["float32"]          # (rounding itself is near 1e-6)

    def differs(change_cfg=None, change_w=None, lo=0):
        other, ow = json.loads(json.dumps(cfg)), dict(w)
        if change_cfg:
            change_cfg([l["mixer"] for l in other["layers"]], other)
        for name, fn in (change_w or {}).items():
            ow[name] = fn(w[name].clone())
        return rel_err(got[lo:], F.forward(other, ow, toks)[lo:]) > far

    for li in (1, 4):
        for delta in (1, -1):
            size = cfg["layers"][li]["mixer"]["left"]["mask"]["size"]
            assert differs(lambda m, c: m[li]["left"]["mask"].update(size=size + delta), lo=size - 1), (li, delta)
    assert differs(lambda m, c: m[2].update(decay=[0.6, 0.95, 0.99]), lo=60)             # the slowest head only: far tokens
    assert differs(lambda m, c: m[1]["right"].update(gate_cap=4.2)) and differs(lambda m, c: m[4]["right"].update(gate_cap=14.0))
    assert differs(lambda m, c: m[1]["left"]["rot"].pop("scaling")) and differs(lambda m, c: m[1]["left"]["rot"]["scaling"].update(high=2.5))
    assert differs(lambda m, c: m[0]["rot"].update(dims=4)) and differs(lambda m, c: m[3].update(scale=0.48))
    assert differs(lambda m, c: c["embedding"].update(scale=6.1)) and differs(lambda m, c: c["norm"].update(eps=3e-2))
    zero = lambda t: t * 0
    for name in ("l0.mix.q.b", "l0.mix.k.b", "l0.mix.v.b", "l0.mix.o.b", "l3.mix.q.b", "l5.mix.o.b", "l1.mix.right.i.b", "l4.mix.right.f.b"):
        assert differs(change_w={name: zero}), name
    swap = lambda t: t.flip(0)
    for name in ("l1.mix.left.out", "l1.mix.right.out", "l4.mix.right.norm", "l0.mix.k.norm", "l1.mix.left.q.norm", "l1.norm2", "final.norm"):
        assert differs(change_w={name: swap}), name


def test_a_layer_that_borrows_keys_writes_none_and_reads_the_owners_pages(tmp_path):
    """Pages exist once per owner; the cache bytes count owners only; and the borrowed pages are those of the NAMED layer: naming another
    owner of the same sizes changes the result."""
    A = F.attention_layer
    sizes = dict(heads=4, kv_heads=2, dim=8, vdim=8)
    cfg = F.make_config([A(**sizes), A(**sizes), A(F.dense_mlp(), kv_from=0, **{**sizes, "heads": 2})], vocab=50, width=40)
    w = F.random_model(cfg, 3)
    toks = tokens(50, 50, 2)
    eng = engine(tmp_path, cfg, w, "float32")
    m = eng.runner.model
    assert m.kv[2] is m.kv[0] and m.kv[1] is not m.kv[0] and m.kv_block_bytes() == 2 * 2 * (8 + 8) * 16 * 4
    got = _replay(eng, "a", toks, [20, 22] + list(range(23, 51)))
    ref = F.forward(cfg, w, toks)
    assert close(got, ref, "float32"), rel_err(got, ref)
    other = json.loads(json.dumps(cfg))
    other["layers"][2]["mixer"]["kv_from"] = 1
    assert rel_err(got, F.forward(other, w, toks)) > 1e-2
    assert close(_replay(engine(tmp_path / "o", other, w, "float32"), "a", toks, [33, 50]), F.forward(other, w, toks), "float32")


def test_one_far_key_at_page_borders_and_window_edges_decides_the_output(tmp_path):
    """A model of one side-by-side layer whose right side carries almost no weight and whose scores are scaled so that the largest one takes
    the whole softmax: every position then copies the value of its best key, wherever it lies -- hundreds of tokens back, at a page's last
    or first slot.  Windowed variants find the best key just inside the edge and not the one just outside."""
    n = 300
    toks = tokens(n, 50, 4)
    refs = {}
    for size in (None, 48, 33):
        cfg = F.make_config([F.parallel_layer(F.attention_sizes(heads=2, kv_heads=1, dim=16, vdim=8, scale=12.0, size=size, rot=F.rotation(4)), F.memory_sizes())],
                            vocab=50, width=32)
        w = F.random_model(cfg, 3)
        w["l0.mix.right.out"] = w["l0.mix.right.out"] * 1e-3
        refs[size] = F.forward(cfg, w, toks)
        eng = engine(tmp_path / f"{size}", cfg, w, "float32", max_tokens=320, block_size=16)
        got = _replay(eng, "a", toks, [100, 101, 103, 160] + list(range(161, n + 1)))
        assert rel_err(got, refs[size]) < 1e-3, (size, rel_err(got, refs[size]))
    assert rel_err(refs[None], refs[48]) > 0.1 and rel_err(refs[48], refs[33]) > 0.1       # the far keys mattered


@pytest.mark.parametrize("bias", [3.5, -4.0])
def test_the_matrix_memorys_running_maximum_and_floor_over_long_decoding(tmp_path, bias):
    """Input gates that jump (the maximum is set by single tokens and decays slowly), or that are so low that the floor of the denominator --
    exp of minus the maximum, which starts at 0 -- decides the read-out; carried over portions and decoded tokens."""
    cfg = F.make_config([F.parallel_layer(F.attention_sizes(size=3), F.memory_sizes(heads=3, dim=12, vdim=10, gate_cap=8.0)),
                         F.parallel_layer(F.attention_sizes(size=2), F.memory_sizes(heads=2, dim=40, vdim=20, gate_cap=8.0))], vocab=60, width=48)
    w = F.random_model(cfg, 8)
    for i in range(2):
        w[f"l{i}.mix.right.i"] = w[f"l{i}.mix.right.i"] * 4
        w[f"l{i}.mix.right.i.b"] = torch.full_like(w[f"l{i}.mix.right.i.b"], bias)
        w[f"l{i}.mix.right.f.b"] = torch.full_like(w[f"l{i}.mix.right.f.b"], 5.0)
    n = 200
    toks = tokens(n, 60, 3)
    ref = F.forward(cfg, w, toks)
    eng = engine(tmp_path, cfg, w, "float32", max_tokens=256)
    whole = _replay(eng, "w", toks, [n])
    assert close(whole, ref, "float32"), rel_err(whole, ref)
    assert torch.equal(_replay(eng, "d", toks, [2, 4, 80, 97] + list(range(98, n + 1))), whole)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_of_unequal_requests_with_pages_and_slots_used_again(tmp_path, dtype):
    """Up to three live requests, prompt portions of some beside single tokens of others, in a pool too small for all of them at once:
    pages and state slots of finished requests (filled by them, never cleared) are taken again; a request pauses for some steps."""
    cfg, w = make("all_kinds", seed=4)
    V = cfg["vocab"]
    reqs = {r: tokens(n, V, 40 + i) for i, (r, n) in enumerate([("a", 61), ("b", 7), ("c", 38), ("d", 1), ("e", 50), ("f", 23)])}
    refs = {r: F.forward(cfg, w, t) for r, t in reqs.items()}
    eng = engine(tmp_path, cfg, w, dtype, max_tokens=176, block_size=16, max_live=3)
    at = {r: 0 for r in reqs}
    got = {r: [] for r in reqs}
    plan = [[("a", 20), ("b", 3)], [("a", 1), ("b", 4), ("c", 2)], [("a", 17), ("c", 1)], [("c", 30), ("a", 1), ("d", 1)],
            [("a", 22), ("c", 5), ("e", 16)], [("e", 1), ("f", 2)], [("e", 33), ("f", 1)], [("f", 20)]]
    for step in plan:
        entries, end = [], []
        for r, k in step:
            entries.append({"id": r, "tokens": reqs[r][at[r]:at[r] + k], "want": list(range(k))})
            at[r] += k
            if at[r] == len(reqs[r]):
                end.append(r)
        out = eng.step(entries, end)
        lo = 0
        for r, k in step:
            got[r].append(out[lo:lo + k])
            lo += k
    assert all(at[r] == len(reqs[r]) for r in reqs)
    assert not eng.live and len(eng.blocks.free_block_ids) == 11 and eng.blocks.free_state_slots == [0, 1, 2]
    for r in reqs:
        g = torch.cat(got[r])
        assert close(g, refs[r], dtype, floor16(cfg, w, reqs[r], refs[r])), (r, rel_err(g, refs[r]))
    if dtype == "float32":
        for r in ("a", "e"):          # each alone gives exactly the same rows
            assert torch.equal(_replay(eng, r + "x", reqs[r], [len(reqs[r])]), torch.cat(got[r]))


@pytest.mark.parametrize("block_size", [32, 64])
def test_bf16_fast_forms_through_the_engine_portions_decoding_and_mixed_steps(tmp_path, block_size):
    """bf16 with 32 / 64-token pages and sizes that the MFMA attention takes: whole prompt, portions cut at and next to page borders,
    decoded tokens (the decode launch), two requests sharing steps; every position against the oracle, the portions against the whole
    prompt, and the MFMA attention against the scalar form on the same inputs."""
    cfg, w = make("fast_forms", seed=9)
    n = 190
    ta, tb = tokens(n, cfg["vocab"], 30), tokens(77, cfg["vocab"], 31)
    ra, rb = F.forward(cfg, w, ta), F.forward(cfg, w, tb)
    fa, fb = floor16(cfg, w, ta, ra), floor16(cfg, w, tb, rb)
    eng = engine(tmp_path, cfg, w, "bfloat16", max_tokens=384, block_size=block_size)
    whole = _replay(eng, "w", ta, [n])
    assert close(whole, ra, "bfloat16", fa), rel_err(whole, ra)
    eng.runner.model.scalar_attention = True
    scalar = _replay(eng, "s", ta, [n])
    eng.runner.model.scalar_attention = False
    assert not torch.equal(whole, scalar) and row_err(whole, scalar.double().cpu()).median() < 0.02
    cuts = sorted({block_size - 1, block_size, block_size + 1, 2 * block_size + 2, 150} | set(range(151, n + 1)))
    got = _replay(eng, "c", ta, cuts)
    assert close(got, ra, "bfloat16", fa), rel_err(got, ra)
    assert row_err(got, whole.double().cpu()).median() < 0.02
    ga, gb, ia, ib = [], [], 0, 0
    for ka, kb in [(40, 1), (1, 1), (1, 30), (25, 1), (1, 44)] + [(1, 0)] * 10 + [(n - 78, 0)]:
        entries = []
        if ka:
            entries.append({"id": "a", "tokens": ta[ia:ia + ka], "want": list(range(ka))})
        if kb:
            entries.append({"id": "b", "tokens": tb[ib:ib + kb], "want": list(range(kb))})
        ia, ib = ia + ka, ib + kb
        out = eng.step(entries, [r for r, done in (("a", ia == n), ("b", ib == 77 and kb)) if done])
        ga.append(out[:ka])
        gb.append(out[ka:ka + kb])
    assert ia == n and ib == 77
    assert close(torch.cat(ga), ra, "bfloat16", fa) and close(torch.cat(gb), rb, "bfloat16", fb)


def test_fast_forms_over_a_long_context_in_both_modes(tmp_path):
    """Hundreds of keys per row (a long window, and none at all: decoded rows cut their keys over workgroups) and states that have absorbed
    hundreds of tokens: a prompt of many pages, then decoding, then a last portion; in fp32 the rows also equal those of the whole prompt
    bit by bit."""
    cfg = F.make_config([F.attention_layer(F.dense_mlp(48), heads=4, kv_heads=2, dim=32, vdim=64, rot=F.rotation(8)),
                         F.parallel_layer(F.attention_sizes(heads=4, kv_heads=2, dim=32, vdim=32, size=400, rot=F.rotation(16)), F.memory_sizes(heads=2, dim=32, vdim=32)),
                         F.retention_layer(heads=2, dim=64, vdim=32, decay=[0.99, 0.9995], rot=F.rotation(64)),
                         F.attention_layer(heads=6, kv_heads=2, dim=32, vdim=64, rot=F.rotation(8), kv_from=0)], vocab=90, width=64)
    w = F.random_model(cfg, 21)
    n = 700
    toks = tokens(n, cfg["vocab"], 22)
    ref = F.forward(cfg, w, toks)
    cuts = [600] + list(range(601, 641)) + [n]
    eng = engine(tmp_path, cfg, w, "bfloat16", max_tokens=768, block_size=64)
    got = _replay(eng, "a", toks, cuts)
    assert close(got, ref, "bfloat16", floor16(cfg, w, toks, ref)), rel_err(got, ref)
    eng32 = engine(tmp_path / "f", cfg, w, "float32", max_tokens=768, block_size=64)
    got32 = _replay(eng32, "a", toks, cuts)
    assert close(got32, ref, "float32"), rel_err(got32, ref)
    assert torch.equal(_replay(eng32, "w", toks, [n]), got32)


def test_long_decoding_over_many_pages(tmp_path):
    cfg, w = make("all_kinds", seed=8)
    n = 230
    toks = tokens(n, cfg["vocab"], 9)
    ref = F.forward(cfg, w, toks)
    for dtype in ("float32", "bfloat16"):
        eng = engine(tmp_path / dtype, cfg, w, dtype, max_tokens=256, block_size=16)
        got = _replay(eng, "a", toks, [5] + list(range(6, n + 1)))
        assert close(got, ref, dtype, floor16(cfg, w, toks, ref)), (dtype, rel_err(got, ref))


def test_pool_and_live_limits_are_enforced(tmp_path):
    cfg, w = make("ones")
    eng = engine(tmp_path, cfg, w, "float32", max_tokens=64, block_size=16, max_live=2)
    eng.step([{"id": "a", "tokens": [1] * 20, "want": []}, {"id": "b", "tokens": [2] * 20, "want": []}])
    with pytest.raises(RuntimeError):
        eng.step([{"id": "c", "tokens": [3], "want": []}])
    eng.step([], ["a"])
    eng.step([{"id": "c", "tokens": [3] * 30, "want": [29]}])
    with pytest.raises(RuntimeError):
        eng.step([{"id": "b", "tokens": [2] * 20, "want": []}])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["all_kinds", "only_attention"])
def test_greedy_generation_through_llm_generate(tmp_path, name, dtype):
    """The framework's own entry point and scheduler: batched prefill, batched decode (hipGraph replays), pages and state slots from the
    scheduler's block manager (three slots for four prompts; a model without recurrent layers has none), argmax kernels."""
    from ssd_amd import LLM, SamplingParams
    cfg, w = make(name, seed=7)
    path = write_model(tmp_path / "m", cfg, w)
    prompts = [tokens(n, cfg["vocab"], 20 + n) for n in (5, 19, 1, 34)]
    new = 24
    llm = LLM(path, dtype=dtype, kvcache_block_size=16, num_kvcache_blocks=32, max_num_seqs=3, max_model_len=128,
              max_num_batched_tokens=128)
    outs, _ = llm.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=new, ignore_eos=True), use_tqdm=False)
    assert len(outs) == len(prompts)
    for i, (p, o) in enumerate(zip(prompts, outs)):
        gen = o["token_ids"]
        assert len(gen) == new
        # teacher forcing: every generated token is the argmax of its step.  The argmax kernels read the logits rounded to bf16, and in
        # bf16 the logits carry the mode's rounding: a runner-up within that of the top may win
        lg = F.forward(cfg, w, p + gen[:-1])[len(p) - 1:]
        top = lg.max(-1).values
        chosen = lg[torch.arange(new), torch.tensor(gen)]
        slack = 1e-3 if dtype == "float32" else 0.3
        assert ((top - chosen) <= 2.0 ** -7 * top.abs() + slack * lg.std()).all(), (i, (top - chosen).max())


@pytest.mark.parametrize("seed", range(4))
def test_random_configurations_in_both_modes_whole_and_in_portions(tmp_path, seed):
    g = torch.Generator().manual_seed(100 + seed)
    r = lambda lo, hi: int(torch.randint(lo, hi + 1, (1,), generator=g))
    layers, owners = [], []

    def rot(dim):
        sc = {"factor": 1.0 + r(1, 40) / 5, "low": 1.0, "high": 1.0 + r(1, 6), "original": r(20, 200)} if r(0, 1) else None
        return F.rotation(2 * r(0, dim // 2), 10.0 ** r(1, 6), sc)

    def attention(size):
        G, dm = r(1, 3), 8 * r(1, 5)
        return dict(heads=G * r(1, 4), kv_heads=G, dim=dm, vdim=r(1, 40), scale=0.1 * r(1, 5), rot=rot(dm), size=size)

    for i in range(r(3, 5)):
        mlp = F.dense_mlp(4 * r(1, 12)) if r(0, 3) else None
        kind = r(0, 3)
        if kind == 0:
            right = F.memory_sizes(heads=r(1, 4), dim=r(1, 48), vdim=r(1, 30), gate_cap=0.5 * r(1, 30))
            layers.append(F.parallel_layer(F.attention_sizes(**attention(r(0, 40) or None)), right, mlp))
        elif kind == 1:
            dm, hh = r(2, 48), r(1, 4)
            layers.append(F.retention_layer(hh, dm, r(1, 30), [1.0 - 0.5 ** r(1, 12) for _ in range(hh)], rot(dm), mlp))
        elif kind == 2 and owners:
            j = owners[r(0, len(owners) - 1)]
            m = layers[j]["mixer"]
            layers.append(F.attention_layer(mlp, **{k: m[k] for k in ("kv_heads", "dim", "vdim", "rot")}, heads=m["kv_heads"] * r(1, 5),
                                            scale=0.1 * r(1, 5), kv_from=j))
        else:
            owners.append(i)
            layers.append(F.attention_layer(mlp, **attention(None)))
    cfg = F.make_config(layers, vocab=r(20, 150), width=4 * r(6, 24), scale=0.5 * r(1, 16))
    w = F.random_model(cfg, seed)
    toks = tokens(60, cfg["vocab"], seed)
    ref = F.forward(cfg, w, toks)
    floor = floor16(cfg, w, toks, ref)
    for dtype in ("float32", "bfloat16"):
        eng = engine(tmp_path / dtype, cfg, w, dtype, max_tokens=128, block_size=16)
        whole = _replay(eng, "w", toks, [60])
        assert close(whole, ref, dtype, floor), (dtype, rel_err(whole, ref))
        parts = _replay(eng, "p", toks, [7, 9, 31, 32, 33] + list(range(34, 61)))
        assert close(parts, ref, dtype, floor), (dtype, rel_err(parts, ref))


def test_trace_runner_command_line(tmp_path):
    """bin/trace_run as a user runs it: steps on standard input, `done <step>` after each, <step>.f32 for the steps that want logits;
    two requests share steps, one ends and its pages and slot go to a third."""
    import subprocess
    import sys
    import numpy as np
    from tests.conftest import ROOT
    cfg, w = make("all_kinds", seed=11)
    path = write_model(tmp_path / "m", cfg, w)
    V = cfg["vocab"]
    ta, tb, tc = tokens(70, V, 1), tokens(9, V, 2), tokens(40, V, 3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ta[:50], "want": [0, 49]}, {"id": "b", "tokens": tb[:8], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": tb[8:], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": ta[50:52], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "c", "tokens": tc, "want": [39]}, {"id": "a", "tokens": ta[52:], "want": [17]}], "end": ["a", "c"]}]
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "192", "--max-live", "2"], input="".join(json.dumps(s) + "\n" for s in steps), text=True,
                       capture_output=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done ")] == [f"done {i}" for i in range(4)]
    assert sorted(os.listdir(out)) == ["0.f32", "1.f32", "3.f32"]
    read = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, V).copy())
    ra, rb, rc = F.forward(cfg, w, ta), F.forward(cfg, w, tb), F.forward(cfg, w, tc)
    assert rel_err(read(0), ra[[0, 49]]) < 1e-3 and rel_err(read(1), rb[[8]]) < 1e-3
    assert rel_err(read(3), torch.stack([rc[39], ra[69]])) < 1e-3
