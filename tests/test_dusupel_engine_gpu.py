"""The Dusupel decoder through the engine (Config -> ModelRunner -> block manager with state slots -> HIP kernels) against the plain
whole-sequence oracle (oracle/dusupel.py, float64): small self-made configurations with random weights.  The fp32 element mode is the
sharp one: a key too many or too few at a window's edge or among the kept first tokens, a wrong page, a lost or stale state, a missing
convolution input or a pass that reads another pass's memory is orders of magnitude above rounding there.  Attention inputs are scaled so
that single keys carry the output, and the decays so that some heads and channels remember hundreds of tokens."""
import json
import os

import pytest
import torch

from oracle import dusupel as F

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
    """What bf16 rounding of every sublayer's input alone does to the float64 statement, per position."""
    return row_err(F.forward(cfg, w, toks, round_input=lambda t: t.bfloat16().double()), ref)


def close(got, ref, dtype, floor=None) -> bool:
    """fp32: every position within 1e-4 of the spread.  bf16 (nothing is chosen by a router here, so no position jumps): every position
    within 6 %, or eight times the largest effect that rounding of the sublayer inputs alone has, when `floor` gives it."""
    e = row_err(got, ref)
    bound = TOL[dtype] if dtype == "float32" or floor is None else max(TOL[dtype], 8 * float(floor.max()))
    return bool(torch.isfinite(got).all() and (e < bound).all())


def configs():
    P, D, A, S, M = F.parallel_layer, F.delta_layer, F.attention_sizes, F.delta_sizes, F.dense_mlp
    return {
        # every layer kind, with and without a feed-forward, a loop over two kinds; sizes chosen so that nothing the kernels index by
        # coincides, unequal tap counts side by side, rotations over a part of a head, shared q / k heads
        "all_kinds": F.make_config([D("channel_delta_2", heads=2, dim=12, vdim=20, conv=4, mlp=M(40)),
                                    P(A(heads=6, kv_heads=3, dim=10, vdim=14, conv=2, size=9, keep_first=3, rot_dims=6, base=300.0),
                                      S(heads=4, kv_heads=2, dim=8, vdim=6, conv=5), -0.9, 1.4, M(24)),
                                    D("channel_delta", heads=6, kv_heads=2, dim=40, vdim=8, conv=2, mlp=None),
                                    P(A(heads=3, kv_heads=1, dim=16, vdim=8, conv=4, scale=0.1, size=37, keep_first=21, rot_dims=16),
                                      S(heads=3, kv_heads=3, dim=6, vdim=18, conv=3), 1.2, 0.3, None)], vocab=101, width=72, residual_mult=0.45,
                                   loop={"start": 1, "stop": 3, "times": 2}),
        # values that are 1 or equal: heads, kv heads, taps, window, no kept tokens, no rotation, multipliers, one pass of a loop over all
        "ones": F.make_config([P(A(heads=1, kv_heads=1, dim=8, vdim=8, conv=1, size=1, keep_first=0, rot_dims=0), S(heads=1, dim=8, vdim=8, conv=1),
                                 1.0, 1.0, M(8)), D(heads=1, dim=1, vdim=1, conv=1, mlp=M(8)),
                               P(A(heads=2, kv_heads=2, dim=2, vdim=2, conv=2, size=2, keep_first=1, rot_dims=2), S(heads=2, dim=8, vdim=8, conv=1), mlp=None)],
                              vocab=33, width=40, residual_mult=1.0, loop={"start": 0, "stop": 3, "times": 1}),
        # no window, more kept tokens than the window or the sequence holds, sizes that are no multiple of 8, a loop over a single layer
        "odd_sizes": F.make_config([P(A(heads=6, kv_heads=2, dim=12, vdim=10, conv=3, size=None, keep_first=0, rot_dims=4), S(heads=5, dim=7, vdim=11, conv=3), mlp=M(52)),
                                    P(A(heads=2, kv_heads=2, dim=20, vdim=36, conv=7, size=4, keep_first=30), S(heads=2, kv_heads=1, dim=33, vdim=5, conv=6), mlp=M(20)),
                                    D(heads=5, dim=9, vdim=13, conv=6, mlp=M(28)),
                                    P(A(heads=2, kv_heads=1, dim=8, vdim=6, conv=3, size=6, keep_first=1000), S(), mlp=None)], vocab=77, width=50,
                                   loop={"start": 2, "stop": 3, "times": 3}),
        # sizes the MFMA attention takes (head sizes in multiples of 32, value tiles that fill and that do not fill the register array),
        # kept tokens that end inside and at the border of a 32-key step, state rows of 32, 64 and 128 channels
        "fast_forms": F.make_config([P(A(heads=8, kv_heads=2, dim=32, vdim=64, conv=4, size=70, keep_first=20, rot_dims=16), S(heads=2, dim=32, vdim=32, conv=4), mlp=M(48)),
                                     D(heads=2, dim=64, vdim=64, conv=4, mlp=M(48)),
                                     P(A(heads=20, kv_heads=1, dim=96, vdim=96, conv=3, size=44, keep_first=32, rot_dims=32), S(heads=2, kv_heads=1, dim=128, vdim=32, conv=4), mlp=M(64)),
                                     P(A(heads=4, kv_heads=4, dim=64, vdim=32, conv=2, size=33, keep_first=65, rot_dims=64), S(heads=1, dim=64, vdim=64, conv=3), mlp=None)],
                                    vocab=120, width=96, loop={"start": 0, "stop": 2, "times": 2}),
        "only_delta": F.make_config([D(mlp=M()), D("channel_delta_2", heads=2, dim=24, vdim=4, conv=4)], vocab=40, width=48),
    }


RANKS = {"all_kinds": lambda i: (6, 11) if i == 0 else (3, 5), "ones": (1, 1), "fast_forms": (16, 8)}


def make(name, seed=0):
    cfg = json.loads(json.dumps(configs()[name]))
    return cfg, F.random_model(cfg, seed, RANKS.get(name, (6, 5)))


def engine(tmp_path, cfg, w, dtype, max_tokens=512, block_size=16, **kw):
    from ssd_amd.engine.trace_engine import TraceEngine
    eng = TraceEngine(write_model(tmp_path / "m", cfg, w), dtype=dtype, max_tokens=max_tokens, block_size=block_size, **kw)
    m = eng.runner.model
    for t in m.kv + m.state:                    # a cache row or a state slot that is read before it is written shows as NaN
        for u in (t or ()):
            u.fill_(float("nan"))
    for u in (m.qk, m.v, m.scal, m.o, m.proj):  # and so do rows that no kernel of the step has written
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
def test_whole_prompt_and_every_layer_run_match_the_oracle(tmp_path, name, dtype):
    cfg, w = make(name)
    toks = tokens(83, cfg["vocab"], 1)
    res = []
    ref = F.forward(cfg, w, toks, res)
    floor = floor16(cfg, w, toks, ref)
    eng = engine(tmp_path, cfg, w, dtype)
    eng.runner.model.tap_residuals = []
    got = eng.step([{"id": "a", "tokens": toks, "want": list(range(len(toks)))}], ["a"])
    taps = eng.runner.model.tap_residuals
    assert len(taps) == len(res) == len(F.layer_order(cfg))
    for i, (a, b) in enumerate(zip(taps, res)):
        assert close(a, b, dtype, floor), f"layer run {i}: {rel_err(a, b)}"
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


def test_window_edges_kept_tokens_convolutions_passes_and_scales_show(tmp_path):
    """The model is sensitive to what the test is about: against an oracle whose window is one key longer or shorter, that keeps one first
    token more or fewer, whose convolutions miss their oldest tap, whose slowest decays are a little off, whose passes are one fewer or
    whose sides carry other scales, the engine is FAR from equal; against the right one it is equal -- in prompts, portions and decoding."""
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
            change_cfg(other["layers"], other)
        if change_w:
            for name, fn in change_w.items():
                ow[name] = fn(w[name].clone())
        return rel_err(got[lo:], F.forward(other, ow, toks)[lo:]) > far

    for li in (1, 3):
        for key in ("size", "keep_first"):
            for delta in (1, -1):
                assert differs(lambda l, c: l[li]["mixer"]["left"]["mask"].update(
                    {key: l[li]["mixer"]["left"]["mask"][key] + delta}), lo=cfg["layers"][li]["mixer"]["left"]["mask"]["size"] - 1), (li, key, delta)

    def no_oldest(t):
        t[:, 0] = 0
        return t

    for name in ("l0.mix.q.conv", "l1.mix.left.k.conv", "l1.mix.left.v.conv", "l1.mix.right.k.conv", "l2.mix.v.conv"):
        assert differs(change_w={name: no_oldest}), name
    assert differs(change_w={"l0.mix.dt_bias": lambda t: torch.where(t < -4, t + 1.0, t)}, lo=60)        # only the slowest channels: far tokens
    assert differs(change_w={"l3.mix.right.A_log": lambda t: t + 0.1})
    assert differs(lambda l, c: c["loop"].update(times=1)) and differs(lambda l, c: c.update(residual_mult=0.46))
    assert differs(lambda l, c: l[1]["mixer"].update(left_scale=0.9)) and differs(lambda l, c: l[3]["mixer"].update(right_scale=0.31))
    assert differs(lambda l, c: l[1]["mixer"]["left"]["rot"].update(dims=4))
    assert differs(change_w={"l0.norm2.b": lambda t: t * 0}) and differs(change_w={"final.norm.b": lambda t: t * 0})


def test_one_far_key_at_page_borders_window_edges_and_among_the_first_decides_the_output(tmp_path):
    """A model of one side-by-side layer whose right side is switched off and whose scores are scaled so that the largest one takes the
    whole softmax: every position then copies the value of its best key, wherever it lies -- hundreds of tokens back, at a page's last or
    first slot, among the kept first tokens.  Windowed variants find the best key just inside an edge and not the one just outside."""
    n = 300
    toks = tokens(n, 50, 4)
    refs = {}
    for size, keep in ((None, 0), (48, 0), (48, 17), (33, 64)):
        cfg = F.make_config([F.parallel_layer(F.attention_sizes(heads=2, kv_heads=1, dim=16, vdim=8, conv=3, scale=12.0, size=size,
                                                                keep_first=keep, rot_dims=4), F.delta_sizes(), 1.0, 0.0)], vocab=50, width=32)
        w = F.random_model(cfg, 3)
        refs[size, keep] = ref = F.forward(cfg, w, toks)
        eng = engine(tmp_path / f"{size}_{keep}", cfg, w, "float32", max_tokens=320, block_size=16)
        got = _replay(eng, "a", toks, [100, 101, 103, 160] + list(range(161, n + 1)))
        assert rel_err(got, ref) < 1e-3, (size, keep, rel_err(got, ref))
    assert rel_err(refs[None, 0], refs[48, 0]) > 0.1 and rel_err(refs[48, 17], refs[48, 0]) > 0.1       # the far and the first keys mattered


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
    decoded tokens (the wave-split form), two requests sharing steps; every position against the oracle, the portions against the whole
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
    """Hundreds of keys per row (a long window, and none at all) and a state that has absorbed hundreds of tokens: a prompt of many pages,
    then decoding, then a last portion; in fp32 the rows also equal those of the whole prompt bit by bit."""
    cfg = F.make_config([F.parallel_layer(F.attention_sizes(heads=4, kv_heads=2, dim=32, vdim=32, conv=4, size=400, keep_first=40, rot_dims=16),
                                          F.delta_sizes(heads=2, dim=32, vdim=32, conv=4), mlp=F.dense_mlp(48)),
                         F.delta_layer(heads=2, dim=64, vdim=32, conv=4),
                         F.parallel_layer(F.attention_sizes(heads=4, kv_heads=1, dim=32, vdim=64, conv=2, size=None, rot_dims=8),
                                          F.delta_sizes(heads=1, dim=64, vdim=16, conv=3))], vocab=90, width=64)
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
def test_greedy_generation_through_llm_generate(tmp_path, dtype):
    """The framework's own entry point and scheduler: batched prefill, batched decode (hipGraph replays), pages and state slots from the
    scheduler's block manager (three slots for four prompts), argmax kernels."""
    from ssd_amd import LLM, SamplingParams
    cfg, w = make("all_kinds", seed=7)
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
    layers = []

    def delta():
        G = r(1, 3)
        return F.delta_sizes(heads=G * r(1, 3), kv_heads=G, dim=r(2, 48), vdim=r(1, 30), conv=r(1, 6))

    for _ in range(r(2, 4)):
        mlp = F.dense_mlp(4 * r(1, 12)) if r(0, 3) else None
        if r(0, 1):
            G, dm = r(1, 3), 8 * r(1, 5)
            a = F.attention_sizes(heads=G * r(1, 4), kv_heads=G, dim=dm, vdim=r(1, 40), conv=r(1, 5), scale=0.1 * r(1, 5), size=r(0, 40) or None,
                                  keep_first=r(0, 30), rot_dims=2 * r(0, dm // 2), base=10.0 ** r(1, 6))
            layers.append(F.parallel_layer(a, delta(), 0.2 * r(1, 8), 0.2 * r(1, 8), mlp))
        else:
            layers.append({"type": ("channel_delta", "channel_delta_2")[r(0, 1)], "mixer": delta(), "mlp": mlp})
    lo = r(0, len(layers) - 1)
    loop = {"start": lo, "stop": r(lo, len(layers)), "times": r(1, 3)} if r(0, 2) else None
    cfg = F.make_config(layers, vocab=r(20, 150), width=4 * r(6, 24), residual_mult=0.1 * r(2, 10), loop=loop)
    w = F.random_model(cfg, seed, (r(1, 12), r(1, 12)))
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
