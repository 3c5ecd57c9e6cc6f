"""CPU-side checks of the Tumudra integration: the config reader, checkpoint names, synthetic weights, projection columns, the rotary layout
change at load, wavelength-scaled frequencies, state slots and shared pages through the trace engine (a recording runner, no GPU), the bench
option, and the oracle's own mechanisms against restatements (the matrix memory as one masked sum without a running maximum, retention as a
masked product, attention with borrowed keys position by position)."""
import json
import math

import pytest
import torch

from oracle import tumudra as F
from ssd_amd.model_config import Rotary, TumudraConfig, read_native_config
from ssd_amd.weights import param_shapes, synthetic_state_dict

F64 = torch.float64
SCALING = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}


def small_config():
    return F.make_config([F.parallel_layer(F.attention_sizes(heads=6, kv_heads=3, dim=10, vdim=6, size=7, rot=F.rotation(4, 100.0, SCALING)),
                                           F.memory_sizes(heads=3, dim=7, vdim=5, gate_cap=9.0), F.dense_mlp(40)),
                          F.attention_layer(F.dense_mlp(), heads=4, kv_heads=2, dim=12, vdim=8, scale=0.2, rot=F.rotation(6, 500.0)),
                          F.retention_layer(heads=3, dim=6, vdim=9, decay=[0.5, 0.9, 0.99], rot=F.rotation(4)),
                          F.attention_layer(None, heads=6, kv_heads=2, dim=12, vdim=8, rot=F.rotation(6, 500.0), kv_from=1)], scale=5.5)


def write(path, cfg, w):
    from safetensors.torch import save_file
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(path / "model.safetensors"))


def test_config_reader_names_and_synthetic_weights(tmp_path):
    cfg = small_config()
    w = F.random_model(cfg, 0)
    write(tmp_path, cfg, w)
    c = read_native_config(str(tmp_path))
    assert isinstance(c, TumudraConfig) and c.family == "tumudra" and c.recurrent and c.num_layers == 4 and c.embed_scale == 5.5
    par, a1, ret, a3 = (l.mixer for l in c.layers)
    assert (par.kind, par.left.window, par.left.bias, par.left.rope.layout, par.left.rope.scaling) == ("parallel", 7, False, "interleaved", SCALING)
    assert (par.right.heads, par.right.dim, par.right.vdim, par.right.gate_cap) == (3, 7, 5, 9.0) and c.layers[0].mlp.ff == 40
    assert (a1.kind, a1.window, a1.bias, a1.scale, a1.rope.layout, a1.rope.dims, a1.kv_from) == ("attention", 0, True, 0.2, "halves", 6, -1)
    assert a3.kv_from == 1 and c.layers[3].mlp is None and (ret.decay, ret.rope.dims) == ([0.5, 0.9, 0.99], 4)
    assert {n: tuple(s) for n, s in param_shapes(c)} == {n: tuple(t.shape) for n, t in w.items()}
    assert not any(n.startswith(("l3.mix.k", "l3.mix.v")) for n, _ in param_shapes(c))
    sd = synthetic_state_dict(c, 0, 0.02)
    assert set(sd) == set(w) and all(sd[n].shape == w[n].shape for n in w)
    for n in ("l0.norm1", "l0.mix.left.q.norm", "l0.mix.left.out", "l0.mix.right.out", "l0.mix.right.norm", "final.norm"):
        assert float(sd[n].float().min()) == float(sd[n].float().max()) == 1.0, n
    assert float(sd["l0.mix.right.i"].float().abs().max()) > 0 == float(sd["l0.mix.right.i.b"].float().abs().max())
    only = F.make_config([F.attention_layer()])
    assert not TumudraConfig.from_json(only).recurrent and TumudraConfig.from_json({**only, "embedding": None}).embed_scale == 1.0
    L = lambda i: (lambda d: d["layers"][i]["mixer"])
    for breakit in (lambda d: d["layers"][0].update(type="delta"), lambda d: d["layers"][1]["mlp"].update(kind="moe"),
                    lambda d: L(1)(d).update(kv_heads=3), lambda d: L(0)(d)["left"].update(kv_heads=4), lambda d: L(1)(d)["rot"].update(dims=14),
                    lambda d: L(1)(d)["rot"].update(dims=3), lambda d: L(2)(d).update(decay=[0.5]), lambda d: L(3)(d).update(kv_from=3),
                    lambda d: L(3)(d).update(kv_from=2), lambda d: L(3)(d).update(kv_from=0), lambda d: L(3)(d).update(dim=10, rot=F.rotation(6)),
                    lambda d: L(3)(d).update(vdim=4), lambda d: L(0)(d)["right"].update(gate_cap=0.0)):
        bad = json.loads(json.dumps(cfg))
        breakit(bad)
        with pytest.raises(ValueError):
            TumudraConfig.from_json(bad)
    short = json.loads(json.dumps(cfg))
    for k in ("kv_heads", "dim", "vdim", "rot"):                  # what the borrowing layer leaves out equals the owner's
        del short["layers"][3]["mixer"][k]
    assert TumudraConfig.from_json(short).layers[3].mixer == a3
    chain = json.loads(json.dumps(cfg))
    chain["layers"].append({**chain["layers"][3], "mixer": {**chain["layers"][3]["mixer"], "kv_from": 3}})
    with pytest.raises(ValueError):               # keys come from a layer that has some
        TumudraConfig.from_json(chain)


def test_projection_columns_are_disjoint_and_complete():
    from ssd_amd.tumudra import _Columns
    c = TumudraConfig.from_json(small_config())
    for l in c.layers:
        m = l.mixer
        p = _Columns(m)
        spans = []
        if p.att:
            spans.append((0, p.att.heads * p.att.dim + p.kv_heads * (p.att.dim + p.att.vdim)))
        if p.lin:
            nk = p.lin.heads * p.lin.dim
            spans += [(p.q, nk), (p.k, nk), (p.v, p.nv), (p.g, p.nv)] + ([(p.i, p.lin.heads), (p.f, p.lin.heads)] if p.lin.kind == "memory" else [])
        assert sorted(x for lo, n in spans for x in range(lo, lo + n)) == list(range(p.NP))
        assert p.lin is None or (p.DP % 32 == 0 and p.columns == p.lin.vdim + (p.lin.kind == "memory"))
    assert _Columns(c.layers[3].mixer).kv_heads == 0 and _Columns(c.layers[1].mixer).kv_heads == 2


@pytest.mark.parametrize("scaling", [None, SCALING, {"factor": 4.0, "low": 2.0, "high": 2.5, "original": 1000}])
@pytest.mark.parametrize("dims,base", [(2, 10.0), (16, 100.0), (64, 1e6)])
def test_frequencies_equal_the_statement_and_each_branch_is_met(dims, base, scaling):
    got, want = Rotary(dims, base, "interleaved", scaling).frequencies(), F.angular_frequencies({"dims": dims, "base": base, "scaling": scaling})
    assert all(math.isclose(a, float(b), rel_tol=1e-12) for a, b in zip(got, want)) and len(got) == dims // 2
    if scaling is SCALING and dims == 64:
        plain = Rotary(dims, base).frequencies()
        ratio = [a / b for a, b in zip(got, plain)]
        assert ratio[0] == 1.0 and math.isclose(ratio[-1], 1 / 8.0) and any(0.13 < r < 0.99 for r in ratio) and ratio == sorted(ratio, reverse=True)


def test_interleaved_heads_in_halves_order_keep_every_score():
    """Reordering the entries of q, k and the norm weights as the loader does and turning (i, i + n / 2) gives the scores of turning
    (2i, 2i + 1) in the checkpoint's order."""
    g = torch.Generator().manual_seed(1)
    D, rot = 10, F.rotation(6, 50.0)
    order = Rotary(6, 50.0, "interleaved").to_halves(D)
    q, k = (torch.randn(7, 1, D, generator=g, dtype=F64) for _ in range(2))
    pos = torch.arange(7) * 3
    plain = F.turn(q, pos, rot, True)[:, 0] @ F.turn(k, pos, rot, True)[:, 0].T
    moved = F.turn(q[..., order], pos, rot, False)[:, 0] @ F.turn(k[..., order], pos, rot, False)[:, 0].T
    assert torch.allclose(plain, moved, rtol=1e-12) and sorted(order) == list(range(D))
    assert not torch.allclose(plain, F.turn(q, pos, rot, False)[:, 0] @ F.turn(k, pos, rot, False)[:, 0].T)


def test_oracle_matrix_memory_without_a_running_maximum():
    """With F_t = f_1 + .. + f_t the memory is S~_t = sum_(j <= t) e^(F_t - F_j + i_j) k_j v_j^T = e^(M_t) S_t, so the output is
    S~^T q / (max(|<n~, q>|, 1) + 1e-6 e^(M_t))."""
    g = torch.Generator().manual_seed(2)
    T, H, D, Dv = 12, 2, 5, 4
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=F64) for n in (D, D, Dv))
    i, f = 3.0 * torch.randn(T, H, generator=g, dtype=F64), F.log_sigmoid(torch.randn(T, H, generator=g, dtype=F64))
    got = F.matrix_memory(q, k, v, i, f)
    run = torch.cumsum(f, 0)
    for h in range(H):
        M = 0.0
        for t in range(T):
            M = max(float(f[t, h]) + M, float(i[t, h]))
            c = torch.exp(run[t, h] - run[:t + 1, h] + i[:t + 1, h]) * (k[:t + 1, h] @ q[t, h])
            want = c @ v[:t + 1, h] / (max(abs(float(c.sum())), 1.0) + 1e-6 * math.exp(M))
            assert torch.allclose(got[t, h], want, rtol=1e-9, atol=1e-12)
    # the maximum starts at 0: with a very negative input gate the floor of the denominator is exp(-0) scaled by the forgetting so far
    quiet = F.matrix_memory(q[:1], k[:1], v[:1], torch.full((1, H), -30.0, dtype=F64), torch.full((1, H), -1.0, dtype=F64))
    want = math.exp(-30.0 + 1.0) * (k[0] * q[0]).sum(-1, keepdim=True) * v[0] / (math.exp(1.0) + 1e-6)
    assert torch.allclose(quiet[0], want, rtol=1e-9)
    assert torch.allclose(F.log_sigmoid(torch.tensor([-800.0, -1.0, 0.0, 800.0], dtype=F64)).exp(), torch.sigmoid(torch.tensor([-800.0, -1.0, 0.0, 800.0], dtype=F64)))


def test_oracle_retention_as_a_masked_product():
    g = torch.Generator().manual_seed(3)
    T, H, D, Dv = 9, 2, 4, 3
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=F64) for n in (D, D, Dv))
    decay = [0.5, 0.97]
    got = F.retention(q, k, v, decay)
    d = (torch.arange(T).view(T, 1) - torch.arange(T).view(1, T)).to(F64)
    for h in range(H):
        mask = torch.where(d >= 0, decay[h] ** d, torch.zeros_like(d))
        assert torch.allclose(got[:, h], ((q[:, h] @ k[:, h].T) * mask) @ v[:, h], rtol=1e-10, atol=1e-12)


def test_oracle_window_softmax_and_borrowed_keys():
    assert [r.nonzero().flatten().tolist() for r in F.visible(5, 2)] == [[0], [0, 1], [1, 2], [2, 3], [3, 4]]
    assert F.visible(4, None).equal(torch.ones(4, 4, dtype=torch.bool).tril())
    cfg = small_config()
    w = F.random_model(cfg, 4)
    toks = [3, 1, 4, 1, 5, 9, 2]
    res = []
    assert torch.isfinite(F.forward(cfg, w, toks, res)).all() and len(res) == 4
    x, x2 = res[2], res[0]                       # layer 3 reads res[2], its keys come from what layer 1 read: res[0]
    m = cfg["layers"][3]["mixer"]
    k, v = F.attention_keys_values(x2, w, "l1.mix.", cfg["layers"][1]["mixer"], 1e-5, False)
    heads = torch.zeros(7, 6, 8, dtype=F64)
    for t in range(7):
        q = F.rms((w["l3.mix.q"].double() @ x[t] + w["l3.mix.q.b"].double()).view(6, 12), 1e-5) * w["l3.mix.q.norm"].double()
        q = F.turn(q.view(1, 6, 12), torch.tensor([t]), m["rot"], False)[0]
        for h in range(6):
            heads[t, h] = torch.softmax(k[:t + 1, h // 3] @ q[h] * m["scale"], 0) @ v[:t + 1, h // 3]
    y = heads.view(7, 48) @ w["l3.mix.o"].double().T + w["l3.mix.o.b"].double()
    y = (y - y.mean(-1, keepdim=True)) / torch.sqrt(y.var(-1, unbiased=False, keepdim=True) + 1e-5) * w["l3.norm1"].double()
    assert torch.allclose(res[3], x + y, rtol=1e-10, atol=1e-10)


class _Recorder:
    """Stands in for the ModelRunner: records which slots and pages every step's sequences hold."""
    def __init__(self, config):
        self.num_kvcache_blocks = config.num_kvcache_blocks
        self.calls = []

    def run_rows(self, seqs, want):
        self.calls.append([(s.state_slot, list(s.block_table), len(s) - s.num_cached_tokens) for s in seqs])
        return torch.zeros(sum(len(x) for x in want), 4)


def test_trace_engine_hands_out_pages_and_state_slots_and_takes_them_again(tmp_path):
    from ssd_amd.engine.trace_engine import TraceEngine
    cfg = small_config()
    write(tmp_path, cfg, F.random_model(cfg, 0))
    eng = TraceEngine(str(tmp_path), max_tokens=128, block_size=16, max_live=2, runner_factory=_Recorder)
    eng.step([{"id": "a", "tokens": [1] * 20, "want": [19]}, {"id": "b", "tokens": [2] * 3, "want": []}])
    assert [c[0] for c in eng.runner.calls[-1]] == [0, 1] and [c[2] for c in eng.runner.calls[-1]] == [20, 3]
    pages_a = list(eng.live["a"].block_table)
    eng.step([{"id": "b", "tokens": [2], "want": []}], end=["a"])
    eng.step([{"id": "c", "tokens": [3] * 100, "want": []}])
    slot, pages_c, _ = eng.runner.calls[-1][0]
    assert slot == 0 and set(pages_a) <= set(pages_c)                      # a's slot and a's pages are in use again
    eng.step([], end=["b", "c"])
    assert eng.blocks.free_state_slots == [0, 1] and len(eng.blocks.free_block_ids) == 8


def test_bench_option_and_equal_size_pairs():
    """bench.py accepts --workload tumudra next to its default; every benchmarked size pairs a Tumudra model with a Dusupel model of the same
    width, layers, vocabulary, attention heads, window, state sizes and (within half a percent) parameter count."""
    import bench
    from ssd_amd.utils import arch_bench
    assert bench.parse([]).workload == "c4"                                  # the default workload is untouched
    a = bench.parse(["--workload", "tumudra", "--arch-size", "w2048", "--arch-batch", "1", "--arch-only", "tumudra"])
    assert a.workload == "tumudra" and a.arch_size == "w2048" and a.arch_batch == 1 and a.arch_only == "tumudra"
    count = lambda c: sum(math.prod(s) for n, s in param_shapes(c) if n not in ("embed", "head"))
    for size in arch_bench.SIZES:
        tum, dus = arch_bench.tumudra_models(size)
        assert (tum.hidden_size, tum.vocab_size, tum.num_layers) == (dus.hidden_size, dus.vocab_size, dus.num_layers)
        par, att, ret, shared = (l.mixer for l in tum.layers)
        assert [m.kind for m in (par, att, ret, shared)] == ["parallel", "attention", "retention", "attention"] and shared.kv_from == 1
        b, delta = dus.layers[0].mixer, dus.layers[1].mixer
        assert (par.left.heads, par.left.kv_heads, par.left.dim, par.left.vdim, par.left.window) == \
            (b.left.heads, b.left.kv_heads, b.left.dim, b.left.vdim, b.left.window)
        assert (par.right.heads, par.right.dim, par.right.vdim) == (b.right.heads, b.right.dim, b.right.vdim)
        assert (ret.heads, ret.dim, ret.vdim) == (delta.heads, delta.dim, delta.vdim)
        assert abs(count(tum) / count(dus) - 1) < 0.005
