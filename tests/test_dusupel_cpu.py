"""CPU-side checks of the Dusupel integration: the config reader, checkpoint names, ranks from tensor shapes, synthetic weights, layer runs,
state slots through the trace engine (a recording runner, no GPU), the bench option, and the oracle's own mechanisms against hand-made
cases and restatements (the delta rule as a sequence of matrix products, the read-out from the decayed state plus the write, the window
with kept first tokens position by position, convolutions of unequal tap counts as one)."""
import json
import math

import pytest
import torch

from oracle import dusupel as F
from ssd_amd.model_config import DusupelConfig, read_native_config
from ssd_amd.weights import param_shapes, synthetic_state_dict

F64 = torch.float64


def small_config():
    return F.make_config([F.delta_layer(mlp=F.dense_mlp()), F.parallel_layer(mlp=F.dense_mlp(40)), F.delta_layer("channel_delta_2", heads=4, kv_heads=2),
                          F.parallel_layer(F.attention_sizes(heads=3, kv_heads=3, conv=2, rot_dims=4), F.delta_sizes(heads=3, kv_heads=1, conv=4))],
                         loop={"start": 1, "stop": 3, "times": 2})


def write(path, cfg, w):
    from safetensors.torch import save_file
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(path / "model.safetensors"))


def test_config_reader_names_ranks_and_synthetic_weights(tmp_path):
    cfg = small_config()
    ranks = lambda i: (6, 5) if i == 0 else (3, 9)
    w = F.random_model(cfg, 0, ranks)
    write(tmp_path, cfg, w)
    c = read_native_config(str(tmp_path))
    assert isinstance(c, DusupelConfig) and c.family == "dusupel" and c.recurrent
    assert [r[0] for r in c.runs()] == [0, 1, 2, 1, 2, 3] == F.layer_order(cfg) and c.num_layers == 6
    d0, p1, d2 = c.layers[0].mixer, c.layers[1].mixer, c.layers[2].mixer
    assert (d0.kind, d0.channel_decay, d0.decay_rank, d0.gate_rank) == ("delta", True, 6, 5) and (d2.decay_rank, d2.gate_rank) == (3, 9)
    assert (d2.heads, d2.kv_heads, c.layers[2].mlp) == (4, 2, None) and c.residual_mult == 0.6
    assert (p1.kind, p1.left.window, p1.left.keep_first, p1.left_scale, p1.right_scale) == ("parallel", 5, 2, 0.7, 1.3)
    assert not p1.right.channel_decay and p1.left.rope.dims == 8 and c.layers[3].mixer.right.conv == 4 and c.layers[1].mlp.ff == 40
    assert {n: tuple(s) for n, s in param_shapes(c)} == {n: tuple(t.shape) for n, t in w.items()}
    sd = synthetic_state_dict(c, 0, 0.02)
    assert set(sd) == set(w) and all(sd[n].shape == w[n].shape for n in w)
    assert float(sd["l0.norm1.b"].float().abs().max()) == 0.0 and float(sd["l0.norm1"].float().min()) == 1.0
    assert float(sd["l0.mix.b"].float().abs().max()) > 0          # a projection whose name happens to end like a norm's bias
    plain = json.loads(json.dumps(cfg))
    plain["loop"] = None
    del plain["layers"][1]["mixer"]["left"]["mask"]
    pc = DusupelConfig.from_json(plain)
    assert pc.num_layers == 4 and (pc.layers[1].mixer.left.window, pc.layers[1].mixer.left.keep_first) == (0, 0)
    for breakit in (lambda d: d["layers"][0].update(type="attention"), lambda d: d["layers"][0]["mlp"].update(kind="moe"),
                    lambda d: d["layers"][1]["mixer"]["left"].update(kv_heads=3), lambda d: d["layers"][1]["mixer"]["right"].update(kv_heads=4),
                    lambda d: d["layers"][1]["mixer"]["left"]["rot"].update(dims=10), lambda d: d["layers"][1]["mixer"]["left"]["rot"].update(dims=3),
                    lambda d: d["loop"].update(stop=9), lambda d: d["loop"].update(times=0)):
        bad = json.loads(json.dumps(cfg))
        breakit(bad)
        with pytest.raises(ValueError):
            DusupelConfig.from_json(bad)
    del w["l2.mix.g1"]
    write(tmp_path, cfg, w)
    with pytest.raises(ValueError):
        read_native_config(str(tmp_path))


def test_projection_and_output_columns_are_disjoint_and_complete():
    from ssd_amd.dusupel import _Plan
    cfg = small_config()
    c = DusupelConfig.from_json(cfg)
    for l in c.layers:
        if l.mixer.kind == "delta":
            l.mixer.decay_rank, l.mixer.gate_rank = 6, 5
        p = _Plan(l)
        spans = [(0, p.CL), (p.CL, p.C - p.CL), (p.lg, p.nl), (p.b, p.d.heads)]
        spans += [(p.lr, p.lr_n)] if p.d.channel_decay else [(p.a, p.d.heads), (p.g, p.nv)]
        cols = sorted(x for lo, n in spans for x in range(lo, lo + n))
        assert cols == list(range(p.NP)) and p.KO % 8 == 0 and 0 <= p.KO - (p.nl + p.nv + p.ff) < 8
        assert p.taps == max(p.d.conv, p.left.conv if p.left else 1)
        if p.d.channel_decay:
            assert p.n2 % 4 == 0 and p.nd == p.d.heads * p.d.padded_dim and p.ld_lr % 8 == 0 and p.ld_lr >= 11


def test_padded_key_channels():
    from ssd_amd.model_config import GatedDelta
    pd = lambda n: GatedDelta(1, 1, n, 1, 1).padded_dim
    assert [pd(n) for n in (1, 32, 33, 64, 65, 96, 128, 129, 512)] == [32, 32, 64, 64, 128, 128, 128, 192, 512]


def test_oracle_delta_rule_as_matrix_products_and_as_a_read_of_the_decayed_state():
    """S_t = (I - beta k k^T) diag(g) S + beta k v^T;  and o = (g S)^T q + u <q, k>: the read-out sees the token's own write."""
    g = torch.Generator().manual_seed(1)
    T, H, D, Dv = 9, 2, 5, 4
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=F64) for n in (D, D, Dv))
    k = F.unit(k)
    beta = torch.sigmoid(torch.randn(T, H, generator=g, dtype=F64))
    decay = torch.rand(T, H, D, generator=g, dtype=F64)
    got = F.delta_rule(q, k, v, beta, decay)
    for h in range(H):
        S = torch.zeros(D, Dv, dtype=F64)
        for t in range(T):
            dS = torch.diag(decay[t, h]) @ S
            u = beta[t, h] * (v[t, h] - dS.T @ k[t, h])
            assert torch.allclose(got[t, h], dS.T @ q[t, h] + u * (q[t, h] @ k[t, h]), rtol=1e-12, atol=1e-12)
            kk = torch.outer(k[t, h], k[t, h])
            S = (torch.eye(D, dtype=F64) - beta[t, h] * kk) @ dS + beta[t, h] * torch.outer(k[t, h], v[t, h])
            assert torch.allclose(got[t, h], S.T @ q[t, h], rtol=1e-10, atol=1e-12)
    # beta 1 and no decay: the state answers the last key with exactly its value
    one = torch.ones(T, H, dtype=F64)
    k = k / k.norm(dim=-1, keepdim=True)
    o = F.delta_rule(k, k, v, one, torch.ones(T, H, 1, dtype=F64))
    assert torch.allclose(o, v, rtol=1e-10, atol=1e-12)


def test_oracle_window_with_kept_first_tokens_position_by_position():
    see = F.visible(12, {"size": 4, "keep_first": 2})
    for i in range(12):
        assert see[i].nonzero().flatten().tolist() == [j for j in range(i + 1) if i - j < 4 or j < 2]
    assert F.visible(5, {"size": 1, "keep_first": 0}).equal(torch.eye(5, dtype=torch.bool))
    assert F.visible(5, None).equal(torch.ones(5, 5, dtype=torch.bool).tril())
    assert F.visible(6, {"size": 2, "keep_first": 10}).equal(torch.ones(6, 6, dtype=torch.bool).tril())


def test_oracle_convolution_and_leading_zero_taps():
    g = torch.Generator().manual_seed(3)
    u, w = torch.randn(7, 3, generator=g, dtype=F64), torch.randn(3, 3, generator=g, dtype=F64)
    y = F.short_conv(u, w)
    for t in range(7):
        for c in range(3):
            assert math.isclose(float(y[t, c]), sum(float(w[c, j] * u[t - 2 + j, c]) for j in range(3) if t - 2 + j >= 0), abs_tol=1e-12)
    assert torch.allclose(F.short_conv(u, torch.nn.functional.pad(w, (2, 0))), y)        # the engine joins unequal tap counts so
    assert torch.allclose(F.short_conv(u, w[:, :1]), u * w[:, 0])


def test_oracle_rotation_keeps_products_a_function_of_the_distance():
    g = torch.Generator().manual_seed(4)
    q, k = torch.randn(1, 1, 10, generator=g, dtype=F64), torch.randn(1, 1, 10, generator=g, dtype=F64)
    at = lambda x, p: F.turn(x, torch.tensor([p]), 6, 100.0)[0, 0]
    assert torch.allclose(at(q, 9) @ at(k, 4), at(q, 105) @ at(k, 100), rtol=1e-10)
    assert torch.equal(at(q, 9)[6:], q[0, 0, 6:]) and abs(float(at(q, 9) @ at(k, 4) - at(q, 9) @ at(k, 5))) > 1e-3


def test_oracle_layer_sums_both_sides_of_one_row_and_repeats_spans():
    cfg = small_config()
    w = F.random_model(cfg, 2)
    toks = [3, 1, 4, 1, 5]
    res = []
    logits = F.forward(cfg, w, toks, res)
    assert len(res) == 6 and torch.isfinite(logits).all()
    x = w["embed"].double()[torch.tensor(toks)]
    h1, h2 = (F.layer_norm(x, w[f"l0.{n}"], w[f"l0.{n}.b"], 1e-5) for n in ("norm1", "norm2"))
    y = F.lin(w["l0.mix.o"], F.channel_delta(h1, w, "l0.mix.", cfg["layers"][0]["mixer"], 1e-5)) + F.dense_ff(h2, w, "l0.mlp.")
    assert torch.allclose(res[0], x + 0.6 * y, rtol=1e-12, atol=1e-12)
    m = x.mean(-1, keepdim=True)
    assert torch.allclose(h1, (x - m) / torch.sqrt(x.var(-1, unbiased=False, keepdim=True) + 1e-5) * w["l0.norm1"].double() + w["l0.norm1.b"].double())
    once = dict(cfg, loop={"start": 1, "stop": 3, "times": 1})
    res1 = []
    F.forward(once, w, toks, res1)
    assert torch.equal(res1[2], res[2]) and len(res1) == 4 and not torch.allclose(res1[3], res[5])


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
    with pytest.raises(RuntimeError):
        eng.step([{"id": "c", "tokens": [3], "want": []}])
    pages_a = list(eng.live["a"].block_table)
    eng.step([{"id": "b", "tokens": [2], "want": []}], end=["a"])
    eng.step([{"id": "c", "tokens": [3] * 100, "want": []}])
    slot, pages_c, _ = eng.runner.calls[-1][0]
    assert slot == 0 and set(pages_a) <= set(pages_c)                      # a's slot and a's pages are in use again
    eng.step([], end=["b", "c"])
    assert eng.blocks.free_state_slots == [0, 1] and len(eng.blocks.free_block_ids) == 8


def test_bench_option_and_equal_size_pairs():
    """bench.py accepts --workload dusupel next to its default; every benchmarked size pairs a Dusupel model with a Fomunex model of the
    same width, layers, vocabulary, attention heads, window and (within half a percent) parameter count."""
    import bench
    from ssd_amd.utils import arch_bench
    assert bench.parse([]).workload == "c4"                                  # the default workload is untouched
    a = bench.parse(["--workload", "dusupel", "--arch-size", "w2048", "--arch-batch", "1", "--arch-only", "dusupel"])
    assert a.workload == "dusupel" and a.arch_size == "w2048" and a.arch_batch == 1 and a.arch_only == "dusupel"
    count = lambda c: sum(math.prod(s) for n, s in param_shapes(c) if n not in ("embed", "pos", "head"))
    for size in arch_bench.SIZES:
        dus, fom = arch_bench.dusupel_models(size)
        assert (dus.hidden_size, dus.vocab_size, dus.num_layers) == (fom.hidden_size, fom.vocab_size, fom.num_layers)
        assert [l.mixer.kind for l in dus.layers] == ["parallel", "delta"] * 2 and dus.recurrent
        a, b = dus.layers[0].mixer.left, fom.layers[0].mixer
        assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window) == (b.heads, b.kv_heads, b.dim, b.vdim, b.window)
        assert abs(count(dus) / count(fom) - 1) < 0.005
