"""The Dusupel decoder on MI355X: PARALLEL layers with a layer norm for each side -- x <- x + m (mixer(ln1(x)) + ff(ln2(x))), both of
the same fp32 residual row --; two kinds of mixer: a gated delta rule with a decay per key channel, or two mixers side by side (windowed
attention that keeps the first tokens, over a paged cache, and a gated delta rule with a decay per head), every q / k / v channel passing
a short causal convolution; dense silu-GLU feed-forwards; a span of layers may run several passes with the same weights, each pass with
cache pages and state of its own.

Launches per layer run (T token rows):
    delta          [q | k | v | b | a1 | g1] GEMM -> delta_prep (convolutions, unit q / k, beta, low-rank rows) -> [a2 | g2] GEMM with the
                   decays and the gate as epilogue -> delta_scan (state slot) -> group_gate_norm
    side by side   [lq | lk | lv | rq | rk | rv | lg | rb | ra | rg] GEMM -> winattn_store_conv_rope (convolutions, rope, cache pages) ->
                   delta_prep -> winattn_paged (window + first tokens, output gate and left scale as epilogue) -> delta_scan (also saves
                   the convolution inputs of both sides) -> group_gate_norm (right scale)
    feed-forward   [gate | up] GEMM with the GLU as epilogue (fp32 mode: + glu_rows)
    [W_o | W_down] ONE GEMM over the row [mixer output | activations]: mixer and feed-forward meet in its accumulator
    lnorm_tail     x += m * its rows; both norms of the next layer
over pre-allocated buffers (nothing is allocated during a forward).  Same interface as ssd_amd.model.HipDecoder towards the ModelRunner.

Arithmetic: residual rows and their sums, norms, rotation angles, scores, softmax, convolutions, unit norms, step sizes, decays, recurrent
states, gates and every GEMM accumulator are fp32 in both modes.  dtype "bfloat16": weights, GEMM-input rows (also the inner rows of the
low-rank projections) and the KV cache are bf16; "float32": they are fp32 and products are FMA chains.
"""
from __future__ import annotations

import torch

from ssd_amd.hip import ops as H
from ssd_amd.model import AttnMeta
from ssd_amd.model_config import DusupelConfig
from ssd_amd.res32 import Res32Decoder

BF16 = torch.bfloat16


def _up8(n: int) -> int:
    return -(-n // 8) * 8


class _Plan:
    """Columns of one layer's fp32 projection row and of its output-GEMM input row.  The convolved channels come first (left q, k, v, then
    the delta rule's q, k, v): they share one convolution state of `taps` - 1 rows, the shorter side's weights padded with zero taps."""

    def __init__(self, lc):
        m = lc.mixer
        left, d = (m.left, m.right) if m.kind == "parallel" else (None, m)
        self.left, self.d, self.ff = left, d, (lc.mlp.ff if lc.mlp is not None else 0)
        self.left_scale, self.right_scale = (m.left_scale, m.right_scale) if left else (1.0, 1.0)
        self.CL = left.conv_channels if left else 0
        self.C = self.CL + d.conv_channels
        self.taps = max(left.conv if left else 1, d.conv)
        self.nl = left.heads * left.vdim if left else 0          # left output entries
        self.nv = d.heads * d.vdim
        o = self.C
        self.lg, o = o, o + self.nl
        self.b, o = o, o + d.heads
        if d.channel_decay:
            self.lr, self.lr_n = o, d.decay_rank + d.gate_rank   # inner rows of the low-rank projections: decay, then gate
            self.ld_lr = _up8(self.lr_n)
            o += self.lr_n
            self.nd = d.heads * d.padded_dim             # decay columns, heads padded as the scan reads them
            self.n2 = -(-(self.nd + self.nv) // 4) * 4
        else:
            self.a, o = o, o + d.heads
            self.g, o = o, o + self.nv
        self.NP = o
        self.KO = _up8(self.nl + self.nv + self.ff)              # output-GEMM input row: [left | delta | activations | zeros]


class HipDusupel(Res32Decoder):
    def __init__(self, cfg: DusupelConfig, *, max_tokens: int, max_seqs: int, max_blocks: int, block_size: int, max_model_len: int,
                 device: torch.device, tp_rank: int = 0, tp_size: int = 1, tp_group=None, max_logit_rows: int | None = None,
                 max_split_tokens: int = 256, force_collectives: bool = False, taps=None, dtype: str = "bfloat16"):
        assert tp_size == 1 and taps is None, "Dusupel models are single-rank and have no activation taps"
        assert dtype in ("bfloat16", "float32")
        self.cfg, self.device = cfg, device
        self.f32 = dtype == "float32"
        self.elem = torch.float32 if self.f32 else BF16
        self.tp_rank, self.tp_size, self.tp_group = 0, 1, None
        self.use_coll, self.custom_ar, self.acts = False, None, None
        self.h = self.W = cfg.hidden_size
        self.V = cfg.vocab_size
        self.Vp = _up8(self.V)
        self.block_size, self.max_blocks = block_size, max_blocks
        self.max_tokens = max_tokens
        self.max_logit_rows = max_logit_rows or max_tokens
        self.runs = cfg.runs()
        self.plans = [_Plan(lc) for lc in cfg.layers]
        self.state_slots = max_seqs if cfg.recurrent else 0      # one per live sequence; the block manager hands them out
        self.w: dict[str, torch.Tensor] = {}
        self.kv: list = []
        self.state: list = []
        self.scalar_attention = False                 # tests / probes: the scalar form of the attention also where the MFMA form fits
        self.tap_residuals: list | None = None         # tests: receives a copy of the residual rows after every layer run (eager only)

        def z(*shape, dtype=torch.float32):
            return torch.zeros(*shape, dtype=dtype, device=device)

        T, W, el, pl = max_tokens, self.W, self.elem, self.plans
        self.x = z(T, W)
        self.hn1 = z(T, W, dtype=el)
        self.hn2 = z(T, W, dtype=el)
        self.y = z(T, W)
        self.proj = z(T * max(p.NP for p in pl))
        self.qk = z(T * max(p.d.kv_heads * 2 * p.d.padded_dim for p in pl))
        self.v = z(T * max(p.nv for p in pl))
        self.scal = z(T * max(4 * p.d.heads for p in pl))
        self.o = z(T * max(p.nv for p in pl))
        if any(p.d.channel_decay for p in pl):
            self.lr = z(T * max(p.ld_lr for p in pl if p.d.channel_decay), dtype=el)
            self.dg = z(T * max(p.n2 for p in pl if p.d.channel_decay))
        if any(p.left for p in pl):
            self.q = z(T * max(p.left.heads * p.left.dim for p in pl if p.left), dtype=el)
        # rows [left | delta | activations | padding] of every distinct layer shape: the padding columns stay zero
        self.cat = {key: z(T * key[0], dtype=el) for key in {(p.KO, p.nl + p.nv + p.ff) for p in pl}}
        if self.f32 and any(p.ff for p in pl):
            self.ab = z(T * 2 * max(p.ff for p in pl))           # fp32 [gate | up] rows (bf16: the GEMM epilogue applies the GLU)
        R = self.max_logit_rows
        self.lastn = z(R, W, dtype=el)
        self.logits32 = z(R, self.V)
        self.logits = z(R, self.Vp, dtype=BF16)

    # ---------------------------------------------------------------------------------------------
    def load_weights(self, weight_iter) -> None:
        """Consumes (name, tensor) pairs under the checkpoint's names.  Matrices that read the same rows are stacked (the projection row of
        _Plan; [gate | up]); [a2 | g2] become one block matrix over the concatenated inner rows, the decay part's heads padded to the
        scan's width; [W_o left | W_o | W_down] are joined along the input side; convolution weights stacked, the shorter side padded with
        leading zero taps; what enters a recurrence directly (exp(A_log), dt_bias) is kept as fp32."""
        raw = {n: t.to(self.device) for n, t in weight_iter}
        cv = lambda t: t.to(self.elem).contiguous()
        w = self.w = {}

        def norm(n):
            w[n], w[n + ".b"] = cv(raw[n]), cv(raw[n + ".b"])

        def conv(p, taps):
            c = torch.cat([raw[p + n + ".conv"] for n in "qkv"], dim=0)
            return torch.nn.functional.pad(c, (taps - c.shape[1], 0))

        w["embed"], w["head"] = cv(raw["embed"]), cv(raw["head"])
        norm("final.norm")
        for i, lc in enumerate(self.cfg.layers):
            p, pl = f"l{i}.", self.plans[i]
            d, q = pl.d, p + ("mix.right." if pl.left else "mix.")
            L = p + "mix.left."
            norm(p + "norm1")
            rate = torch.exp(raw[q + "A_log"].float())
            rows = [raw[L + n] for n in "qkv"] if pl.left else []
            rows += [raw[q + n] for n in "qkv"]
            rows += ([raw[L + "g"]] if pl.left else []) + [raw[q + "b"]]
            if d.channel_decay:
                rows += [raw[q + "a1"], raw[q + "g1"]]
                D, DP = d.dim, d.padded_dim
                m2 = torch.zeros(pl.n2, pl.ld_lr, dtype=torch.float32, device=self.device)
                a2 = torch.zeros(d.heads, DP, d.decay_rank, dtype=torch.float32, device=self.device)
                a2[:, :D] = raw[q + "a2"].float().view(d.heads, D, -1)
                m2[:pl.nd, :d.decay_rank] = a2.view(pl.nd, -1)
                m2[pl.nd:pl.nd + pl.nv, d.decay_rank:pl.lr_n] = raw[q + "g2"].float()
                w[p + "mix.low2"] = cv(m2)
                bias = torch.zeros(d.heads, DP, dtype=torch.float32, device=self.device)
                bias[:, :D] = raw[q + "dt_bias"].float().view(d.heads, D)
                w[p + "mix.bias"] = bias.view(-1).contiguous()
                w[p + "mix.rate"] = rate.repeat_interleave(DP).contiguous()
            else:
                rows += [raw[q + "a"], raw[q + "g"]]
                w[p + "mix.bias"], w[p + "mix.rate"] = raw[q + "dt_bias"].float().contiguous(), rate.contiguous()
            w[p + "mix.in"] = cv(torch.cat(rows, dim=0))
            assert w[p + "mix.in"].shape[0] == pl.NP
            w[p + "mix.conv"] = cv(conv(q, pl.taps))
            w[p + "mix.norm"] = cv(raw[q + "norm"])
            outs = [raw[q + "o"]]
            if pl.left:
                w[p + "mix.left.conv"] = cv(conv(L, pl.taps))
                w[p + "mix.left.freqs"] = torch.tensor(pl.left.rope.frequencies() or [0.0], dtype=torch.float64).to(torch.float32).to(self.device)
                outs = [raw[L + "o"]] + outs
            if pl.ff:
                norm(p + "norm2")
                gate, up = raw[p + "mlp.gate"], raw[p + "mlp.up"]
                # bf16: rows interleaved (gate_0, up_0, gate_1, ...) for the GEMM's paired epilogue; fp32: [gate | up], a GLU launch follows
                w[p + "mlp.gu"] = cv(torch.cat([gate, up], dim=0) if self.f32 else torch.stack([gate, up], dim=1).reshape(-1, self.W))
                outs.append(raw[p + "mlp.down"])
            out = torch.cat(outs, dim=1)
            w[p + "out"] = cv(torch.nn.functional.pad(out, (0, pl.KO - out.shape[1])))
        torch.cuda.synchronize(self.device)

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.w.values())

    def active_weight_bytes(self, T: int = 1) -> int:
        """HBM bytes of weights one forward of T tokens must stream at least: every matrix once per layer RUN, the LM head once, one
        embedding row per token."""
        per = {n: t.numel() * t.element_size() for n, t in self.w.items()}
        total = per["head"] + per["final.norm"] * 2
        for li, _ in self.runs:
            total += sum(v for n, v in per.items() if n.startswith(f"l{li}."))
        return total

    def kv_block_bytes(self) -> int:
        es = 4 if self.f32 else 2
        n = sum(p.left.kv_heads * (p.left.dim + p.left.vdim) * self.block_size * es for p in (self.plans[li] for li, _ in self.runs) if p.left)
        return max(n, 1)

    def state_bytes(self) -> int:
        """Bytes of recurrent state one live sequence holds (all layer runs)."""
        return sum((p.d.heads * p.d.vdim * p.d.padded_dim + (p.taps - 1) * p.C) * 4 for p in (self.plans[li] for li, _ in self.runs))

    def alloc_kv(self, num_blocks: int) -> None:
        """Per layer RUN: the attention side -> K pages [blocks][G][block][dim] and V pages transposed [blocks][G][vdim][block]; the delta
        rule -> state [slots][H][vdim][key channels, padded] fp32 (transposed) and the last taps - 1 convolution inputs of both sides
        [slots][taps - 1][channels] fp32.  A slot is not cleared when it is handed out: a forward whose rows start at position 0 starts
        from zero by itself."""
        self.num_blocks = num_blocks
        self.kv, self.state = [], []
        dev, bs, S = self.device, self.block_size, self.state_slots
        for li, _ in self.runs:
            p = self.plans[li]
            a, d = p.left, p.d
            self.kv.append(None if a is None else (torch.zeros(num_blocks, a.kv_heads, bs, a.dim, dtype=self.elem, device=dev),
                                                   torch.zeros(num_blocks, a.kv_heads, a.vdim, bs, dtype=self.elem, device=dev)))
            self.state.append((torch.zeros(S, d.heads, d.vdim, d.padded_dim, dtype=torch.float32, device=dev),
                               torch.zeros(S, max(p.taps - 1, 1), p.C, dtype=torch.float32, device=dev)))

    # ---------------------------------------------------------------------------------------------
    def launch_mixer(self, run: int, li: int, T: int, positions, meta: AttnMeta, cat: torch.Tensor) -> None:
        """hn1 -> the mixer's columns of the output-GEMM input rows."""
        cfg, w, f, W = self.cfg, self.w, self.f32, self.W
        p, pl = f"l{li}.mix.", self.plans[li]
        d, a = pl.d, pl.left
        assert meta.state_slots is not None, "a model with recurrent layers needs the sequences' state slots"
        S, conv = self.state[run]
        seqs = dict(cu_q=meta.cu_q) if meta.cu_q is not None else dict(q_per_seq=meta.q_per_seq)
        proj, NP, slots = self.proj, pl.NP, meta.state_slots
        H.gemm_rows(self.hn1, w[p + "in"], proj, T, NP, W, f)
        if a is not None:
            kc, vc = self.kv[run]
            H.winattn_store_conv_rope(proj, NP, 0, w[p + "left.conv"], pl.taps, conv, pl.C, slots, positions, meta.B, w[p + "left.freqs"],
                                      a.rope.dims, meta.slot_mapping, self.q, kc, vc, T, a.heads, a.kv_heads, a.dim, a.vdim, self.block_size,
                                      f, **seqs)
        low = dict(lr_off=pl.lr, lr_n=pl.lr_n, lr_out=self.lr, ld_lr=pl.ld_lr) if d.channel_decay else \
            dict(a_off=pl.a, rate=w[p + "rate"], bias=w[p + "bias"])
        H.delta_prep(proj, NP, pl.CL, w[p + "conv"], pl.taps, conv, pl.C, pl.CL, slots, positions, meta.B, pl.b, self.qk, self.v, self.scal, T,
                     d.heads, d.kv_heads, d.dim, d.vdim, d.padded_dim, f, **low, **seqs)
        if d.channel_decay:
            H.gemm_rows_decay_gate(self.lr, w[p + "low2"], self.dg, T, pl.n2, pl.ld_lr, w[p + "rate"], w[p + "bias"], pl.nd, f)
        if a is not None:
            H.winattn_paged(self.q, kc, vc, None, None, meta.block_tables, self.max_blocks, positions, meta.B, T, a.heads, a.kv_heads, a.dim,
                            a.vdim, self.block_size, a.window, a.scale, 0.0, cat, f, max_q=0 if self.scalar_attention else meta.max_q,
                            keep_first=a.keep_first, gate=proj[pl.lg:], ldg=NP, out_scale=pl.left_scale, ldo=pl.KO, **seqs)
        H.delta_scan(self.qk, self.v, self.scal, positions, slots, S, self.o, meta.B, d.heads, d.kv_heads, d.dim, d.vdim,
                     d.padded_dim, proj, NP, 0, pl.C, conv, pl.taps, **(dict(decay=self.dg, ldd=pl.n2) if d.channel_decay else {}), **seqs)
        gate = (self.dg[pl.nd:], pl.n2, H.GATE_NONE) if d.channel_decay else (proj[pl.g:], NP, H.GATE_SILU)
        H.group_gate_norm(self.o, gate[0], gate[1], w[p + "norm"], cfg.norm_eps, cat[pl.nl:], T, pl.nv, d.heads, False, f, gate_act=gate[2],
                          w_period=d.vdim, out_scale=pl.right_scale, ldo=pl.KO)

    def launch_mlp(self, li: int, T: int, cat: torch.Tensor) -> None:
        """hn2 -> the activations' columns of the output-GEMM input rows."""
        pl, gu = self.plans[li], self.w[f"l{li}.mlp.gu"]
        act = cat[pl.nl + pl.nv:]
        if self.f32:
            H.gemm_rows(self.hn2, gu, self.ab, T, 2 * pl.ff, self.W, True)
            H.glu_rows(self.ab, act, T, pl.ff, H.GLU_SILU, True, ldo=pl.KO)
        else:
            H.gemm_rows_batched(self.hn2, gu, act, T, 2 * pl.ff, self.W, 1, self.W, 0, pl.KO, 0, False, H.GR_GLU_SILU)

    def _norms(self, run: int) -> dict:
        """The norms that a layer run starts with, as the tail before it writes them."""
        if run >= len(self.runs):
            return {}
        w, li = self.w, self.runs[run][0]
        n = lambda name, out: (w[f"l{li}.{name}"], w[f"l{li}.{name}.b"], out)
        return dict(norm1=n("norm1", self.hn1), **({"norm2": n("norm2", self.hn2)} if self.plans[li].ff else {}))

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, T: int, meta: AttnMeta) -> None:
        """Runs every layer run over the T token rows; leaves the fp32 residual rows in self.x."""
        cfg, w, f, W = self.cfg, self.w, self.f32, self.W
        assert T <= self.max_tokens and meta.mode == H.MODE_CAUSAL and (meta.cu_q is not None or meta.q_per_seq > 0)
        H.lnorm_embed(input_ids, w["embed"], self.x, cfg.norm_eps, T, W, f, **self._norms(0))
        for run, (li, _) in enumerate(self.runs):
            pl = self.plans[li]
            cat = self.cat[(pl.KO, pl.nl + pl.nv + pl.ff)]
            self.launch_mixer(run, li, T, positions, meta, cat)
            if pl.ff:
                self.launch_mlp(li, T, cat)
            H.gemm_rows(cat, w[f"l{li}.out"], self.y, T, W, pl.KO, f)
            H.lnorm_tail(self.x, self.y, cfg.residual_mult, cfg.norm_eps, T, W, f, **self._norms(run + 1))
            if self.tap_residuals is not None:
                self.tap_residuals.append(self.x[:T].clone())

    def compute_logits(self, T: int, gather: torch.Tensor | None = None, rows: int | None = None) -> int:
        """Final norm (optionally of the `gather` rows only) and the LM head: fp32 logits in logits32[:n], their bf16 rounding (row
        stride Vp, padding -inf) in logits[:n] for the sampling kernels.  Returns n."""
        n = T if gather is None else rows
        assert n <= self.max_logit_rows
        w, e = self.w, "final.norm"
        H.lnorm_rows(self.x, w[e], w[e + ".b"], self.lastn, self.cfg.norm_eps, n, self.W, self.f32, gather=gather)
        H.gemm_rows(self.lastn, w["head"], self.logits32, n, self.V, self.W, self.f32)
        H.rows_f32_to_bf16(self.logits32, self.logits, n, self.V, self.V, self.Vp)
        return n
