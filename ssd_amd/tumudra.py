"""The Tumudra decoder on MI355X: layers that layer-norm a sublayer's OUTPUT only -- x <- x + ln1(mixer(x)), x <- x + ln2(ff(x)), the
sublayers read the fp32 residual row itself --; three kinds of mixer: grouped-query attention with biases, per-head q / k norms and rotary
positions over a paged cache (a layer may read another layer's pages instead of writing its own), retention (linear attention with a fixed
decay per head and rotary q / k), or two mixers side by side (windowed attention, and an xLSTM matrix memory with exponential gates), each
RMS-normed before they are averaged; dense relu^2 feed-forwards; embeddings times a constant.

Launches per layer (T token rows):
    attention      [q | k | v] GEMM + bias -> winattn_store_norm_rope (head norms, rope, cache pages) -> winattn_paged -> W_o GEMM + bias
                   (a layer with kv_from: q alone; the pages are the other layer's)
    retention      [q | k | v | g] GEMM -> rope_rows (q, k in place; k scaled) -> memory_scan (state slot, fixed decays) -> group_gate_norm
                   (per-head unit RMS, silu gate) -> W_o GEMM
    side by side   [lq | lk | lv | rq | rk | rv | rg | ri | rf] GEMM -> winattn_store_norm_rope -> winattn_paged (window) -> memory_scan
                   (state slot, gates; portions of many rows: memory_gates first) -> group_gate_norm (normaliser, per-head unit RMS,
                   sigmoid gate) -> [W_o left | W_o right] GEMMs, one launch when their inner sizes are equal
    lnorm_post_tail  (both sides' norms and their average ->) layer norm of the output, residual sum, the next sublayer's input rows
    feed-forward   W_up GEMM with relu^2 as epilogue -> W_down GEMM -> lnorm_post_tail
over pre-allocated buffers (nothing is allocated during a forward).  Same interface as ssd_amd.model.HipDecoder towards the ModelRunner.

Rotary layouts: the kernels pair entry i with i + dims / 2.  The side-by-side attention's checkpoint pairs 2i with 2i + 1: the output rows of
its q and k projections and their norms' weights are permuted at load (Rotary.to_halves), which leaves every score unchanged.

Arithmetic: residual rows and their sums, norms, rotation angles, scores, softmax, gates and decays, recurrent states and normalisers,
biases and every GEMM accumulator are fp32 in both modes.  dtype "bfloat16": weights, GEMM-input rows and the KV cache are bf16;
"float32": they are fp32 and products are FMA chains.
"""
from __future__ import annotations

import torch

from ssd_amd.hip import ops as H
from ssd_amd.model import AttnMeta
from ssd_amd.model_config import TumudraConfig, padded_channels
from ssd_amd.res32 import Res32Decoder

BF16 = torch.bfloat16
PAIR_SCALE = 0.5                # a side-by-side layer's result is half the sum of its normed sides
GATES_AHEAD = 16                # portions of more rows than this get their gates from a launch of their own


class _Columns:
    """Column offsets of one layer's fp32 projection row."""

    def __init__(self, m):
        att = m if m.kind == "attention" else (m.left if m.kind == "parallel" else None)
        lin = m if m.kind == "retention" else (m.right if m.kind == "parallel" else None)
        self.att, self.lin = att, lin
        self.nl = att.heads * att.vdim if att else 0             # output entries of the attention, of the linear mixer
        self.nv = lin.heads * lin.vdim if lin else 0
        o = 0
        if att:
            self.kv_heads = att.kv_heads if att.kv_from < 0 else 0       # key / value heads this layer projects and stores
            o = att.heads * att.dim + self.kv_heads * (att.dim + att.vdim)
        if lin:
            nk = lin.heads * lin.dim
            self.q, self.k, self.v, self.g = o, o + nk, o + 2 * nk, o + 2 * nk + self.nv
            o = self.g + self.nv
            if lin.kind == "memory":
                self.i, self.f = o, o + lin.heads
                o += 2 * lin.heads
            self.DP = padded_channels(lin.dim)
            self.columns = lin.vdim + (1 if lin.kind == "memory" else 0)         # state columns of a head: values (+ the normaliser)
        self.NP = o


class HipTumudra(Res32Decoder):
    def __init__(self, cfg: TumudraConfig, *, max_tokens: int, max_seqs: int, max_blocks: int, block_size: int, max_model_len: int,
                 device: torch.device, tp_rank: int = 0, tp_size: int = 1, tp_group=None, max_logit_rows: int | None = None,
                 max_split_tokens: int = 256, force_collectives: bool = False, taps=None, dtype: str = "bfloat16"):
        assert tp_size == 1 and taps is None, "Tumudra models are single-rank and have no activation taps"
        assert dtype in ("bfloat16", "float32")
        self.cfg, self.device = cfg, device
        self.f32 = dtype == "float32"
        self.elem = torch.float32 if self.f32 else BF16
        self.tp_rank, self.tp_size, self.tp_group = 0, 1, None
        self.use_coll, self.custom_ar, self.acts = False, None, None
        self.h = self.W = cfg.hidden_size
        self.V = cfg.vocab_size
        self.Vp = -(-self.V // 8) * 8
        self.block_size, self.max_blocks = block_size, max_blocks
        self.max_tokens = max_tokens
        self.max_logit_rows = max_logit_rows or max_tokens
        self.cols = [_Columns(l.mixer) for l in cfg.layers]
        self.state_slots = max_seqs if cfg.recurrent else 0      # one per live sequence; the block manager hands them out
        self.w: dict[str, torch.Tensor] = {}
        self.kv: list = []
        self.state: list = []
        self.scalar_attention = False                 # tests / probes: the scalar form of the attention also where the MFMA form fits
        self.tap_residuals: list | None = None         # tests: receives a copy of the residual rows after every layer (eager only)

        def z(*shape, dtype=torch.float32):
            return torch.zeros(*shape, dtype=dtype, device=device)

        T, W, el, cols = max_tokens, self.W, self.elem, self.cols
        self.x = z(T, W)
        self.hn = z(T, W, dtype=el)
        self.y = z(2, T, W)                            # mixer / feed-forward output rows; [1]: the right side's
        self.proj = z(T * max(c.NP for c in cols))
        self.cat = z(T * max(c.nl + c.nv for c in cols), dtype=el)        # output-GEMM input rows [attention | linear]
        att = [c.att for c in cols if c.att]
        lin = [c for c in cols if c.lin]
        if att:
            self.q = z(T * max(a.heads * a.dim for a in att), dtype=el)
            # partial rows of decode batches whose keys are cut over workgroups (winattn_paged)
            self.att_ws = z(1024 * 16 * (max(a.vdim for a in att) + 2)) if not self.f32 else None
        if lin:
            self.o = z(T * max(c.nv for c in lin))
            self.ones = torch.ones(max(c.nv for c in lin), dtype=el, device=device)
            Hm = max(c.lin.heads for c in lin)
            self.den, self.gates = z(T * Hm), z(T * Hm * 4)
        ffs = [l.mlp.ff for l in cfg.layers if l.mlp is not None]
        if ffs:
            self.act = z(T * max(ffs), dtype=el)
        R = self.max_logit_rows
        self.lastn = z(R, W, dtype=el)
        self.logits32 = z(R, self.V)
        self.logits = z(R, self.Vp, dtype=BF16)

    # ---------------------------------------------------------------------------------------------
    def load_weights(self, weight_iter) -> None:
        """Consumes (name, tensor) pairs under the checkpoint's names.  Matrices that read the same rows are stacked (_Columns), their
        biases alike; the two output matrices of a side-by-side layer become one [2][W][K] stack when their inner sizes are equal;
        interleaved rotary layouts are permuted into halves; biases and decays are kept as fp32."""
        raw = {n: t.to(self.device) for n, t in weight_iter}
        cv = lambda t: t.to(self.elem).contiguous()
        f32 = lambda t: t.float().reshape(-1).contiguous()
        dev_f32 = lambda vals: torch.tensor(vals, dtype=torch.float64).to(torch.float32).to(self.device)
        w = self.w = {}

        def attention(p, a):
            """The projection's rows and biases; stores the norms and frequencies."""
            order = torch.tensor(a.rope.to_halves(a.dim), device=self.device)
            heads = lambda t, n: t.view(n, a.dim, -1)[:, order].reshape(n * a.dim, -1)
            rows, bias = [heads(raw[p + "q"], a.heads)], [heads(raw[p + "q.b"], a.heads)] if a.bias else []
            w[p + "q.norm"] = cv(raw[p + "q.norm"][order])
            if a.kv_from < 0:
                rows += [heads(raw[p + "k"], a.kv_heads), raw[p + "v"]]
                bias += [heads(raw[p + "k.b"], a.kv_heads), raw[p + "v.b"].view(-1, 1)] if a.bias else []
                w[p + "k.norm"] = cv(raw[p + "k.norm"][order])
            w[p + "freqs"] = dev_f32(a.rope.frequencies() or [0.0])
            return rows, bias

        w["embed"], w["head"], w["final.norm"] = cv(raw["embed"]), cv(raw["head"]), cv(raw["final.norm"])
        for i, (lc, c) in enumerate(zip(self.cfg.layers, self.cols)):
            p, m = f"l{i}.mix.", lc.mixer
            w[f"l{i}.norm1"] = cv(raw[f"l{i}.norm1"])
            rows, bias = [], []
            if c.att:
                rows, bias = attention(p + "left." if c.lin else p, c.att)
            if c.lin:
                r = p + "right." if c.att else p
                rows += [raw[r + n] for n in "qkvg"]
                if m.kind == "retention":
                    assert m.rope.layout == "halves"
                    w[p + "decay"], w[p + "freqs"] = dev_f32(m.decay), dev_f32(m.rope.frequencies() or [0.0])
                else:
                    rows += [raw[r + "i"], raw[r + "f"]]
                    w[r + "i.b"], w[r + "f.b"] = f32(raw[r + "i.b"]), f32(raw[r + "f.b"])
                    w[r + "norm"] = cv(raw[r + "norm"])
            w[p + "in"] = cv(torch.cat(rows, dim=0))
            assert w[p + "in"].shape[0] == c.NP
            if m.kind == "parallel":
                w[p + "left.out"], w[p + "right.out"] = cv(raw[p + "left.out"]), cv(raw[p + "right.out"])
                outs = [raw[p + "left.o"], raw[p + "right.o"]]
                if c.nl == c.nv:
                    w[p + "o"] = cv(torch.stack(outs))
                else:
                    w[p + "left.o"], w[p + "right.o"] = cv(outs[0]), cv(outs[1])
            else:
                w[p + "o"] = cv(raw[p + "o"])
                if bias:
                    w[p + "in.b"], w[p + "o.b"] = f32(torch.cat(bias, dim=0)), f32(raw[p + "o.b"])
            if lc.mlp is not None:
                q = f"l{i}."
                w[q + "norm2"], w[q + "mlp.up"], w[q + "mlp.down"] = cv(raw[q + "norm2"]), cv(raw[q + "mlp.up"]), cv(raw[q + "mlp.down"])
        torch.cuda.synchronize(self.device)

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.w.values())

    def active_weight_bytes(self, T: int = 1) -> int:
        """HBM bytes of weights one forward of T tokens must stream at least: everything once, of the embedding one row per token."""
        return self.weight_bytes() - self.w["embed"].numel() * self.w["embed"].element_size()

    def kv_block_bytes(self) -> int:
        es = 4 if self.f32 else 2
        n = sum(c.kv_heads * (c.att.dim + c.att.vdim) * self.block_size * es for c in self.cols if c.att)
        return max(n, 1)

    def state_bytes(self) -> int:
        """Bytes of recurrent state one live sequence holds (all layers)."""
        return sum(c.lin.heads * c.columns * (c.DP + (1 if c.lin.kind == "memory" else 0)) * 4 for c in self.cols if c.lin)

    def alloc_kv(self, num_blocks: int) -> None:
        """Per layer: attention -> K pages [blocks][G][block][dim] and V pages transposed [blocks][G][vdim][block] (a layer with kv_from:
        the same tensors as that layer); retention / matrix memory -> state [slots][H][columns][key channels, padded] fp32 (transposed; a
        matrix memory's last column is its normaliser) and, for the latter, the running maxima [slots][H][columns].  A slot is not
        cleared when it is handed out: a forward whose rows start at position 0 starts from zero by itself."""
        self.num_blocks = num_blocks
        self.kv, self.state = [], []
        dev, bs, S = self.device, self.block_size, self.state_slots
        for c in self.cols:
            a, m = c.att, c.lin
            if a is None:
                self.kv.append(None)
            elif a.kv_from >= 0:
                self.kv.append(self.kv[a.kv_from])
            else:
                self.kv.append((torch.zeros(num_blocks, a.kv_heads, bs, a.dim, dtype=self.elem, device=dev),
                                torch.zeros(num_blocks, a.kv_heads, a.vdim, bs, dtype=self.elem, device=dev)))
            if m is None:
                self.state.append(None)
            else:
                self.state.append((torch.zeros(S, m.heads, c.columns, c.DP, dtype=torch.float32, device=dev),
                                   torch.zeros(S, m.heads, c.columns, dtype=torch.float32, device=dev) if m.kind == "memory" else None))

    # ---------------------------------------------------------------------------------------------
    def _attention(self, li: int, p: str, T: int, positions, meta: AttnMeta, seqs: dict, ldo: int) -> None:
        """Projection rows -> the attention's columns of the output-GEMM input rows."""
        w, f, c = self.w, self.f32, self.cols[li]
        a, (kc, vc) = c.att, self.kv[li]
        own = c.kv_heads > 0
        H.winattn_store_norm_rope(self.proj, c.NP, w[p + "q.norm"], w[p + "k.norm"] if own else None, self.cfg.norm_eps, positions, w[p + "freqs"],
                                  a.rope.dims, meta.slot_mapping, self.q, kc if own else None, vc if own else None, T, a.heads, c.kv_heads,
                                  a.dim, a.vdim, self.block_size, f)
        H.winattn_paged(self.q, kc, vc, None, None, meta.block_tables, self.max_blocks, positions, meta.B, T, a.heads, a.kv_heads, a.dim, a.vdim,
                        self.block_size, a.window, a.scale, 0.0, self.cat, f, max_q=0 if self.scalar_attention else meta.max_q, ldo=ldo,
                        workspace=self.att_ws, **seqs)

    def launch_mixer(self, li: int, T: int, positions, meta: AttnMeta) -> dict:
        """hn (the residual rows in the element type) -> y (fp32 mixer output rows); returns the keyword arguments that hand them to
        lnorm_post_tail."""
        cfg, w, f, W = self.cfg, self.w, self.f32, self.W
        m, p, c = cfg.layers[li].mixer, f"l{li}.mix.", self.cols[li]
        seqs = dict(cu_q=meta.cu_q) if meta.cu_q is not None else dict(q_per_seq=meta.q_per_seq)
        y, proj, NP, ld = self.y[0], self.proj, c.NP, c.nl + c.nv
        if m.kind == "attention":
            H.gemm_rows_bias(self.hn, w[p + "in"], proj, T, NP, W, w[p + "in.b"], f)
            self._attention(li, p, T, positions, meta, seqs, ld)
            H.gemm_rows_bias(self.cat, w[p + "o"], y, T, W, c.nl, w[p + "o.b"], f)
            return dict(y_rows=y)
        assert meta.state_slots is not None, "a model with recurrent layers needs the sequences' state slots"
        S, running = self.state[li]
        H.gemm_rows(self.hn, w[p + "in"], proj, T, NP, W, f)
        n, D, Dv = c.lin.heads, c.lin.dim, c.lin.vdim
        scan = (proj, NP, c.q, c.k, c.v, positions, meta.state_slots, S, self.o, meta.B, n, D, Dv, c.DP)
        gate = proj[c.g:]
        if m.kind == "retention":
            H.rope_rows(proj, NP, positions, w[p + "freqs"], m.rope.dims, n, D, T, c.q, 1.0, c.k, float(D) ** -0.5)
            H.memory_scan(*scan, decay=w[p + "decay"], **seqs)
            H.group_gate_norm(self.o, gate, NP, self.ones, cfg.norm_eps, self.cat, T, c.nv, n, False, f)
            H.gemm_rows(self.cat, w[p + "o"], y, T, W, c.nv, f)
            return dict(y_rows=y)
        self._attention(li, p + "left.", T, positions, meta, seqs, ld)
        r = p + "right."
        gating = dict(i_off=c.i, f_off=c.f, bias_i=w[r + "i.b"], bias_f=w[r + "f.b"], cap=m.right.gate_cap, m_state=running)
        ahead = meta.max_q > GATES_AHEAD
        if ahead:
            H.memory_gates(proj, NP, positions=positions, state_slots=meta.state_slots, gates=self.gates, B=meta.B, H=n, Dv=Dv, **gating, **seqs)
        H.memory_scan(*scan, q_scale=float(D) ** -0.5, gates=self.gates if ahead else None, den=self.den, **gating, **seqs)
        H.group_gate_norm(self.o, gate, NP, w[r + "norm"], cfg.norm_eps, self.cat[c.nl:], T, c.nv, n, False, f, gate_act=H.GATE_SIGMOID, ldo=ld,
                          den=self.den)
        y2 = self.y[1]
        if c.nl == c.nv:
            H.gemm_rows_batched(self.cat, w[p + "o"], self.y, T, W, c.nl, 2, ld, c.nl, W, self.max_tokens * W, f)
        else:
            H.gemm_rows_batched(self.cat, w[p + "left.o"], y, T, W, c.nl, 1, ld, 0, W, 0, f)
            H.gemm_rows_batched(self.cat[c.nl:], w[p + "right.o"], y2, T, W, c.nv, 1, ld, 0, W, 0, f)
        return dict(y_rows=y, y2_rows=y2, w1=w[p + "left.out"], w2=w[p + "right.out"], pair_scale=PAIR_SCALE)

    def launch_mlp(self, li: int, T: int) -> dict:
        """hn -> the feed-forward's rows, as launch_mixer returns them."""
        w, f, ff, p = self.w, self.f32, self.cfg.layers[li].mlp.ff, f"l{li}.mlp."
        H.gemm_rows(self.hn, w[p + "up"], self.act, T, ff, self.W, f, H.GR_RELU2)
        H.gemm_rows(self.act, w[p + "down"], self.y[0], T, self.W, ff, f)
        return dict(y_rows=self.y[0])

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, T: int, meta: AttnMeta) -> None:
        """Runs every layer over the T token rows; leaves the fp32 residual rows in self.x."""
        cfg, w, f, W = self.cfg, self.w, self.f32, self.W
        eps = cfg.norm_eps
        assert T <= self.max_tokens and meta.mode == H.MODE_CAUSAL and (meta.cu_q is not None or meta.q_per_seq > 0)
        H.embed_hist(input_ids, w["embed"], self.x, T, W, f, rows_out=self.hn, scale=cfg.embed_scale)
        for li, lc in enumerate(cfg.layers):
            H.lnorm_post_tail(self.x, weight=w[f"l{li}.norm1"], eps=eps, T=T, W=W, f32=f, next_out=self.hn,
                              **self.launch_mixer(li, T, positions, meta))
            if lc.mlp is not None:
                H.lnorm_post_tail(self.x, weight=w[f"l{li}.norm2"], eps=eps, T=T, W=W, f32=f, next_out=self.hn, **self.launch_mlp(li, T))
            if self.tap_residuals is not None:
                self.tap_residuals.append(self.x[:T].clone())

    def compute_logits(self, T: int, gather: torch.Tensor | None = None, rows: int | None = None) -> int:
        """Final norm (optionally of the `gather` rows only) and the LM head: fp32 logits in logits32[:n], their bf16 rounding (row
        stride Vp, padding -inf) in logits[:n] for the sampling kernels.  Returns n."""
        n = T if gather is None else rows
        assert n <= self.max_logit_rows
        H.lnorm_rows(self.x, self.w["final.norm"], None, self.lastn, self.cfg.norm_eps, n, self.W, self.f32, gather=gather)
        H.gemm_rows(self.lastn, self.w["head"], self.logits32, n, self.V, self.W, self.f32)
        H.rows_f32_to_bf16(self.logits32, self.logits, n, self.V, self.V, self.Vp)
        return n
