"""Whole-sequence float64 statement of the Dusupel decoder: one function per mechanism, no cache, no state slots, no batching -- a
sequence goes in as a list of token ids and every position's logits come out.  Shares nothing with ssd_amd/ (it reads the
configuration as the plain dict of config.json and the weights as a name -> tensor dict under the checkpoint's names).

Notation: W = width, E = norm eps, M = residual_mult, T = tokens of the sequence, positions 0 .. T - 1,
ln_n(x) = (x - mean x) / sqrt(var x + E) * w_n + b_n (var = mean of squared deviations), rms(v) = v / sqrt(mean v^2 + E),
unit(v) = v / sqrt(sum v^2 + 1e-6), sig = logistic sigmoid, silu(z) = z sig(z).

    layer:   x <- x + M (mixer(ln_1(x)) + ff(ln_2(x)))          both read the SAME x; a layer may have no ff
    ff(h)  = W_down (silu(W_gate h) * W_up h)
    output:  logits = head ln_final(x);   x_0 = embed[token]
    loop {start, stop, times}: layers start .. stop - 1 run `times` passes, each with a memory of its own (nothing between passes)
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def lin(w, x):
    return x @ w.to(F64).T


def silu(z):
    return z * torch.sigmoid(z)


def layer_norm(x, w, b, eps):
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * w.to(F64) + b.to(F64)


def rms(v, eps):
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps)


def unit(v):
    return v / torch.sqrt((v * v).sum(dim=-1, keepdim=True) + 1e-6)


def short_conv(u, w):
    """u [T, C], w [C, taps]: y_t[c] = sum_j w[c, j] u_(t - taps + 1 + j)[c], u = 0 before the sequence."""
    T, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F64), u])
    return sum(pad[j:j + T] * w[:, j].to(F64) for j in range(taps))


def turn(x, pos, n, base):
    """x [T, heads, D]: of the first n entries of a head, entry i (a) and i + n / 2 (b) become (a cos t - b sin t, b cos t + a sin t),
    t = pos * base^(-2i/n)."""
    if n == 0:
        return x
    i = torch.arange(n // 2, dtype=F64)
    t = pos.to(F64).view(-1, 1, 1) * (base ** (-2.0 * i / n)).view(1, 1, -1)
    c, s = torch.cos(t), torch.sin(t)
    a, b = x[..., :n // 2], x[..., n // 2:n]
    return torch.cat([a * c - b * s, b * c + a * s, x[..., n:]], dim=-1)


# ------------------------------------------------------------------------------------------------------------------
def visible(T, mask):
    """[T, T] bool: row i sees key j <= i if it lies fewer than `size` tokens back or is one of the first `keep_first` tokens."""
    d = torch.arange(T).view(T, 1) - torch.arange(T).view(1, T)
    size = (mask or {}).get("size")
    if not size:
        return d >= 0
    return (d >= 0) & ((d < size) | (torch.arange(T).view(1, T) < (mask.get("keep_first") or 0)))


def attention(h, w, p, m):
    """Grouped-query attention: short convolutions on q, k and v, rotary q and k, windowed softmax that always keeps the first tokens;
    returns the concatenated heads times sig(W_g h)  (before the output projection)."""
    T = h.shape[0]
    H, G, D, Dv, r = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["rot"]
    pos = torch.arange(T)
    q, k, v = (short_conv(lin(w[p + n], h), w[p + n + ".conv"]) for n in "qkv")
    q, k = turn(q.view(T, H, D), pos, r["dims"], r["base"]), turn(k.view(T, G, D), pos, r["dims"], r["base"])
    v = v.view(T, G, Dv)
    see = visible(T, m.get("mask"))
    out = torch.zeros(T, H, Dv, dtype=F64)
    for hh in range(H):
        g = hh // (H // G)
        s = (q[:, hh] @ k[:, g].T) * m["scale"]
        out[:, hh] = torch.softmax(torch.where(see, s, torch.full_like(s, -math.inf)), dim=-1) @ v[:, g]
    return out.reshape(T, H * Dv) * torch.sigmoid(lin(w[p + "g"], h))


def delta_inputs(h, w, p, m):
    """Per head h (q / k head h // (H / G)): unit q times dim^-0.5, unit k, v, step beta = sig(W_b h)."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(lin(w[p + n], h), w[p + n + ".conv"])) for n in "qkv")
    q, k = unit(q.view(T, G, D)) * D ** -0.5, unit(k.view(T, G, D))
    rep = lambda t: t.repeat_interleave(H // G, dim=1)
    return rep(q), rep(k), v.view(T, H, Dv), torch.sigmoid(lin(w[p + "b"], h))


def delta_rule(q, k, v, beta, decay):
    """S <- decay_t S (rows of S = key channels; decay [T, H, D] or [T, H, 1]);  u = beta_t (v_t - S^T k_t);  S <- S + k_t u^T;
    o_t = S^T q_t, from S = 0."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    o = torch.zeros_like(v)
    for t in range(T):
        S = decay[t].unsqueeze(-1) * S
        u = beta[t].unsqueeze(-1) * (v[t] - (S * k[t].unsqueeze(-1)).sum(1))
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        o[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return o


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def head_delta(h, w, p, m, eps):
    """Gated delta rule with ONE decay per head; heads normed by their root mean square, times a weight shared by the heads, times
    silu(W_g h)  (before the output projection)."""
    T, H = h.shape[0], m["heads"]
    q, k, v, beta = delta_inputs(h, w, p, m)
    decay = torch.exp(-torch.exp(w[p + "A_log"].to(F64)) * softplus(lin(w[p + "a"], h) + w[p + "dt_bias"].to(F64)))
    o = rms(delta_rule(q, k, v, beta, decay.unsqueeze(-1)), eps) * w[p + "norm"].to(F64)
    return o.reshape(T, -1) * silu(lin(w[p + "g"], h))


def channel_delta(h, w, p, m, eps):
    """Gated delta rule with one decay per head and key channel from a low-rank projection; the gate is sig of another one."""
    T, H, D = h.shape[0], m["heads"], m["dim"]
    q, k, v, beta = delta_inputs(h, w, p, m)
    z = (lin(w[p + "a2"], lin(w[p + "a1"], h)) + w[p + "dt_bias"].to(F64)).view(T, H, D)
    decay = torch.exp(-torch.exp(w[p + "A_log"].to(F64)).view(1, H, 1) * softplus(z))
    o = rms(delta_rule(q, k, v, beta, decay), eps) * w[p + "norm"].to(F64)
    return o.reshape(T, -1) * torch.sigmoid(lin(w[p + "g2"], lin(w[p + "g1"], h)))


def mixer(kind, h, w, p, m, eps):
    if kind == "parallel":
        left = lin(w[p + "left.o"], attention(h, w, p + "left.", m["left"]))
        right = lin(w[p + "right.o"], head_delta(h, w, p + "right.", m["right"], eps))
        return m["left_scale"] * left + m["right_scale"] * right
    assert kind in ("channel_delta", "channel_delta_2"), kind
    return lin(w[p + "o"], channel_delta(h, w, p, m, eps))


def dense_ff(h, w, p):
    return lin(w[p + "down"], silu(lin(w[p + "gate"], h)) * lin(w[p + "up"], h))


def layer_order(cfg):
    lp = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    a, b, n = lp["start"], lp["stop"], lp["times"]
    L = len(cfg["layers"])
    return list(range(L)) if b <= a else list(range(a)) + list(range(a, b)) * n + list(range(b, L))


def forward(cfg: dict, w: dict, tokens, residuals: list | None = None, round_input=None) -> torch.Tensor:
    """Logits [T, vocab] of every position.  residuals: receives x after every layer run.  round_input: applied to every sublayer's
    input (what rounding of the inputs alone does to the statement)."""
    eps = cfg["norm"]["eps"]
    rd = round_input or (lambda t: t)
    ln = lambda v, n: rd(layer_norm(v, w[n], w[n + ".b"], eps))
    x = w["embed"].to(F64)[torch.tensor(tokens)]
    for i in layer_order(cfg):
        p, lc = f"l{i}.", cfg["layers"][i]
        y = mixer(lc["type"], ln(x, p + "norm1"), w, p + "mix.", lc["mixer"], eps)
        if lc.get("mlp") is not None:
            y = y + dense_ff(ln(x, p + "norm2"), w, p + "mlp.")
        x = x + cfg["residual_mult"] * y
        if residuals is not None:
            residuals.append(x.clone())
    return lin(w["head"], ln(x, "final.norm"))


# ------------------------------------------------------------------------------------------------------------------
# small configurations and random weights for the tests
def dense_mlp(ff=24):
    return {"kind": "dense", "ff": ff}


def delta_sizes(heads=2, kv_heads=None, dim=8, vdim=8, conv=3):
    return {"heads": heads, "kv_heads": heads if kv_heads is None else kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def attention_sizes(heads=4, kv_heads=2, dim=8, vdim=8, conv=3, scale=None, size=5, keep_first=2, rot_dims=None, base=10000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": dim ** -0.5 if scale is None else scale,
            "mask": {"size": size, "keep_first": keep_first}, "rot": {"dims": dim if rot_dims is None else rot_dims, "base": base}}


def parallel_layer(left=None, right=None, left_scale=0.7, right_scale=1.3, mlp=None):
    return {"type": "parallel", "mixer": {"left": left or attention_sizes(), "right": right or delta_sizes(), "left_scale": left_scale,
                                          "right_scale": right_scale}, "mlp": mlp}


def delta_layer(kind="channel_delta", mlp=None, **sizes):
    return {"type": kind, "mixer": delta_sizes(**sizes), "mlp": mlp}


def make_config(layers, vocab=64, width=32, eps=1e-5, residual_mult=0.6, loop=None):
    return {"architecture": "Dusupel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": residual_mult,
            "layers": layers, "loop": loop}


def tensor_shapes(cfg: dict, ranks=(6, 5)) -> list:
    """ranks: inner sizes of the low-rank decay and gate projections (a number, or a function of the layer index giving the pair)."""
    W = cfg["width"]
    norm = lambda n: [(n, (W,)), (n + ".b", (W,))]
    out = [("embed", (cfg["vocab"], W))]

    def qkv(p, nq, nk, nv, taps):
        return [t for n, c in (("q", nq), ("k", nk), ("v", nv)) for t in ((p + n, (c, W)), (p + n + ".conv", (c, taps)))]

    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        out += norm(p + "norm1") + (norm(p + "norm2") if lc.get("mlp") is not None else [])
        d, dp = (m["right"], p + "mix.right.") if lc["type"] == "parallel" else (m, p + "mix.")
        if lc["type"] == "parallel":
            a, ap = m["left"], p + "mix.left."
            nv = a["heads"] * a["vdim"]
            out += qkv(ap, a["heads"] * a["dim"], a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"], a["conv"])
            out += [(ap + "g", (nv, W)), (ap + "o", (W, nv))]
        H, nk, nv = d["heads"], d["kv_heads"] * d["dim"], d["heads"] * d["vdim"]
        out += qkv(dp, nk, nk, nv, d["conv"]) + [(dp + "b", (H, W)), (dp + "A_log", (H,)), (dp + "norm", (d["vdim"],)), (dp + "o", (W, nv))]
        if lc["type"] == "parallel":
            out += [(dp + "a", (H, W)), (dp + "dt_bias", (H,)), (dp + "g", (nv, W))]
        else:
            ra, rg = ranks(i) if callable(ranks) else ranks
            out += [(dp + "a1", (ra, W)), (dp + "a2", (H * d["dim"], ra)), (dp + "dt_bias", (H * d["dim"],)), (dp + "g1", (rg, W)),
                    (dp + "g2", (nv, rg))]
        if lc.get("mlp") is not None:
            ff = lc["mlp"]["ff"]
            out += [(p + "mlp.gate", (ff, W)), (p + "mlp.up", (ff, W)), (p + "mlp.down", (W, ff))]
    return out + norm("final.norm") + [("head", (cfg["vocab"], W))]


def random_model(cfg: dict, seed: int = 0, ranks=(6, 5)) -> dict:
    """bf16 weights: matrices ~ N(0, 1 / fan_in) (attention q / k larger so that single keys carry the output), norms around one,
    their biases around zero, decays spread so that some heads and channels remember hundreds of tokens and some only a few."""
    g = torch.Generator().manual_seed(seed)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float32)
    w = {}
    for name, shape in tensor_shapes(cfg, ranks):
        if name.endswith((".norm1", ".norm2", "norm")):
            t = 1.0 + 0.2 * rn(*shape)
        elif name.endswith((".norm1.b", ".norm2.b", "norm.b")):
            t = 0.3 * rn(*shape)
        elif name.endswith(".A_log"):
            t = 0.5 * rn(*shape)
        elif name.endswith(".dt_bias"):
            t = -3.0 + 2.0 * rn(*shape)
        elif name.endswith(".conv"):
            t = 0.5 * rn(*shape)
            t[:, -1] += 1.0
        elif name == "embed":
            t = rn(*shape)
        else:
            boost = 2.0 if name.endswith((".left.q", ".left.k")) else 1.0
            t = boost * rn(*shape) / math.sqrt(shape[-1])
        w[name] = t.to(torch.bfloat16)
    return w
