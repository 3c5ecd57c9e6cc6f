"""Whole-sequence float64 statement of the Tumudra decoder: one function per mechanism, no cache, no state slots, no batching -- a
sequence goes in as a list of token ids and every position's logits come out.  Shares nothing with ssd_amd/ (it reads the
configuration as the plain dict of config.json and the weights as a name -> tensor dict under the checkpoint's names).

Notation: W = width, E = norm eps, T = tokens of the sequence, positions 0 .. T - 1, ln_n(y) = (y - mean y) / sqrt(var y + E) * w_n
(var = mean of squared deviations, no bias), rms(y) = y / sqrt(mean y^2 + E), sig = logistic sigmoid, silu(z) = z sig(z).

    x_0    = embedding.scale * embed[token]
    layer:   x <- x + ln_1(mixer(x)),  then  x <- x + ln_2(ff(x))  unless the layer has no ff        (sublayers read x as it is)
    ff(x)  = W_down relu(W_up x)^2
    output:  logits = head ln_final(x)
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def lin(w, n, x):
    y = x @ w[n].to(F64).T
    return y + w[n + ".b"].to(F64) if n + ".b" in w else y


def layer_norm(y, w, eps):
    d = y - y.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * w.to(F64)


def rms(y, eps):
    return y / torch.sqrt((y * y).mean(dim=-1, keepdim=True) + eps)


# ------------------------------------------------------------------------------------------------------------------
def angular_frequencies(rot):
    """base^(-2i/n) for the n / 2 pairs.  scaling {factor, low, high, original}: a pair that turns more than `high` times over `original`
    positions keeps its frequency, one that turns fewer than `low` times is slowed down by `factor`, those between are blended
    linearly in the number of turns."""
    n = rot["dims"]
    f = rot["base"] ** (-2.0 * torch.arange(n // 2, dtype=F64) / n)
    sc = rot.get("scaling")
    if not sc:
        return f
    turns = sc["original"] * f / (2.0 * math.pi)
    keep = (turns - sc["low"]) / (sc["high"] - sc["low"])
    blend = (1.0 - keep) * f / sc["factor"] + keep * f
    return torch.where(turns > sc["high"], f, torch.where(turns < sc["low"], f / sc["factor"], blend))


def turn(x, pos, rot, interleaved):
    """x [T, heads, D]: pairs (a, b) of the first n entries become (a cos t - b sin t, b cos t + a sin t), t = position * frequency.
    Pairs are entries (i, i + n / 2), or (2i, 2i + 1) when interleaved."""
    n = rot["dims"]
    t = pos.to(F64).view(-1, 1, 1) * angular_frequencies(rot).view(1, 1, -1)
    c, s = torch.cos(t), torch.sin(t)
    a, b = (x[..., 0:n:2], x[..., 1:n:2]) if interleaved else (x[..., :n // 2], x[..., n // 2:n])
    a2, b2 = a * c - b * s, b * c + a * s
    head = torch.stack([a2, b2], dim=-1).flatten(-2) if interleaved else torch.cat([a2, b2], dim=-1)
    return torch.cat([head, x[..., n:]], dim=-1)


def visible(T, size):
    """[T, T] bool: row i sees the keys j <= i, of these only the nearest `size` (itself included) when size is given."""
    d = torch.arange(T).view(T, 1) - torch.arange(T).view(1, T)
    return (d >= 0) & (d < size) if size else d >= 0


def softmax_attention(q, k, v, scale, see):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]; query head h reads key / value head h // (H / G); concatenated heads [T, H Dv]."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // (H // G)].T) * scale
        out.append(torch.softmax(torch.where(see, s, torch.full_like(s, -math.inf)), dim=-1) @ v[:, h // (H // G)])
    return torch.cat(out, dim=-1)


def attention_keys_values(x, w, p, m, eps, interleaved):
    T, G = x.shape[0], m["kv_heads"]
    k = rms(lin(w, p + "k", x).view(T, G, m["dim"]), eps) * w[p + "k.norm"].to(F64)
    return turn(k, torch.arange(T), m["rot"], interleaved), lin(w, p + "v", x).view(T, G, m["vdim"])


def attention_heads(x, kv, w, p, m, eps, interleaved):
    T = x.shape[0]
    q = rms(lin(w, p + "q", x).view(T, m["heads"], m["dim"]), eps) * w[p + "q.norm"].to(F64)
    q = turn(q, torch.arange(T), m["rot"], interleaved)
    return softmax_attention(q, *kv, m["scale"], visible(T, (m.get("mask") or {}).get("size")))


# ------------------------------------------------------------------------------------------------------------------
def log_sigmoid(z):
    return torch.minimum(z, torch.zeros_like(z)) - torch.log1p(torch.exp(-z.abs()))


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def matrix_memory(q, k, v, i, f):
    """Per head, from S = 0, n = 0, M = 0 with log input gate i and log forget gate f [T, H]:
    M' = max(f + M, i);  S <- e^(f + M - M') S + e^(i - M') k v^T;  n likewise with k;  o = S^T q / (max(|<n, q>|, e^(-M')) + 1e-6)."""
    T, H, D = q.shape
    S, n, M = torch.zeros(H, D, v.shape[-1], dtype=F64), torch.zeros(H, D, dtype=F64), torch.zeros(H, dtype=F64)
    o = torch.zeros_like(v)
    for t in range(T):
        top = torch.maximum(f[t] + M, i[t])
        a, b = torch.exp(f[t] + M - top).view(H, 1), torch.exp(i[t] - top).view(H, 1)
        S = a.unsqueeze(-1) * S + (b * k[t]).unsqueeze(-1) * v[t].unsqueeze(1)
        n = a * n + b * k[t]
        M = top
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-M)) + 1e-6
        o[t] = (S * q[t].unsqueeze(-1)).sum(1) / den.view(H, 1)
    return o


def memory_heads(x, w, p, m, eps):
    """Unit-rms heads times a weight over all of them, times sig(W_g x)  (before the output projection)."""
    T, H, D, Dv = x.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = lin(w, p + "q", x).view(T, H, D) * D ** -0.5, lin(w, p + "k", x).view(T, H, D)
    i = soft_cap(lin(w, p + "i", x), m["gate_cap"])
    f = log_sigmoid(soft_cap(lin(w, p + "f", x), m["gate_cap"]))
    o = rms(matrix_memory(q, k, lin(w, p + "v", x).view(T, H, Dv), i, f), eps)
    return o.reshape(T, H * Dv) * w[p + "norm"].to(F64) * torch.sigmoid(lin(w, p + "g", x))


def retention(q, k, v, decay):
    """S <- decay S + k v^T, o = S^T q, from S = 0."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    o = torch.zeros_like(v)
    dc = torch.tensor(decay, dtype=F64).view(H, 1, 1)
    for t in range(T):
        S = dc * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        o[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return o


def retention_heads(x, w, p, m, eps):
    T, H, D, Dv = x.shape[0], m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q = turn(lin(w, p + "q", x).view(T, H, D), pos, m["rot"], False)
    k = turn(lin(w, p + "k", x).view(T, H, D), pos, m["rot"], False) * D ** -0.5
    g = lin(w, p + "g", x)
    o = rms(retention(q, k, lin(w, p + "v", x).view(T, H, Dv), m["decay"]), eps)
    return o.reshape(T, H * Dv) * (g * torch.sigmoid(g))


# ------------------------------------------------------------------------------------------------------------------
def mixer(kind, x, w, p, m, eps, i, keys, round_input):
    """keys: layer -> (keys, values), filled here; a layer with 'kv_from' reads another layer's.  round_input: see forward."""
    if kind == "parallel":
        lp, rp = p + "left.", p + "right."
        kv = attention_keys_values(x, w, lp, m["left"], eps, True)
        left = lin(w, lp + "o", round_input(attention_heads(x, kv, w, lp, m["left"], eps, True)))
        right = lin(w, rp + "o", round_input(memory_heads(x, w, rp, m["right"], eps)))
        return 0.5 * (rms(left, eps) * w[lp + "out"].to(F64) + rms(right, eps) * w[rp + "out"].to(F64))
    if kind == "attention":
        keys[i] = keys[m["kv_from"]] if m.get("kv_from") is not None else attention_keys_values(x, w, p, m, eps, False)
        return lin(w, p + "o", round_input(attention_heads(x, keys[i], w, p, m, eps, False)))
    assert kind == "retention", kind
    return lin(w, p + "o", round_input(retention_heads(x, w, p, m, eps)))


def dense_ff(x, w, p, round_input):
    z = torch.clamp(lin(w, p + "up", x), min=0.0)
    return lin(w, p + "down", round_input(z * z))


def forward(cfg: dict, w: dict, tokens, residuals: list | None = None, round_input=None) -> torch.Tensor:
    """Logits [T, vocab] of every position.  residuals: receives x after every layer.  round_input: applied to the input of every
    projection (what rounding of those inputs alone does to the statement)."""
    eps = cfg["norm"]["eps"]
    rd = round_input or (lambda t: t)
    x = w["embed"].to(F64)[torch.tensor(tokens)] * cfg["embedding"]["scale"]
    keys: dict = {}
    for i, lc in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + layer_norm(mixer(lc["type"], rd(x), w, p + "mix.", lc["mixer"], eps, i, keys, rd), w[p + "norm1"], eps)
        if lc.get("mlp") is not None:
            x = x + layer_norm(dense_ff(rd(x), w, p + "mlp.", rd), w[p + "norm2"], eps)
        if residuals is not None:
            residuals.append(x.clone())
    return lin(w, "head", rd(layer_norm(x, w["final.norm"], eps)))


# ------------------------------------------------------------------------------------------------------------------
# small configurations and random weights for the tests
def dense_mlp(ff=24):
    return {"kind": "dense", "ff": ff}


def rotation(dims=8, base=10000.0, scaling=None):
    return {"base": base, "dims": dims, **({"scaling": scaling} if scaling else {})}


def attention_sizes(heads=4, kv_heads=2, dim=8, vdim=8, scale=None, rot=None, size=None, kv_from=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
            "rot": rot or rotation(dim), **({"mask": {"size": size}} if size else {}), **({"kv_from": kv_from} if kv_from is not None else {})}


def attention_layer(mlp=None, **sizes):
    return {"type": "attention", "mixer": attention_sizes(**sizes), "mlp": mlp}


def memory_sizes(heads=2, dim=8, vdim=8, gate_cap=6.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}


def parallel_layer(left=None, right=None, mlp=None):
    return {"type": "parallel", "mixer": {"left": left or attention_sizes(size=5), "right": right or memory_sizes()}, "mlp": mlp}


def retention_layer(heads=2, dim=8, vdim=8, decay=None, rot=None, mlp=None):
    decay = [1.0 - 2.0 ** -(2 + 2 * h) for h in range(heads)] if decay is None else decay
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": rot or rotation(dim)}, "mlp": mlp}


def make_config(layers, vocab=64, width=32, eps=1e-5, scale=4.0):
    return {"architecture": "Tumudra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}


def tensor_shapes(cfg: dict) -> list:
    W = cfg["width"]
    out = [("embed", (cfg["vocab"], W))]

    def att(p, m, bias):
        n = {"q": m["heads"] * m["dim"]}
        if m.get("kv_from") is None:
            n.update(k=m["kv_heads"] * m["dim"], v=m["kv_heads"] * m["vdim"])
        mats = [(p + x, (rows, W)) for x, rows in n.items()] + [(p + "o", (W, m["heads"] * m["vdim"]))]
        return mats + [(p + x + ".norm", (m["dim"],)) for x in n if x != "v"] + ([(x + ".b", (s[0],)) for x, s in mats] if bias else [])

    def lin(p, m):
        nk, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        return [(p + "q", (nk, W)), (p + "k", (nk, W)), (p + "v", (nv, W)), (p + "g", (nv, W)), (p + "o", (W, nv))]

    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        out.append((p + "norm1", (W,)))
        if lc["type"] == "attention":
            out += att(p + "mix.", m, True)
        elif lc["type"] == "retention":
            out += lin(p + "mix.", m)
        else:
            r, H = p + "mix.right.", m["right"]["heads"]
            out += att(p + "mix.left.", m["left"], False) + lin(r, m["right"]) + [(r + "norm", (H * m["right"]["vdim"],))]
            out += [(r + "i", (H, W)), (r + "i.b", (H,)), (r + "f", (H, W)), (r + "f.b", (H,)), (p + "mix.left.out", (W,)), (p + "mix.right.out", (W,))]
        if lc.get("mlp") is not None:
            out += [(p + "norm2", (W,)), (p + "mlp.up", (lc["mlp"]["ff"], W)), (p + "mlp.down", (W, lc["mlp"]["ff"]))]
    return out + [("final.norm", (W,)), ("head", (cfg["vocab"], W))]


def random_model(cfg: dict, seed: int = 0) -> dict:
    """bf16 weights: matrices ~ N(0, 1 / fan_in), smaller where they read the residual row (whose entries grow with the embedding scale);
    q / k norm weights large enough that single keys carry the output; biases away from zero; forget gates from a few tokens to
    hundreds."""
    g = torch.Generator().manual_seed(seed)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float32)
    w = {}
    for name, shape in tensor_shapes(cfg):
        if name.endswith((".q.norm", ".k.norm")):
            t = 1.6 + 0.3 * rn(*shape)
        elif "norm" in name.rsplit(".", 1)[-1] or name.endswith(".out"):
            t = 1.0 + 0.2 * rn(*shape)
        elif name.endswith(".f.b"):
            t = 1.0 + 2.5 * torch.rand(*shape, generator=g)
        elif name.endswith(".b"):
            t = 0.5 * rn(*shape)
        elif name == "embed":
            t = 0.5 * rn(*shape)
        elif name.endswith((".right.i", ".right.f")):
            t = 0.6 * rn(*shape) / math.sqrt(shape[-1])
        else:
            t = rn(*shape) / math.sqrt(shape[-1])
        w[name] = t.to(torch.bfloat16)
    return w
