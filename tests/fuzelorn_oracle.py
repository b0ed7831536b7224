"""A slow float64 model of the Fuzelorn design, one function per mechanism,
written from the design's equations and sharing nothing with arks_amd.

A model is (cfg, weights): cfg the dict of config.json, weights a dict of
float64 tensors by checkpoint name. forward() runs one whole sequence and
returns the logits of every position and the residual after every layer run;
there is no cache: attention looks back over the full prefix, a convolution
sees zeros before position 0, a recurrent state starts at zero and the token
in front of the first one does not exist.

The design in short: scaled token embedding plus a hashed embedding of
(previous token, token); pre-norm layers, x <- x + mixer(n1(x)), x <- x +
ff(n2(x)); every mixer is two mixers on the same rows, windowed softmax
attention (whole-projection q/k norms, query factor, linear distance bias,
sink) beside a gated delta rule (scalar decay per head), each normed over the
model width before half their sum is taken. Feed-forward: squared-relu with
biases, or clamped-GLU experts chosen by group with corrected sigmoid scores
beside a gated shared expert. Some layers loop with the same weights. Logits
through a head of their own, capped by tanh.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


# ------------------------------------------------------------- small pieces
def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(z.clamp(max=30.0))))


def conv_silu(u, taps_w):
    """u [n, C], taps_w [C, K]: silu(sum_j taps_w[:, j] u_(t-K+1+j))."""
    n, C = u.shape
    K = taps_w.shape[1]
    y = torch.zeros(n, C, dtype=F64)
    for t in range(n):
        for j in range(K):
            src = t - K + 1 + j
            if src >= 0:
                y[t] += taps_w[:, j] * u[src]
    return silu(y)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


# --------------------------------------------------------------- embedding
def bigram_rows(tokens, spec):
    """Row of the hashed table for every token: (mul_prev * previous +
    mul_cur * token) mod buckets; the first token has a row of its own
    behind the buckets."""
    rows = [spec["buckets"]]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((prev * spec["mul_prev"] + cur * spec["mul_cur"])
                    % spec["buckets"])
    return rows


def embed(tokens, weights, spec):
    x = weights["embed"][torch.tensor(tokens)] * spec["scale"]
    if spec.get("bigram"):
        x = x + weights["bigram"][torch.tensor(bigram_rows(tokens, spec["bigram"]))]
    return x


# ------------------------------------------------------------------ mixers
def query_factor(n, temp):
    """1 + coef ln(floor((p + 1) / every) + 1) for positions 0 .. n-1."""
    return torch.tensor([1.0 + temp["coef"] * math.log((p + 1) // temp["every"] + 1)
                         for p in range(n)], dtype=F64)


def bias_slopes(H):
    return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def biased_attend(q, k, v, scale, window, slopes, sinks, rows=None):
    """q [n, H, D], k [n, H, D], v [n, H, V]. Row i sees j with
    0 <= i - j < window at score q.k scale - slope (i - j); the denominator
    also holds exp(sink). rows: the only rows asked for."""
    n, H, _ = q.shape
    out = torch.zeros(n, H, v.shape[2], dtype=F64)
    for h in range(H):
        for i in rows or range(n):
            lo = max(0, i - window + 1)
            s = k[lo:i + 1, h] @ q[i, h] * scale
            s = s - slopes[h] * (i - torch.arange(lo, i + 1, dtype=F64))
            m = max(float(s.max()), float(sinks[h]))
            p = torch.exp(s - m)
            out[i, h] = (p @ v[lo:i + 1, h]) / (p.sum() + math.exp(float(sinks[h]) - m))
    return out


def window_attention(h, w, m, eps):
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ w["q"].T, w["q.norm"], eps).view(n, H, D)
    k = rms_norm(h @ w["k"].T, w["k.norm"], eps).view(n, G, D)
    v = (h @ w["v"].T).view(n, G, V)
    if m.get("q_temp"):
        q = q * query_factor(n, m["q_temp"])[:, None, None]
    of_head = [i // (H // G) for i in range(H)]
    o = biased_attend(q, k[:, of_head], v[:, of_head], m["scale"],
                      m["mask"]["size"], bias_slopes(H), w["sink"])
    return o.reshape(n, H * V) @ w["o"].T


def delta_rule(q, k, v, g, beta):
    """q, k [n, H, D], v [n, H, V], g and beta [n, H]. Per head: S <- g S,
    u = beta (v - S^T k), S <- S + k u^T, o = S^T q."""
    n, H, D = q.shape
    V = v.shape[2]
    S = torch.zeros(H, D, V, dtype=F64)
    out = torch.zeros(n, H, V, dtype=F64)
    for t in range(n):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def head_decay(h, w):
    return torch.exp(-torch.exp(w["A_log"]) * softplus(h @ w["a"].T + w["dt_bias"]))


def gated_delta(h, w, m, eps):
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = conv_silu(h @ w["q"].T, w["q.conv"]).view(n, G, D)
    k = conv_silu(h @ w["k"].T, w["k.conv"]).view(n, G, D)
    v = conv_silu(h @ w["v"].T, w["v.conv"]).view(n, H, V)
    of_head = [i // (H // G) for i in range(H)]
    q = (unit_vector(q) * D ** -0.5)[:, of_head]
    k = unit_vector(k)[:, of_head]
    beta = sigmoid(h @ w["b"].T)
    o = delta_rule(q, k, v, head_decay(h, w), beta)
    o = rms_norm(o, w["norm"], eps) * silu(h @ w["g"].T).view(n, H, V)
    return o.reshape(n, H * V) @ w["o"].T


def parallel(h, w, m, eps):
    left = window_attention(h, sub(w, "left."), m["left"], eps)
    right = gated_delta(h, sub(w, "right."), m["right"], eps)
    return 0.5 * (rms_norm(left, w["left.out"], eps)
                  + rms_norm(right, w["right.out"], eps))


# ------------------------------------------------------------ feed-forward
def squared_relu_ff(h, w):
    a = (h @ w["up"].T + w["up.b"]).clamp(min=0.0) ** 2
    return a @ w["down"].T + w["down.b"]


def clamped_glu(h, gate, up, down, limit):
    g = (h @ gate.T).clamp(max=limit)
    u = (h @ up.T).clamp(-limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def choose_experts(choice, top, groups, keep):
    """The `top` largest choice scores of one row among the experts of the
    `keep` groups whose two largest scores sum highest; and by how much the
    decision was taken (the smaller of the groups' and the experts'
    margins)."""
    E = choice.shape[0]
    size = E // groups
    by_group = choice.view(groups, size)
    strength = torch.topk(by_group, min(2, size), -1).values.sum(-1)
    order = torch.sort(strength, descending=True)
    margin = math.inf
    if keep < groups:
        margin = float(order.values[keep - 1] - order.values[keep])
    open_ = torch.full((groups, size), -math.inf, dtype=F64)
    for g in order.indices[:keep].tolist():
        open_[g] = by_group[g]
    ranked = torch.sort(open_.view(-1), descending=True)
    if top < keep * size:
        margin = min(margin, float(ranked.values[top - 1] - ranked.values[top]))
    return ranked.indices[:top].tolist(), margin


def grouped_experts(h, w, mlp, margins=None):
    r = mlp["router"]
    s = sigmoid(h @ w["router"].T)
    out = torch.zeros(h.shape[0], h.shape[1], dtype=F64)
    rows = []
    for t in range(h.shape[0]):
        ids, margin = choose_experts(s[t] + w["correction"], r["top"],
                                     r["groups"]["count"], r["groups"]["keep"])
        rows.append(margin)
        total = float(s[t, ids].sum()) + 1e-20
        for e in ids:
            out[t] += s[t, e] / total * clamped_glu(
                h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"],
                mlp["expert"]["limit"])
    if margins is not None:
        margins.append(torch.tensor(rows, dtype=F64))
    if mlp.get("shared"):
        y = clamped_glu(h, w["shared.gate"], w["shared.up"], w["shared.down"],
                        mlp["shared"]["limit"])
        out = out + sigmoid(h @ w["shared.sg"].T) * y
    return out


def feed_forward(h, w, mlp, margins=None):
    if mlp.get("kind", "dense") == "dense":
        return squared_relu_ff(h, w)
    return grouped_experts(h, w, mlp, margins)


# ------------------------------------------------------------------- model
def sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def layer_order(cfg):
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(cfg, weights, tokens, margins=None):
    eps = cfg["norm"]["eps"]
    x = embed(tokens, weights, cfg["embedding"])
    after = []
    for i in layer_order(cfg):
        spec, lw = cfg["layers"][i], sub(weights, f"l{i}.")
        x = x + parallel(rms_norm(x, lw["norm1"], eps), sub(lw, "mix."),
                         spec["mixer"], eps)
        if spec.get("mlp") is not None:
            x = x + feed_forward(rms_norm(x, lw["norm2"], eps),
                                 sub(lw, "mlp."), spec["mlp"], margins)
        after.append(x.clone())
    z = rms_norm(x, weights["final.norm"], eps) @ weights["head"].T
    cap = cfg.get("logit_softcap")
    return (cap * torch.tanh(z / cap) if cap else z), after


# ------------------------------------------------------- configs and weights
def clear_rows(margins, least=0.01):
    """How many rows from the start every router chooses by a margin of at
    least `least` between choice scores (margins as forward() collects
    them)."""
    close = torch.stack(margins).amin(0) < least
    return int(close.nonzero()[0]) if bool(close.any()) else close.numel()


def left_spec(heads=4, kv_heads=2, dim=8, vdim=12, window=21, coef=0.4,
              every=7, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "mask": {"size": window}, "q_temp": {"coef": coef, "every": every},
            "scale": dim ** -0.5 if scale is None else scale}


def right_spec(heads=4, kv_heads=2, dim=8, vdim=12, conv=4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "conv": conv}


def dense_spec(ff=30):
    return {"kind": "dense", "ff": ff}


def moe_spec(experts=6, top=2, ff=24, limit=1.2, groups=3, keep=2,
             shared_ff=18, shared_limit=0.9):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "top": top,
                       "groups": {"count": groups, "keep": keep}},
            "shared": {"ff": shared_ff, "limit": shared_limit}}


def layer_spec(left=None, right=None, mlp=None):
    return {"type": "parallel",
            "mixer": {"left": left or left_spec(),
                      "right": right or right_spec()}, "mlp": mlp}


def make_config(layers, width=40, vocab=96, eps=1e-5, scale=1.7, cap=6.0,
                loop=None, buckets=53, mul_prev=11, mul_cur=5):
    cfg = {"architecture": "Fuzelorn", "vocab": vocab, "width": width,
           "norm": {"eps": eps}, "logit_softcap": cap,
           "embedding": {"scale": scale,
                         "bigram": {"buckets": buckets, "mul_prev": mul_prev,
                                    "mul_cur": mul_cur}},
           "layers": list(layers)}
    if loop is not None:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def tensor_shapes(cfg):
    W, out = cfg["width"], {}
    out["embed"] = out["head"] = (cfg["vocab"], W)
    out["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, W)
    out["final.norm"] = (W,)
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        out[p + "norm1"] = (W,)
        m, x = spec["mixer"]["left"], p + "mix.left."
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out[x + "q"], out[x + "q.norm"] = (H * D, W), (H * D,)
        out[x + "k"], out[x + "k.norm"] = (G * D, W), (G * D,)
        out[x + "v"], out[x + "sink"] = (G * V, W), (H,)
        out[x + "o"], out[x + "out"] = (W, H * V), (W,)
        m, x = spec["mixer"]["right"], p + "mix.right."
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for leaf, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
            out[x + leaf], out[x + leaf + ".conv"] = (rows, W), (rows, m["conv"])
        out[x + "b"] = out[x + "a"] = (H, W)
        out[x + "A_log"] = out[x + "dt_bias"] = (H,)
        out[x + "g"], out[x + "norm"] = (H * V, W), (V,)
        out[x + "o"], out[x + "out"] = (W, H * V), (W,)
        mlp, x = spec.get("mlp"), p + "mlp."
        if mlp is None:
            continue
        out[p + "norm2"] = (W,)
        if mlp["kind"] == "dense":
            ff = mlp["ff"]
            out[x + "up"], out[x + "up.b"] = (ff, W), (ff,)
            out[x + "down"], out[x + "down.b"] = (W, ff), (W,)
            continue
        E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        out[x + "router"], out[x + "correction"] = (E, W), (E,)
        for e in range(E):
            out[x + f"e{e}.gate"] = out[x + f"e{e}.up"] = (ff, W)
            out[x + f"e{e}.down"] = (W, ff)
        if mlp.get("shared"):
            ff = mlp["shared"]["ff"]
            out[x + "shared.gate"] = out[x + "shared.up"] = (ff, W)
            out[x + "shared.down"], out[x + "shared.sg"] = (W, ff), (1, W)
    return out


def random_weights(cfg, seed=0):
    """Random weights, rounded to bfloat16 (what a checkpoint holds), as
    float64. Norm weights, sinks, biases, corrections and gates are of order
    one, and decays spread between nearly none and strong, so that leaving
    any of them out shows."""
    gen = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]

        def rn(std):
            return torch.randn(shape, generator=gen, dtype=F64) * std

        if leaf in ("norm1", "norm2", "norm", "out"):
            t = 1.0 + rn(0.3)
        elif leaf == "conv":
            t = rn(0.6)
        elif leaf == "sink":
            t = rn(1.2)
        elif leaf == "A_log":
            t = rn(0.7)
        elif leaf == "dt_bias":
            t = rn(1.5) - 2.5
        elif leaf == "correction":
            t = rn(0.25)
        elif leaf == "b" and len(shape) == 1:
            t = rn(0.5)
        elif leaf in ("router", "sg"):
            t = rn(2.0 * shape[-1] ** -0.5)
        elif leaf in ("embed", "bigram"):
            t = rn(0.7)
        elif leaf in ("b", "a", "g"):
            t = rn(1.5 * shape[-1] ** -0.5)
        else:
            t = rn(shape[-1] ** -0.5)
        w[name] = t.to(torch.bfloat16).to(F64)
    return w
