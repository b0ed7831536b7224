"""A slow float64 model of the Pazilorn design, one function per mechanism,
written from the design's equations and sharing nothing with arks_amd.

A model is (cfg, weights): cfg the dict of config.json, weights a dict of
float64 tensors by checkpoint name. forward() runs one whole sequence and
returns the logits of every position and the residual after every layer;
there is no cache: attention looks back over the full prefix, a convolution
sees zeros before position 0 and a recurrent state starts at zero.

The design in short: every sublayer sits between two RMS norms,
x <- x + m * post(sub(pre(x))), x starting as the scaled embedding. Mixers:
"channel_delta" (delta rule with one decay per head and key channel, unit
queries and keys behind short convolutions, gated unit-RMS read-out) and
"latent_attention" (windowed attention through latents, ramp-scaled rotary
on its rotated part, one sigmoid gate per head). Feed-forward: routed
silu-GLU experts, softmax over the chosen logits. A layer may borrow the
weights of another. Logits through the embedding table, capped by tanh.
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


# ------------------------------------------------------------------ mixers
def delta_rule(q, k, v, g, beta):
    """q, k [n, H, D], v [n, H, V], g [n, H, D] decay factors, beta [n, H].
    Per head: S <- g S (rows), u = beta (v - S^T k), S <- S + k u^T,
    o = S^T q."""
    n, H, D = q.shape
    V = v.shape[2]
    S = torch.zeros(H, D, V, dtype=F64)
    out = torch.zeros(n, H, V, dtype=F64)
    for t in range(n):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def delta_decay(h, w, H, D):
    z = (h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]
    rate = torch.exp(w["A_log"])[:, None]
    return torch.exp(-rate * softplus(z).view(-1, H, D))


def channel_delta(h, w, m, eps):
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = conv_silu(h @ w["q"].T, w["q.conv"]).view(n, G, D)
    k = conv_silu(h @ w["k"].T, w["k.conv"]).view(n, G, D)
    v = conv_silu(h @ w["v"].T, w["v.conv"]).view(n, H, V)
    of_head = [i // (H // G) for i in range(H)]
    q = (unit_vector(q) * D ** -0.5)[:, of_head]
    k = unit_vector(k)[:, of_head]
    beta = sigmoid(h @ w["b"].T)
    o = delta_rule(q, k, v, delta_decay(h, w, H, D), beta)
    gate = sigmoid((h @ w["g1"].T) @ w["g2"].T).view(n, H, V)
    o = rms_norm(o, w["norm"], eps) * gate
    return o.reshape(n, H * V) @ w["o"].T


def ramped_freqs(rot):
    """Rotary frequencies f_i = base^(-2i/dims), divided by `factor` where
    the wavelength is long, untouched where it is short, blended between;
    and the factor on cos and sin."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F64), 1.0

    def at(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(at(sc["fast"])), 0)
    hi = min(math.ceil(at(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_half(x, rot):
    """x [n, heads, dims]: dims i and i + dims/2 turn by position * f_i."""
    f, mag = ramped_freqs(rot)
    half = rot["dims"] // 2
    a = torch.arange(x.shape[0], dtype=F64)[:, None, None] * f
    c, s = torch.cos(a) * mag, torch.sin(a) * mag
    u, v = x[..., :half], x[..., half:]
    return torch.cat([u * c - v * s, v * c + u * s], -1)


def window_attend(q, k, v, scale, window):
    """q, k [n, H, D], v [n, H, V]; row i sees j with 0 <= i - j < window."""
    n, H, _ = q.shape
    out = torch.zeros(n, H, v.shape[2], dtype=F64)
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    seen = (i - j >= 0) & (i - j < window)
    for h in range(H):
        s = (q[:, h] @ k[:, h].T) * scale
        out[:, h] = torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ v[:, h]
    return out


def latent_attention(h, w, m, eps):
    n = h.shape[0]
    H, D, R, V, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = rms_norm(h @ w["dq"].T, w["dq.norm"], eps)
    q = (cq @ w["uq"].T).view(n, H, D + R)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :rank], w["dkv.norm"], eps)
    kr = rotate_half(down[:, None, rank:], m["rot"])
    q = torch.cat([q[..., :D], rotate_half(q[..., D:], m["rot"])], -1)
    k = torch.cat([(c @ w["uk"].T).view(n, H, D), kr.expand(n, H, R)], -1)
    v = (c @ w["uv"].T).view(n, H, V)
    o = window_attend(q, k, v, m["scale"], m["mask"]["size"])
    o = o * sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(n, H * V) @ w["o"].T


# ------------------------------------------------------------ feed-forward
def routed_experts(h, w, mlp, margins=None):
    """Router logits with a bias; the `top` largest are chosen and weighted
    by the softmax over themselves. margins (a list) receives, per row, how
    far the last chosen logit lies above the first one left out."""
    E, top = mlp["router"]["experts"], mlp["router"]["top"]
    z = h @ w["router"].T + w["router.b"]
    if margins is not None and E > top:
        ranked = torch.sort(z, -1, descending=True).values
        margins.append(ranked[:, top - 1] - ranked[:, top])
    out = torch.zeros(h.shape[0], w["e0.down"].shape[0], dtype=F64)
    for t in range(h.shape[0]):
        best = torch.topk(z[t], top)
        share = torch.softmax(best.values, -1)
        for s, e in zip(share, best.indices.tolist()):
            y = silu(w[f"e{e}.gate"] @ h[t]) * (w[f"e{e}.up"] @ h[t])
            out[t] += s * (w[f"e{e}.down"] @ y)
    return out


# ------------------------------------------------------------------- model
def sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


MIXERS = {"channel_delta": channel_delta, "latent_attention": latent_attention}


def forward(cfg, weights, tokens, margins=None):
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = weights["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    after = []
    for i, spec in enumerate(cfg["layers"]):
        lw = sub(weights, f"l{spec.get('weights_of', i)}.")
        y = MIXERS[spec["type"]](rms_norm(x, lw["norm1"], eps),
                                 sub(lw, "mix."), spec["mixer"], eps)
        x = x + m * rms_norm(y, lw["norm1b"], eps)
        if spec.get("mlp") is not None:
            y = routed_experts(rms_norm(x, lw["norm2"], eps), sub(lw, "mlp."),
                               spec["mlp"], margins)
            x = x + m * rms_norm(y, lw["norm2b"], eps)
        after.append(x.clone())
    z = rms_norm(x, weights["final.norm"], eps) @ weights["embed"].T
    cap = cfg["logit_softcap"]
    return cap * torch.tanh(z / cap), after


def clear_rows(margins, least=0.06):
    """How many rows from the start every router chooses by a margin of at
    least `least` between logits (margins as forward() collects them)."""
    close = torch.stack(margins).amin(0) < least
    return int(close.nonzero()[0]) if bool(close.any()) else close.numel()


# ------------------------------------------------------- configs and weights
def moe_spec(experts=6, top=2, ff=24):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top}}


def delta_spec(heads=4, kv_heads=2, dim=8, vdim=12, conv=4, mlp="default",
               weights_of=None):
    spec = {"type": "channel_delta",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "conv": conv},
            "mlp": moe_spec() if mlp == "default" else mlp}
    if weights_of is not None:
        spec["weights_of"] = weights_of
    return spec


def latent_spec(heads=3, dim=8, rot_dim=6, vdim=10, kv_rank=20, q_rank=14,
                window=11, base=500.0, scaling="default", scale=None,
                mlp="default", weights_of=None):
    if scaling == "default":
        scaling = {"factor": 4.0, "original": 24, "fast": 6.0, "slow": 1.0}
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = scaling
    spec = {"type": "latent_attention", "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
        "kv_rank": kv_rank, "q_rank": q_rank, "rot": rot,
        "mask": {"size": window},
        "scale": (dim + rot_dim) ** -0.5 if scale is None else scale},
        "mlp": moe_spec() if mlp == "default" else mlp}
    if weights_of is not None:
        spec["weights_of"] = weights_of
    return spec


def make_config(layers, width=40, vocab=96, eps=1e-5, mult=0.6, scale=3.0,
                cap=6.0):
    return {"architecture": "Pazilorn", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "embedding": {"scale": scale},
            "residual_mult": mult, "logit_softcap": cap,
            "layers": list(layers)}


def tensor_shapes(cfg, ranks=(5, 7)):
    """ranks: rows of the low-rank decay and gate projections, which only
    the tensors' shapes give."""
    W, out = cfg["width"], {}
    out["embed"], out["final.norm"] = (cfg["vocab"], W), (W,)
    ra, rg = ranks
    for i, spec in enumerate(cfg["layers"]):
        if "weights_of" in spec:
            continue
        p, m = f"l{i}.", spec["mixer"]
        x = p + "mix."
        H, V = m["heads"], m["vdim"]
        out[p + "norm1"] = out[p + "norm1b"] = (W,)
        if spec["type"] == "channel_delta":
            G, D, K = m["kv_heads"], m["dim"], m["conv"]
            for leaf, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
                out[x + leaf], out[x + leaf + ".conv"] = (rows, W), (rows, K)
            out[x + "b"], out[x + "A_log"], out[x + "norm"] = (H, W), (H,), (V,)
            out[x + "a1"], out[x + "a2"] = (ra, W), (H * D, ra)
            out[x + "g1"], out[x + "g2"] = (rg, W), (H * V, rg)
            out[x + "dt_bias"] = (H * D,)
        else:
            D, R, rk, rq = m["dim"], m["rot_dim"], m["kv_rank"], m["q_rank"]
            out[x + "dq"], out[x + "dq.norm"] = (rq, W), (rq,)
            out[x + "uq"] = (H * (D + R), rq)
            out[x + "dkv"], out[x + "dkv.norm"] = (rk + R, W), (rk,)
            out[x + "uk"], out[x + "uv"] = (H * D, rk), (H * V, rk)
            out[x + "g"] = (H, W)
        out[x + "o"] = (W, H * V)
        mlp = spec.get("mlp")
        if mlp is not None:
            out[p + "norm2"] = out[p + "norm2b"] = (W,)
            E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            out[p + "mlp.router"], out[p + "mlp.router.b"] = (E, W), (E,)
            for e in range(E):
                out[p + f"mlp.e{e}.gate"] = out[p + f"mlp.e{e}.up"] = (ff, W)
                out[p + f"mlp.e{e}.down"] = (W, ff)
    return out


def random_weights(cfg, seed=0, ranks=(5, 7)):
    """Random weights, rounded to bfloat16 (what a checkpoint holds), as
    float64. Norm weights, taps, router biases and gates are of order one,
    and decays spread between nearly none and strong, so that leaving any of
    them out shows."""
    gen = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg, ranks).items():
        leaf = name.rsplit(".", 1)[-1]

        def rn(std):
            return torch.randn(shape, generator=gen, dtype=F64) * std

        if leaf in ("norm1", "norm2", "norm1b", "norm2b", "norm"):
            t = 1.0 + rn(0.3)
        elif leaf == "conv":
            t = rn(0.6)
        elif leaf == "A_log":
            t = rn(0.7)
        elif leaf == "dt_bias":
            t = rn(1.5) - 2.5
        elif name.endswith("router"):
            t = rn(2.0 * shape[-1] ** -0.5)
        elif name.endswith("router.b"):
            t = rn(0.7)
        elif leaf == "embed":
            t = rn(0.4)
        elif leaf in ("b", "g", "g1"):
            t = rn(1.5 * shape[-1] ** -0.5)
        else:
            t = rn(shape[-1] ** -0.5)
        w[name] = t.to(torch.bfloat16).to(F64)
    return w
