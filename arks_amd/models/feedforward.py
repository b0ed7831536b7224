"""Feed-forward sublayers of the layer-list decoders, each with its
constants as constructor parameters:

- GLU: W_down act(W_gate x, W_up x) for the activations of ops.glu_act.
- ClampedGLU: W_down act(W_gate x, W_up x) with the gate capped from above,
  the up branch clamped on both sides and offset by one:
  g = min(gate, limit), u = clamp(up, -limit, limit),
  act = g * sigmoid(alpha g) * (u + 1). Gate and up are one fused GEMM.
- GroupedMoE: `experts` small silu-GLU feed-forwards of which every row
  uses `top`; the router's softmax runs over all experts in fp32, experts
  are cut into `groups` contiguous runs and only the `keep` runs holding the
  highest single scores stay eligible; the chosen scores are renormalised.
  The gate|up matrices of all experts are stacked in ONE [experts * 2ff,
  width] matrix in the checkpoint's own [out, in] layout; the down matrices
  are kept pre-transposed ([in, out] per expert) like the framework's other
  sparse feed-forward (models/llama_family.py MoEMLP). Two execution paths
  as there: up to DENSE_TOKENS rows every expert runs on every row — one
  linear() for all gate|up projections (no per-expert copies of the rows),
  one batched GEMM down — with data-independent shapes, so the step can be
  captured; above it the (row, expert) pairs are sorted by expert and every
  expert runs plain GEMMs on its own segment (its row block of the stacked
  matrix).
- RoutedMoE: `experts` small silu-GLU feed-forwards of which every row
  uses the `top` with the highest sigmoid or softmax score, optionally
  renormalised over the chosen ones (for a softmax: the softmax over the
  chosen logits only); the router may have a bias; a shared expert of its
  own size may run on every row. weigh="input": the score multiplies the
  expert's INPUT, expert(s h), and the results are summed as they are;
  weigh="output": the sum of s expert(h). Since W (s h) = s (W h), the
  factor is applied in the activation kernel, in fp32, to the gate and up
  projections of h (input) or to their activated product (output: the down
  projection is linear). One matrix holds every gate|up
  projection, per expert and then the shared one, one matrix [width,
  experts * ff + shared_ff] every down projection. Up to DENSE_TOKENS rows
  the step is three GEMMs with data-independent shapes: all gate|up
  projections, an activation whose factor is 0 for the experts a row does
  not use (so their columns are exactly 0), and ONE down GEMM over all
  columns, which sums the chosen experts and the shared one. Above it the
  (row, expert) pairs are sorted by expert as in GroupedMoE. Experts may also
  be chosen in groups, by scores with a correction per expert that the
  weights do not see, and a group ranked by its best or its two best;
  the activation may be ClampedGLU's (limit, and shared_limit for the shared
  expert); and the shared expert may be weighed by sigmoid(W_sg h), a row of
  the router's matrix.
- SquaredReLU: W_down max(W_up x + b_up, 0)^2 + b_down.
"""

from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from .mixers import _param, linear, linear_f32


# rows of one expert's product are rounded up to a multiple of this
SEGMENT_ROWS = 64


def sort_by_expert(h, ids, experts: int):
    """The rows of h gathered in expert order, SEGMENT_ROWS - 1 more behind
    them; every (row, choice) pair's place there [T, k]; how many rows each
    expert has (the step's one host read)."""
    rows, place, counts = ops.moe_sort_pairs(ids, experts, SEGMENT_ROWS - 1)
    return h.index_select(0, rows), place, counts.tolist()


def expert_products(x, counts: list, weight) -> torch.Tensor:
    """x: rows in expert order and SEGMENT_ROWS - 1 spare ones; rows of
    expert e times weight(e). A product's row count is rounded up, so that
    the library meets few different shapes (it prepares each new one on the
    host); the rows too many belong to the experts behind, whose products
    come later and overwrite them, or are spare."""
    out = None
    at = 0
    for e, n in enumerate(counts):
        if n:
            w = weight(e)
            if out is None:
                out = torch.empty((x.shape[0], w.shape[1]), dtype=x.dtype,
                                  device=x.device)
            m = -(-n // SEGMENT_ROWS) * SEGMENT_ROWS
            torch.mm(x[at:at + m], w, out=out[at:at + m])
        at += n
    return out


class GLU(nn.Module):
    """W_down act(W_gate x, W_up x); act is one of ops.glu_act's kinds
    ("gelu_tanh": gelu_tanh(gate) * up; "swiglu"; "clamped"). Gate and up
    are one fused GEMM. Without projections of its own it follows the split
    protocol of models/mixers.py (in_spans, core, out_cols), so that a block
    can fuse them with its mixer's."""

    def __init__(self, width: int, ff: int, dtype, act: str = "gelu_tanh",
                 limit: float = 0.0, alpha: float = 1.0,
                 own_projections: bool = True):
        super().__init__()
        self.ff, self.act = ff, act
        self.limit, self.alpha = float(limit), float(alpha)
        self.out_cols = ff
        if own_projections:
            self.gate_up = _param(2 * ff, width, dtype=dtype)
            self.down = _param(width, ff, dtype=dtype)

    def in_spans(self) -> list:
        return [("gate", self.ff, False), ("up", self.ff, False)]

    def extra_weights(self) -> dict:
        return {}

    def weight_map(self) -> dict:
        return {"gate": (self.gate_up, 0), "up": (self.gate_up, self.ff),
                "down": (self.down, 0)}

    def core(self, p, batch, cache, out, out_scale) -> None:
        assert out_scale == 1.0
        ops.glu_act(p, self.act, self.limit, self.alpha, out=out)

    def forward(self, h, batch=None, cache=None) -> torch.Tensor:
        gu = linear(h, self.gate_up)
        return linear(ops.glu_act(gu, self.act, self.limit, self.alpha),
                      self.down)


class ClampedGLU(GLU):
    def __init__(self, width: int, ff: int, limit: float, dtype,
                 alpha: float = 1.702):
        super().__init__(width, ff, dtype, act="clamped", limit=limit,
                         alpha=alpha)


class SquaredReLU(nn.Module):
    """W_down max(W_up x + b_up, 0)^2 + b_down."""

    def __init__(self, width: int, ff: int, dtype):
        super().__init__()
        self.up = _param(ff, width, dtype=dtype)
        self.up_b = _param(ff, dtype=dtype)
        self.down = _param(width, ff, dtype=dtype)
        self.down_b = _param(width, dtype=dtype)

    def weight_map(self) -> dict:
        return {"up": (self.up, 0), "up.b": (self.up_b, 0),
                "down": (self.down, 0), "down.b": (self.down_b, 0)}

    def forward(self, h, batch=None, cache=None) -> torch.Tensor:
        return linear(ops.relu_square(linear(h, self.up, self.up_b)),
                      self.down, self.down_b)


class GroupedMoE(nn.Module):
    DENSE_TOKENS = 256  # see models/llama_family.py MoEMLP.DENSE_TOKENS

    def __init__(self, width: int, experts: int, ff: int, top: int,
                 groups: int, keep: int, dtype):
        super().__init__()
        assert experts % groups == 0 and keep <= groups
        assert top <= keep * (experts // groups)
        self.E, self.ff, self.top = experts, ff, top
        self.groups, self.keep, self.width = groups, keep, width
        self.router = _param(experts, width, dtype=dtype)
        self.w13 = _param(experts * 2 * ff, width, dtype=dtype)
        self.w2 = _param(experts, ff, width, dtype=dtype)

    def weight_map(self) -> dict:
        m = {"router": (self.router, 0)}
        W, ff = self.width, self.ff
        for e in range(self.E):
            m[f"e{e}.gate"] = (self.w13, e * 2 * ff, 0, (ff, W))
            m[f"e{e}.up"] = (self.w13, e * 2 * ff + ff, 0, (ff, W))
            # (param, row, col, shape, expert index, transposed)
            m[f"e{e}.down"] = (self.w2, 0, 0, (W, ff), e, True)
        return m

    def forward(self, h, batch=None, cache=None) -> torch.Tensor:
        T = h.shape[0]
        E, ff, W, k = self.E, self.ff, self.width, self.top
        z = linear_f32(h, self.router)  # fp32 logits
        weights, ids = ops.moe_route_grouped(z, k, self.groups, self.keep)
        if T <= self.DENSE_TOKENS:
            gu = linear(h, self.w13)  # [T, E * 2ff]
            a = ops.glu_act(gu.view(T * E, 2 * ff), "swiglu")
            y = torch.bmm(a.view(T, E, ff).transpose(0, 1), self.w2)
            return ops.moe_mix_seq(y, weights, ids)
        xs, place, counts = sort_by_expert(h, ids, E)
        gu = expert_products(
            xs, counts, lambda e: self.w13[e * 2 * ff:(e + 1) * 2 * ff].t())
        a = ops.glu_act(gu, "swiglu")
        y = expert_products(a, counts, lambda e: self.w2[e])
        return ops.moe_mix_rows_seq(y, weights, place)


class RoutedMoE(nn.Module):
    DENSE_TOKENS = 256  # see models/llama_family.py MoEMLP.DENSE_TOKENS

    def __init__(self, width: int, experts: int, ff: int, top: int, dtype,
                 shared_ff: int = 0, score: str = "sigmoid",
                 renorm: bool = False, weigh: str = "input",
                 router_bias: bool = False, groups: int = 1, keep: int = 1,
                 group_top: int = 1, correction: bool = False,
                 act: str = "swiglu", limit: float = 0.0,
                 shared_limit: float = 0.0, alpha: float = 1.0,
                 shared_gate: bool = False):
        super().__init__()
        assert experts % groups == 0 and keep <= groups
        assert top <= keep * (experts // groups)
        assert act == "swiglu" or weigh == "output"
        assert not shared_gate or (shared_ff and weigh == "output")
        self.groups, self.keep, self.group_top = groups, keep, group_top
        self.act, self.alpha = act, float(alpha)
        self.limit, self.shared_limit = float(limit), float(shared_limit)
        self.shared_gate = shared_gate
        self.correction = (_param(experts, dtype=torch.float32) if correction
                           else None)
        assert 1 <= top <= experts and score in ("sigmoid", "softmax")
        assert weigh in ("input", "output")
        self.weigh_input = weigh == "input"
        self.E, self.ff, self.top, self.sff = experts, ff, top, int(shared_ff)
        self.width, self.score, self.renorm = width, score, renorm
        # the shared expert's gate is one row more
        self.router = _param(experts + bool(shared_gate), width, dtype=dtype)
        self.router_b = (_param(experts, dtype=torch.float32) if router_bias
                         else None)
        self.w_gu = _param(experts * 2 * ff + 2 * self.sff, width, dtype=dtype)
        self.w_down = _param(width, experts * ff + self.sff, dtype=dtype)

    def weight_map(self) -> dict:
        W, ff, E, sff = self.width, self.ff, self.E, self.sff
        m = {"router": (self.router, 0, 0, (E, W))}
        if self.router_b is not None:
            m["router.b"] = (self.router_b, 0)
        if self.correction is not None:
            m["correction"] = (self.correction, 0)
        if self.shared_gate:
            m["shared.sg"] = (self.router, E, 0, (1, W))
        for e in range(E):
            m[f"e{e}.gate"] = (self.w_gu, e * 2 * ff)
            m[f"e{e}.up"] = (self.w_gu, e * 2 * ff + ff)
            m[f"e{e}.down"] = (self.w_down, 0, e * ff, (W, ff))
        if sff:
            m["shared.gate"] = (self.w_gu, E * 2 * ff)
            m["shared.up"] = (self.w_gu, E * 2 * ff + sff)
            m["shared.down"] = (self.w_down, 0, E * ff, (W, sff))
        return m

    def forward(self, h, batch=None, cache=None) -> torch.Tensor:
        T = h.shape[0]
        E, ff, sff, k = self.E, self.ff, self.sff, self.top
        z = linear_f32(h, self.router)  # fp32 logits
        route = dict(score=self.score, renorm=self.renorm, bias=self.router_b,
                     correction=self.correction, group_top=self.group_top,
                     shared_gate=self.shared_gate)
        if T <= self.DENSE_TOKENS:
            _, _, scale = ops.moe_route_grouped(
                z, k, self.groups, self.keep, matrix=True, **route)
            gu = linear(h, self.w_gu)
            return linear(ops.moe_glu_scaled(
                gu, scale, E, ff, sff, self.weigh_input, self.act, self.limit,
                self.shared_limit, self.alpha, self.shared_gate), self.w_down)
        weights, ids = ops.moe_route_grouped(z, k, self.groups, self.keep,
                                             **route)
        xs, place, counts = sort_by_expert(h, ids, E)
        gu = expert_products(
            xs, counts, lambda e: self.w_gu[e * 2 * ff:(e + 1) * 2 * ff].t())
        row_scale = None
        if self.weigh_input:
            row_scale = torch.zeros(gu.shape[0], dtype=torch.float32,
                                    device=h.device)
            row_scale[place.reshape(-1).long()] = weights.reshape(-1)
        a = ops.glu_act(gu, self.act, self.limit, self.alpha,
                        row_scale=row_scale)
        y = expert_products(
            a, counts, lambda e: self.w_down[:, e * ff:(e + 1) * ff].t())
        shared = None
        if sff:
            su = linear(h, self.w_gu[E * 2 * ff:])
            if self.shared_gate:  # one expert that every row uses
                sa = ops.moe_glu_scaled(
                    su, torch.sigmoid(z[:, E:]), 1, sff, 0, False, self.act,
                    self.shared_limit, 0.0, self.alpha)
            else:
                sa = ops.glu_act(su, self.act, self.shared_limit, self.alpha)
            shared = linear(sa, self.w_down[:, E * ff:])
        return ops.moe_mix_rows_seq(y, torch.ones_like(weights)
                                    if self.weigh_input else weights,
                                    place, shared)


def build_feedforward(mlp: dict, width: int, dtype, arch: str = "") -> nn.Module:
    kind = mlp.get("kind", "dense")
    if arch == "Rivolix":
        if kind != "moe":
            raise ValueError(f"unknown feed-forward kind {kind!r}")
        r = mlp["router"]
        return RoutedMoE(width, r["experts"], mlp["expert"]["ff"],
                         r["top"], dtype,
                         shared_ff=(mlp.get("shared") or {}).get("ff", 0))
    if arch == "Pazilorn":
        if kind != "moe":
            raise ValueError(f"unknown feed-forward kind {kind!r}")
        r = mlp["router"]
        return RoutedMoE(width, r["experts"], mlp["expert"]["ff"], r["top"],
                         dtype, score="softmax", renorm=True, weigh="output",
                         router_bias=True)
    if arch == "Fuzelorn":
        if kind == "dense":
            return SquaredReLU(width, mlp["ff"], dtype)
        if kind != "moe":
            raise ValueError(f"unknown feed-forward kind {kind!r}")
        r, shared = mlp["router"], mlp.get("shared") or {}
        groups = r.get("groups") or {}
        return RoutedMoE(
            width, r["experts"], mlp["expert"]["ff"], r["top"], dtype,
            shared_ff=shared.get("ff", 0), score="sigmoid", renorm=True,
            weigh="output", groups=groups.get("count", 1),
            keep=groups.get("keep", 1), group_top=2, correction=True,
            act="clamped", limit=mlp["expert"]["limit"],
            shared_limit=shared.get("limit", 0.0), alpha=1.702,
            shared_gate=bool(shared))
    if kind == "dense":
        return ClampedGLU(width, mlp["ff"], mlp["limit"], dtype)
    if kind == "moe":
        r = mlp["router"]
        return GroupedMoE(width, r["experts"], mlp["expert"]["ff"], r["top"],
                          r["groups"]["count"], r["groups"]["keep"], dtype)
    raise ValueError(f"unknown feed-forward kind {kind!r}")
