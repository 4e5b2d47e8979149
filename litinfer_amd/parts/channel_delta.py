"""A delta-rule mixer whose decay and whose removal rate are numbers of every key channel: a matrix state of fixed size
per request.

r = Wr xn, k = Wk xn (H heads x dim), v = Wv xn (H x vdim), no biases.  Per head and key channel:
    w = exp(-exp(-1/2) sigmoid(Ww2 tanh(Ww1 xn) + w0))      (the decay; Ww1 and Ww2 are a pair of low-rank matrices),
    a = sigmoid(Wa xn + a_bias)                             (the removal rate).
Per head, with the unit key u = k / sqrt(sum k^2 + 1e-6) and S of dim x vdim values:
    S <- diag(w) S - (a * u) (u^T S) + k v^T      (both terms read the old S; the key that is written is not normed),
    o = S^T r.
Each head's o is divided by its root mean square, the heads side by side are multiplied by the weights `norm`
[H vdim] and by sigmoid(Wg xn), and projected back by Wo.

A request keeps the dim x vdim matrices of all heads in its slot, float32 and zero at admission.  The projections run in
the engine's dtype with a float32 result; tanh, both sigmoids, the decays, the unit keys, the recurrence and the norm are
float32 in both engine dtypes (the low-rank pair's second product takes the tanh in the engine's dtype, as a projection).
One packed product gives a token's row [gate: H vdim | r: H dim | k: H dim | v: H vdim | a: H dim | w1: rank].  The rank is
in no configuration: the stored tensors decide it.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from ..weights.loader import ParamSpec
from .base import BatchNeeds, Mixer, StateNeed, register_part
from .linear import Linear

RANDOM_RANK = 64          # the low-rank pair's rank where weights are drawn rather than read


class ChannelDeltaMixer(Mixer):
    graph_safe = True

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        a = spec.args
        self.hidden = int(a["hidden_size"])
        self.heads = int(a["num_heads"])
        self.dim = int(a["head_dim"])
        self.vdim = int(a.get("value_dim") or self.dim)
        self.eps = float(a.get("eps", 1e-6))
        self.rank = int(a.get("rank") or RANDOM_RANK)
        if min(self.heads, self.dim, self.vdim, self.rank) <= 0:
            raise ValueError("channel delta: sizes must be positive")
        if self.dim > 256:
            raise ValueError("channel delta: the kernels take states of at most 256 values a column")
        self.state_name = str(a.get("state_name") or "channel_delta")
        self.inner = self.heads * self.vdim
        self.n_key = self.heads * self.dim
        self.names = {"r": "r", "k": "k", "v": "v", "gate": "g", "a": "a", "a_bias": "a.b", "w1": "w1", "w2": "w2", "w0": "w0",
                      "norm": "norm", "out": "o", **(a.get("names") or {})}
        self.proj = self.low = self.out = self.norm_w = None

    def cache_need(self):
        return StateNeed((self.heads, self.dim, self.vdim), torch.float32, name=self.state_name)

    def batch_needs(self):
        return BatchNeeds(row_tile=self.proj.row_tile() if self.proj is not None else 1)

    def expected_params(self):
        p, n = self.prefix, self.names
        e = {p + n[x]: ParamSpec((size, self.hidden)) for x, size in
             (("r", self.n_key), ("k", self.n_key), ("v", self.inner), ("gate", self.inner), ("a", self.n_key))}
        e.update({p + n["a_bias"]: ParamSpec((self.n_key,)), p + n["w0"]: ParamSpec((self.n_key,)),
                  p + n["w1"]: ParamSpec((self.rank, self.hidden), free_dims=(0,)),
                  p + n["w2"]: ParamSpec((self.n_key, self.rank), free_dims=(1,)),
                  p + n["norm"]: ParamSpec((self.inner,), init="one_plus_normal"),
                  p + n["out"]: ParamSpec((self.hidden, self.inner))})
        return e

    def load_params(self, get):
        p, n = self.prefix, self.names
        ws = [get(p + n[x]) for x in ("gate", "r", "k", "v", "a", "w1")]
        w2 = get(p + n["w2"])
        self.rank = int(ws[-1].shape[0])
        if int(w2.shape[1]) != self.rank:
            raise ValueError(f"{p + n['w2']} has {w2.shape[1]} columns, {p + n['w1']} has {self.rank} rows")
        dt = torch.float32 if any(w.dtype is torch.float32 for w in ws) else ws[0].dtype
        bias = torch.zeros(2 * self.inner + 3 * self.n_key + self.rank, dtype=torch.float32)
        bias[2 * self.inner + 2 * self.n_key:2 * self.inner + 3 * self.n_key] = get(p + n["a_bias"]).to(torch.float32)
        self.proj = Linear(self.rt, torch.cat([w.to(dt) for w in ws], dim=0), bias)
        self.low = Linear(self.rt, w2, get(p + n["w0"]).to(torch.float32))
        self.out = Linear(self.rt, get(p + n["out"]))
        self.norm_w = self.rt.vector(get(p + n["norm"]))

    def forward(self, xn, residual, ctx, cache):
        t, inner, n_key = xn.shape[0], self.inner, self.n_key
        n_scan = 3 * n_key + inner
        proj = ctx.ws.buffer("channel_delta.proj32", (t, inner + n_scan + self.rank), torch.float32)
        self.proj(xn, proj, ws=ctx.ws)
        th = ctx.ws.buffer("channel_delta.tanh", (t, self.rank), self.rt.dtype)
        ops.tanh_rows(proj[:, inner + n_scan:], th)
        low = ctx.ws.buffer("channel_delta.low32", (t, n_key), torch.float32)
        self.low(th, low, ws=ctx.ws)
        y = ctx.ws.buffer("channel_delta.y", (t, inner), torch.float32)
        ops.channel_delta(proj[:, inner:inner + n_scan], low, cache.states[self.state_name], ctx, y, self.heads, self.vdim, self.dim,
                          ws=ctx.ws)
        g = ctx.ws.buffer("channel_delta.gated", (t, inner), self.rt.dtype)
        ops.gated_group_norm(y, proj[:, :inner], self.norm_w, self.eps, self.heads, g, gate_after=True, gate="sigmoid")
        residual.add_linear(self.out, g)


register_part("mixer", "channel_delta", ChannelDeltaMixer)
