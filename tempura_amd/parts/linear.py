"""Mixers around a linear recurrence whose state is a matrix per head with a decay per key channel that depends on the
token (``ops.linear_scan``).  Per head, with S [key, value] from zero at a request's start:

    S <- diag(w) S + k v^T

and a read-out either behind the update, o = S^T q, or in front of it with a bonus u for the current token,
o = (S + diag(u) k v^T)^T q.  Everything between the projections is float32 whatever the compute dtype.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import BranchMixer, Mixer, StateSpec, WeightInfo, pad_rows, register_part


class WkvMixer(Mixer):
    """Token-shifted inputs in front of the recurrence with a bonus.  With H = ``num_heads`` heads of D = ``head_dim``, x a
    token's normed row and x' the row of the token before it (zeros for a request's first): each of five inputs is its own
    mix x + (x' - x) * mu_s.  q (called r here), k and v are projections of their mixes [H, D]; the gate is
    silu(W_g mix_g); the decay is w = exp(-exp(W_w2 tanh(W_w1 mix_w) + w0)), the bonus u a tensor [H, D].  Each head's
    read-out is divided by its root mean square (``norm_eps``), the concatenated heads are multiplied by a weight [H D] and
    by the gate, then projected back.

    The part reads its normed rows in float32, so that the mixes are formed from unrounded rows and rounded once.  The rank
    of the decay's low-rank projection is the checkpoint's own.  Per request it keeps one float32 row: the state
    column by column [H, D, D], then the last token's normed row [hidden]."""
    graph_safe = True
    returns_output = True      # with ``residual`` None the output comes back instead of being added
    input_dtype = torch.float32
    MIXES = ("r", "k", "v", "g", "w")

    def __init__(self, spec, hidden_size, dtype, device):
        super().__init__(spec, hidden_size, dtype, device)
        p = spec.params
        self.num_heads = int(p["num_heads"])
        self.head_dim = int(p["head_dim"])
        self.norm_eps = float(p["norm_eps"])
        self.inner = self.num_heads * self.head_dim
        self.row_off = self.inner * self.head_dim      # where the last token's row starts in the state row

    @classmethod
    def expected_weights(cls, spec, hidden_size):
        p, w = spec.params, spec.weights
        n, rank = int(p["num_heads"]) * int(p["head_dim"]), p.get("decay_rank")
        out = {w["mu_" + s]: WeightInfo((hidden_size,)) for s in cls.MIXES}
        out.update({w[name]: WeightInfo((n, hidden_size)) for name in ("r", "k", "v", "gate")})
        out.update({w["w1"]: WeightInfo((rank, hidden_size)), w["w2"]: WeightInfo((n, rank)), w["w0"]: WeightInfo((n,)),
                    w["u"]: WeightInfo((p["num_heads"], p["head_dim"])), w["norm"]: WeightInfo((n,), "ones"),
                    w["o"]: WeightInfo((hidden_size, n))})
        return out

    def state_spec(self):
        return StateSpec((self.row_off + self.hidden_size,), torch.float32)

    def load_weights(self, get):
        w = self.spec.weights
        f32 = lambda name: self._to_device(get(w[name]), torch.float32)
        self.mu = torch.stack([f32("mu_" + s) for s in self.MIXES]).contiguous()
        w1, w2 = get(w["w1"]), f32("w2")
        if w2.shape[1] != w1.shape[0]:
            raise ValueError("wkv: the two halves of the decay's projection disagree on its rank")
        self.w2_t = w2.t().contiguous()      # [rank, columns]: lanes read neighbours
        self.w0, self.norm_w = f32("w0"), f32("norm")
        self.bonus = f32("u").reshape(-1)
        # one weight per mix, in the order of the mixes: rows of one stacked weight, which a step of a few rows takes in one launch
        rows = [pad_rows(self._to_device(t), 16) for t in [get(w[name]) for name in ("r", "k", "v", "gate")] + [w1]]
        self.ends, self.cols = [], []
        for t in rows:
            self.cols.append(self.ends[-1] if self.ends else 0)
            self.ends.append(self.cols[-1] + t.shape[0])
        self.w_all = ops.tile_weight(torch.cat(rows, dim=0).contiguous())
        self.w_in = [ops.weight_rows(self.w_all, lo, hi) for lo, hi in zip(self.cols, self.ends)]
        self.w_out = ops.tile_weight(self._to_device(get(w["o"])))

    def forward(self, x, ctx, cache, residual=None):
        few = {"blocked": True} if ctx.max_q_len == 1 and ops.group_linear_ok(x.shape[0], self.w_all) else {}
        mixes = ops.token_shift(x, self.mu, cache.state, self.row_off, ctx.cu_seqlens, ctx.token_req, ctx.state_slots,
                                ctx.num_requests, self.dtype, max_run=ctx.max_q_len, **few)
        if few:
            proj = ops.group_linear(mixes, self.w_all, self.ends)
            r, k, v, (g, g_col), (w, w_col) = ((proj, col) for col in self.cols)
        else:
            r, k, v, (g, g_col), (w, w_col) = ((ops.linear(m, wt, torch.float32), 0) for m, wt in zip(mixes, self.w_in))
        decay = ops.lowrank_up(w, w_col, self.w2_t, "exp_exp", bias=self.w0, in_act="tanh")
        o = ops.linear_scan(r, k, v, decay, cache.state, 0, ctx.cu_seqlens, ctx.state_slots, ctx.num_requests,
                            self.num_heads, self.head_dim, self.head_dim, bonus=self.bonus, max_run=ctx.max_q_len)
        act = torch.empty((o.shape[0], self.inner), dtype=self.dtype, device=o.device)
        ops.head_norm_gate(o, self.norm_w, None, self.norm_eps, 1.0, self.num_heads, act, 0, gate_rows=g, gate_col0=g_col, gate_act="silu")
        return ops.linear(act, self.w_out, torch.float32, residual=residual)


register_part("mixer", "wkv", WkvMixer)


class GatedLinearMixer(BranchMixer):
    """Gated linear attention.  With H = ``num_heads``, D = ``head_dim`` and Dv = ``value_dim``: q = W_q x * ``q_scale`` and
    k = W_k x [H, D], v = W_v x [H, Dv]; a decay per head and key channel w = sigmoid(W_a2 (W_a1 x) + bias)^(1 /
    ``decay_root``).  The read-out follows the update.  Each head's o is divided by its root mean square (``norm_eps``)
    and multiplied by a weight [Dv] shared by the heads, the concatenated heads by silu(W_g x), then projected back.

    The columns of its input product are [q | k | v | gate | a1]; the rank of the decay's low-rank projection is the
    checkpoint's own.  Per request it keeps the state column by column in one float32 row, [H, Dv, D]."""

    def __init__(self, spec, hidden_size, dtype, device):
        super().__init__(spec, hidden_size, dtype, device)
        p = spec.params
        self.num_heads = int(p["num_heads"])
        self.head_dim = int(p["head_dim"])
        self.value_dim = int(p["value_dim"])
        self.norm_eps = float(p["norm_eps"])
        self.q_scale = float(p.get("q_scale", self.head_dim ** -0.5))
        self.decay_root = float(p["decay_root"])
        if self.decay_root <= 0:
            raise ValueError("gated_linear: decay_root must be positive")
        self.qk_dim = self.num_heads * self.head_dim
        self.inner = self.num_heads * self.value_dim

    @classmethod
    def expected_weights(cls, spec, hidden_size):
        p, w = spec.params, spec.weights
        H, D, Dv, rank = int(p["num_heads"]), int(p["head_dim"]), int(p["value_dim"]), p.get("decay_rank")
        return {
            w["q"]: WeightInfo((H * D, hidden_size)), w["k"]: WeightInfo((H * D, hidden_size)), w["v"]: WeightInfo((H * Dv, hidden_size)),
            w["gate"]: WeightInfo((H * Dv, hidden_size)), w["a1"]: WeightInfo((rank, hidden_size)), w["a2"]: WeightInfo((H * D, rank)),
            w["a2_bias"]: WeightInfo((H * D,)), w["norm"]: WeightInfo((Dv,), "ones"), w["o"]: WeightInfo((hidden_size, H * Dv)),
        }

    def state_floats(self) -> int:
        return self.num_heads * self.value_dim * self.head_dim

    def load_branch(self, get):
        w = self.spec.weights
        f32 = lambda name: self._to_device(get(w[name]), torch.float32)
        a1, a2 = get(w["a1"]), f32("a2")
        if a2.shape[1] != a1.shape[0]:
            raise ValueError("gated_linear: the two halves of the decay's projection disagree on its rank")
        self.a2_t = a2.t().contiguous()      # [rank, columns]: lanes read neighbours
        self.a2_bias, self.norm_w = f32("a2_bias"), f32("norm")
        rows = [get(w["q"]), get(w["k"]), get(w["v"]), get(w["gate"]), a1]
        self.v_col = 2 * self.qk_dim
        self.gate_col = self.v_col + self.inner
        self.a1_col = self.gate_col + self.inner
        return torch.cat([self._to_device(t) for t in rows], dim=0).contiguous(), self._to_device(get(w["o"]))

    def run(self, proj, col0, ctx, cache, out, out_col0, scale):
        decay = ops.lowrank_up(proj, col0 + self.a1_col, self.a2_t, "root_sigmoid", bias=self.a2_bias, rate=1.0 / self.decay_root)
        o = ops.linear_scan((proj, col0), (proj, col0 + self.qk_dim), (proj, col0 + self.v_col), decay, cache.state, self.state_off,
                            ctx.cu_seqlens, ctx.state_slots, ctx.num_requests, self.num_heads, self.head_dim, self.value_dim,
                            q_scale=self.q_scale, max_run=ctx.max_q_len)
        ops.head_norm_gate(o, self.norm_w, None, self.norm_eps, scale, self.num_heads, out, out_col0, gate_rows=proj,
                           gate_col0=col0 + self.gate_col, gate_act="silu")


register_part("mixer", "gated_linear", GatedLinearMixer)
