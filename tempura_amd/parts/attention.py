"""Grouped-query attention over the paged cache.

Per token: q, k, v projections (no bias), position encoding on q and k, k and v
stored into the cache pages, causal (optionally windowed) softmax attention
over the request's cached keys with ``kv_head = head // (heads / kv_heads)``,
output projection added into the residual stream
(/root/reference/engine/src/model.rs:1007-1152,
/root/reference/kernels/src/attention.rs:28-87).
A window of ``w`` lets query position p see keys p-w+1 .. p
(/root/reference/kernels/src/attention.rs:55-59).

Options beyond that, each a parameter of the part:
* ``bias``: the q and k projections have biases (tensors ``q_bias``, ``k_bias``);
* ``values: "keys"``: there is no value projection, a head's values are its keys as projected;
* ``distance_bias``: a learned bias per head and distance is added to the scaled score (the scale does not
  multiply it).  Kind ``"log_buckets"``: the tensor has B rows of one value per head, and distance n reads row
  n while n < B // 2, else row min(B - 1, B // 2 + floor(ln(n / (B // 2)) / ln(max_distance / (B // 2)) * (B - B // 2))).
  B is the tensor's own first dimension.
The first two need a position encoding that does not rotate (``"none"``).
* ``qk_norm`` (``{"eps"}``, tensors ``q_norm``, ``k_norm`` of [head_dim]): every head of q and of k is divided by its
  root mean square and multiplied by the weight (one weight for all q heads, one for all k heads), before any rotation;
* ``value_dim``: the values of a head have another size than its keys;
* ``sink`` (tensor ``sink`` [heads]): the softmax's denominator holds one more term exp(sink[head]) that has no key
  and no value;
  A number instead of True: every head's sink has that score, and there is no tensor;
* ``keep_first``: under a ``window`` a query also sees the request's first ``keep_first`` keys (their pages stay held).
The last four run with own values and a rows-in-float32 projection (no split norm).
* ``chunk`` (instead of ``window``): a query sees the keys of its own aligned chunk of that many positions, counted from
  the request's start; pages of finished chunks go back to the pool;
* ``softcap``: a scaled score s becomes softcap * tanh(s / softcap);
* ``gate``: the concatenated heads are multiplied by sigmoid(W_g x) (tensor ``gate``) before the output projection.
Between the projection and the cache, in this order (``bias``, this form of ``qk_norm`` and ``value_position`` select one
kernel that does all of it on the projection's float32 rows, ``ops.qkv_rows``):
* ``bias`` with values of their own: q, k and v have biases (tensors ``q_bias``, ``k_bias``, ``v_bias``);
* ``qk_norm`` with ``over: "projection"``: q is divided by the root mean square of the whole q projection, all heads
  together, and multiplied by its weight (one value per row of the projection); k likewise;
* ``value_position``: a rotary position part over ``value_dim`` elements that turns the values by their own positions
  before they are cached; every head's output is turned back by the query's position (in front of the gate).
"""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from ..kernels import ops
from .base import BranchMixer, CacheSpec, Mixer, WeightInfo, build_part, pad_rows, part_class, register_part
from .rope import paired_order, reorder_heads


def log_bucket(n: int, buckets: int, max_distance: int) -> int:
    """The row of a ``log_buckets`` table that distance ``n`` >= 0 reads: exact below half the table, then
    logarithmic up to ``max_distance``, then the last row."""
    half = buckets // 2
    if n < half:
        return n
    if half == 0 or max_distance <= half:
        return buckets - 1
    return min(buckets - 1, half + int(math.floor(math.log(n / half) / math.log(max_distance / half) * (buckets - half))))


def distance_table(rows: torch.Tensor, max_distance: int, window) -> torch.Tensor:
    """float32 [heads, L] from a ``log_buckets`` tensor [B, heads]: entry n is the bias of distance n; every
    distance from L - 1 on has the value of entry L - 1 (the last row, or never occurs under the window)."""
    buckets = rows.shape[0]
    length = 1
    while log_bucket(length - 1, buckets, max_distance) < buckets - 1 and (window is None or length < window):
        length += 1
    index = torch.tensor([log_bucket(n, buckets, max_distance) for n in range(length)], dtype=torch.long)
    return rows.to(torch.float32)[index].t().contiguous()


class PagedAttention(Mixer):
    graph_safe = True      # only kernels on device-resident step data: may be captured in a graph
    #: the value cache is transposed, eight consecutive tokens of one element being one 16-byte piece: a portion that
    #: starts at a multiple of eight positions (and of eight rows of the batch) has its values stored piece by piece
    preferred_portion_align = 8
    split_norm = True      # takes rows whose norm its first product finishes; prepares the next norm in its last
    returns_output = True  # with ``residual`` None the output comes back instead of being added
    takes_side_rows = True  # (behind the gate's rows, or behind q | k | v where one kernel reads the projection's rows)

    def __init__(self, spec, hidden_size, dtype, device):
        super().__init__(spec, hidden_size, dtype, device)
        p = spec.params
        self.num_heads = int(p["num_heads"])
        self.num_kv_heads = int(p["num_kv_heads"])
        self.head_dim = int(p["head_dim"])
        if self.num_heads % self.num_kv_heads != 0:
            raise ValueError("attention: heads must be a multiple of kv heads")
        self.scale = float(p["scale"])
        self.window = p.get("window")
        self.q_dim = self.num_heads * self.head_dim
        self.kv_dim = self.num_kv_heads * self.head_dim
        self.position = build_part("position", p["position"], hidden_size, dtype, device)
        self.has_bias = bool(p.get("bias", False))
        values = p.get("values", "own")
        if values not in ("own", "keys"):
            raise ValueError(f"attention: values {values!r} unknown (known: own, keys)")
        self.values_are_keys = values == "keys"
        self.distance_bias = p.get("distance_bias")
        if self.distance_bias is not None and self.distance_bias.get("kind") != "log_buckets":
            raise ValueError(f"attention: distance bias {self.distance_bias.get('kind')!r} unknown (known: log_buckets)")
        if self.values_are_keys and self.position.rotary() is not None:
            raise ValueError("attention: values that are the keys need a position encoding that does not rotate")
        #: q and k come straight from the projection (biases added, keys stored as keys and as values): no rotation kernel
        self.plain_qk = self.values_are_keys
        self.qk_norm = p.get("qk_norm")
        self.value_dim = int(p.get("value_dim") or self.head_dim)
        sink = p.get("sink", False)
        self.has_sink = sink is not None and sink is not False
        #: the score of every head's sink when it is a constant (None: a tensor holds the scores)
        self.sink_score = float(sink) if self.has_sink and sink is not True else None
        self.keep_first = int(p.get("keep_first") or 0)
        if self.keep_first < 0 or (self.keep_first and self.window is None):
            raise ValueError("attention: keep_first needs a window and must not be negative")
        self.chunk = int(p.get("chunk") or 0)
        self.softcap = float(p.get("softcap") or 0.0)
        if self.chunk < 0 or self.softcap < 0 or (self.chunk and self.window is not None):
            raise ValueError("attention: chunks exclude a window; chunk and softcap must not be negative")
        if self.softcap and self.distance_bias is not None:
            raise ValueError("attention: a softcap and a distance bias do not combine")
        self.gate = bool(p.get("gate", False))
        over = self.qk_norm.get("over", "head") if self.qk_norm is not None else "head"
        if over not in ("head", "projection"):
            raise ValueError(f"attention: qk_norm over {over!r} unknown (known: head, projection)")
        vp = p.get("value_position")
        self.value_position = None if vp is None else build_part("position", vp, hidden_size, dtype, device)
        if vp is not None and (self.value_position.rotary() is None or self.value_position.rotary()[1] != self.value_dim
                               or self.value_position.factor != 1.0):
            raise ValueError("attention: value_position must turn all value_dim elements, without a factor")
        #: biases, the norm over the whole projection and turned values are one kernel on the projection's rows
        self.rows_path = (self.has_bias and not self.values_are_keys) or over == "projection" or vp is not None
        if self.rows_path and self.qk_norm is not None and over == "head":
            raise ValueError("attention: a norm per head does not combine with biases on own values or turned values")
        #: the options that take the projection's float32 rows through kernels of their own
        self.extended = self.rows_path or self.qk_norm is not None or self.value_dim != self.head_dim or self.has_sink or self.keep_first > 0
        if self.extended and (self.plain_qk or self.distance_bias is not None):
            raise ValueError("attention: qk_norm, value_dim, sink, keep_first, biases on own values and turned values do not combine with "
                             "values that are the keys or a distance bias")
        self.v_dim = self.num_kv_heads * self.value_dim
        # sizes the matrix-core attention kernels take once q and the cached keys have zeros behind their own elements
        # (no score changes): keys narrower than values, or than the key size of a pair that the kernels are built for
        self.key_dim = self.head_dim
        pair = ops.fast_pair(self.head_dim, self.value_dim)
        if (self.extended and dtype == torch.bfloat16 and pair is not None and self.head_dim % 2 == 0
                and ops.fast_attention_takes(self.has_sink, self.keep_first)):
            self.key_dim = pair[0]
        self.split_norm = not self.plain_qk and not self.extended      # (these projections take finished rows only)
        self.q_norm_w = self.k_norm_w = self.sink_w = None
        self.v_bias = None
        self.w_gates = None        # rows of the gate and side rows, where they are no part of wqkv
        self.wqkv = None
        self.wo = None
        self.q_bias = self.k_bias = self.dist_table = None

    @classmethod
    def expected_weights(cls, spec, hidden_size):
        p, w = spec.params, spec.weights
        q_dim = p["num_heads"] * p["head_dim"]
        kv_dim = p["num_kv_heads"] * p["head_dim"]
        out = {
            w["q"]: WeightInfo((q_dim, hidden_size)),
            w["k"]: WeightInfo((kv_dim, hidden_size)),
            w["o"]: WeightInfo((hidden_size, q_dim)),
        }
        vd = int(p.get("value_dim") or p["head_dim"])
        if p.get("values", "own") != "keys":
            out[w["v"]] = WeightInfo((p["num_kv_heads"] * vd, hidden_size))
        out[w["o"]] = WeightInfo((hidden_size, p["num_heads"] * vd))
        if p.get("qk_norm") is not None:
            whole = p["qk_norm"].get("over", "head") == "projection"
            out[w["q_norm"]] = WeightInfo((q_dim if whole else p["head_dim"],), "ones")
            out[w["k_norm"]] = WeightInfo((kv_dim if whole else p["head_dim"],), "ones")
        if p.get("sink", False) is True:
            out[w["sink"]] = WeightInfo((p["num_heads"],))
        if p.get("bias", False):
            out[w["q_bias"]] = WeightInfo((q_dim,))
            out[w["k_bias"]] = WeightInfo((kv_dim,))
            if p.get("values", "own") != "keys":
                out[w["v_bias"]] = WeightInfo((p["num_kv_heads"] * vd,))
        if p.get("gate", False):
            out[w["gate"]] = WeightInfo((p["num_heads"] * vd, hidden_size))
        if p.get("distance_bias") is not None:
            # (the number of rows is the tensor's own; a configuration may name it for random weights)
            out[w["distance_bias"]] = WeightInfo((p["distance_bias"].get("buckets"), p["num_heads"]))
        # a position encoding may have tensors of its own (a rotary one has none)
        out.update(part_class("position", p["position"].kind).expected_weights(p["position"], hidden_size))
        return out

    def _paired(self, t: torch.Tensor) -> torch.Tensor:
        """The rows of a q or k projection with every head's rotary elements in paired order: rows
        (2 d, 2 d + 1) of a head are rows (d, d + rotary_dim / 2) of the checkpoint's split-half order, so
        that the two elements that rotate together are neighbours (the rotation kernels expect that, and a
        product's epilogue can rotate what it holds).  q and k are permuted alike, which leaves every score
        as it was; the cache then holds keys in this order."""
        rot = self.position.rotary()
        if rot is None:
            return t
        return reorder_heads(t, self.head_dim, paired_order(self.head_dim, rot[1], getattr(self.position, "layout", "halves")))

    def _paired_values(self, t: torch.Tensor) -> torch.Tensor:
        """The rows of a value projection (its bias, the gate's rows) with every head's elements in the order in which
        turned values are kept."""
        if self.value_position is None:
            return t
        return reorder_heads(t, self.value_dim, paired_order(self.value_dim, self.value_dim, self.value_position.layout))

    def load_weights(self, get):
        w = self.spec.weights
        if self.has_bias:
            self.q_bias = self._to_device(self._paired(get(w["q_bias"])), torch.float32)
            self.k_bias = self._to_device(self._paired(get(w["k_bias"])), torch.float32)
            if not self.values_are_keys:
                self.v_bias = self._to_device(self._paired_values(get(w["v_bias"])), torch.float32)
        if self.distance_bias is not None:
            self.dist_table = self._to_device(distance_table(get(w["distance_bias"]), int(self.distance_bias["max_distance"]),
                                                             self.window), torch.float32)
        # One [q_dim + 2 kv_dim, hidden] matrix: one product instead of three.
        parts = [self._paired(get(w["q"])), self._paired(get(w["k"]))]
        if not self.values_are_keys:
            parts.append(self._paired_values(get(w["v"])))
        # what else reads the same input: the gate's rows, then the side rows.  Where one kernel takes the projection's
        # rows anyway they are columns of the same product; else (the projection may rotate and store in its epilogue)
        # they are a product of their own.
        beside = [self._paired_values(get(w["gate"]))] if self.gate else []
        if self.side_rows is not None:
            beside.append(self.side_rows)
            self.side_rows = True
        self.gate_col0 = self.q_dim + self.kv_dim + self.v_dim if self.rows_path else 0
        self.side_col0 = self.gate_col0 + (self.num_heads * self.value_dim if self.gate else 0)
        if self.rows_path:
            parts, beside = parts + beside, []
        rows = torch.cat([self._to_device(t) for t in parts], dim=0).contiguous()
        # (stored tiled where the sizes allow: the products then read whole cache lines)
        self.wqkv = ops.tile_weight(pad_rows(rows, 16) if self.rows_path else rows)
        if beside:
            self.w_gates = ops.tile_weight(pad_rows(torch.cat([self._to_device(t) for t in beside], dim=0), 16))
        wo = get(w["o"])
        if self.value_position is not None:
            wo = self._paired_values(wo.t()).t()
        self.wo = ops.tile_weight(self._to_device(wo))
        if self.qk_norm is not None:
            # (a weight per head is the same for all heads: it is ordered like one of them)
            self.q_norm_w = self._to_device(self._paired(get(w["q_norm"])), torch.float32)
            self.k_norm_w = self._to_device(self._paired(get(w["k_norm"])), torch.float32)
        if self.sink_score is not None:
            self.sink_w = torch.full((self.num_heads,), self.sink_score, dtype=torch.float32, device=self.device)
        elif self.has_sink:
            self.sink_w = self._to_device(get(w["sink"]), torch.float32)
        self.position.load_weights(get)

    def cache_spec(self):
        kind, span = ("window", self.window) if self.window is not None else ("chunk", self.chunk) if self.chunk else ("full", None)
        if self.keep_first:
            return SizedValueCacheSpec("window_keep_first", self.num_kv_heads, self.key_dim, self.window, self.value_dim, self.keep_first)
        if self.value_dim != self.key_dim:
            return SizedValueCacheSpec(kind, self.num_kv_heads, self.key_dim, span, self.value_dim)
        return CacheSpec(kind, self.num_kv_heads, self.key_dim, span)

    def forward(self, x, ctx, cache, residual, next_norm=None):
        rot = self.position.rotary()
        q = None
        gates = None       # float32 rows that hold the gate's and the side rows' columns
        if self.rows_path:
            q, gates = self._project_rows(x, ctx, cache, rot)
        elif self.plain_qk:
            q = self._project_plain(x, ctx, cache)
        elif rot is not None and cache.writes and not self.extended:
            rows = x.x if isinstance(x, ops.Prenormed) else x
            if ops.linear_rope_ok(x.shape[0], self.wqkv.shape[0], x.shape[1], self.head_dim, rot[1], cache.k.shape[2],
                                  rows.dtype, cache.k.dtype, isinstance(x, ops.Prenormed)):
                # a few rows (decoding) or a long step: the projection rotates and stores its rows itself
                table = self.position.table(ctx, always=True) if hasattr(self.position, "table") else None
                q = ops.linear_rope_kv(x, self.wqkv, ctx.positions, ctx.slot_mapping[cache.group], rot[0], rot[1], rot[2],
                                       self.num_heads, self.num_kv_heads, self.head_dim, cache.k, cache.v, table)
        if q is None:
            q = self._project_and_rotate(x, ctx, cache, rot)
        if self.w_gates is not None:
            gates = ops.linear(x, self.w_gates, torch.float32)
        if self.extended or self.chunk or self.softcap:
            a = ops.paged_attention(
                q, cache.k, cache.v, ctx.block_tables[cache.group], ctx.cu_seqlens, ctx.context_lens,
                ctx.token_req, self.scale, int(self.window or 0), ctx.max_q_len, ctx.max_context_len,
                ctx.num_single, sink=self.sink_w, keep_first=self.keep_first, chunk=self.chunk, softcap=self.softcap)
        elif self.dist_table is not None:
            a = ops.paged_attention(
                q, cache.k, cache.v, ctx.block_tables[cache.group], ctx.cu_seqlens, ctx.context_lens,
                ctx.token_req, self.scale, int(self.window or 0), ctx.max_q_len, ctx.max_context_len,
                ctx.num_single, dist_bias=self.dist_table)
        else:
            a = ops.paged_attention(
                q, cache.k, cache.v, ctx.block_tables[cache.group], ctx.cu_seqlens, ctx.context_lens,
                ctx.token_req, self.scale, int(self.window or 0), ctx.max_q_len, ctx.max_context_len,
                ctx.num_single)
        if self.value_position is not None:
            vp = self.value_position
            a = ops.turn_gate(a, ctx.positions, vp.inv_freq, self.value_dim, gates if self.gate else None, self.gate_col0, vp.table(ctx))
        elif self.gate:
            gated = torch.empty_like(a)
            ops.sigmoid_gate(a, gates, self.gate_col0, 1.0, gated, 0)
            a = gated
        if self.side_rows is not None:
            if residual is not None:
                raise ValueError("attention: with side rows the output comes back, it is not added")
            return ops.linear(a, self.wo, torch.float32), (gates, self.side_col0)
        if residual is None:
            return ops.linear(a, self.wo, torch.float32)
        if next_norm is None:
            ops.linear(a, self.wo, torch.float32, residual=residual)
            return None
        return ops.linear(a, self.wo, torch.float32, residual=residual, next_norm=next_norm)[1]

    def _project_rows(self, x, ctx, cache, rot):
        """(q, the product's float32 rows): biases, the norm over the whole projection, rotation of q, k and v and the
        cache write are one kernel behind one product, whose columns behind q | k | v are the gate's and the side rows'."""
        if not cache.writes:
            raise ValueError("attention: a projection with biases, a norm over all heads or turned values writes its own cache")
        rows = ops.linear(x, self.wqkv, torch.float32)
        inv_freq, rotary_dim, factor = rot if rot is not None else (None, 0, 1.0)
        vp = self.value_position
        q = ops.qkv_rows(rows, ctx.positions, ctx.slot_mapping[cache.group], self.num_heads, self.num_kv_heads, self.head_dim, self.value_dim,
                         cache.k, cache.v, inv_freq, rotary_dim, factor, self.position.table(ctx) if rot is not None else None,
                         (self.q_bias, self.k_bias, self.v_bias), None if self.qk_norm is None else (self.q_norm_w, self.k_norm_w),
                         0.0 if self.qk_norm is None else float(self.qk_norm["eps"]), None if vp is None else vp.inv_freq,
                         None if vp is None else vp.table(ctx), self.key_dim)
        return q, rows

    def _project_plain(self, x, ctx, cache):
        """q ([n, heads, head_dim]) of a projection without rotation: biases added, k stored as keys and, when the
        values are the keys, as values too (the value cache is transposed, so it is a second store, not a view)."""
        if isinstance(x, ops.Prenormed):
            raise ValueError("attention: rows with an unfinished norm need a rotary projection")
        if cache.writes:
            rows = ops.linear(x, self.wqkv, torch.float32)
            return ops.qk_store(rows, self.q_bias, self.k_bias, ctx.slot_mapping[cache.group], self.num_heads,
                                self.num_kv_heads, self.head_dim, cache.k, cache.v, self.dtype)
        rows = ops.linear(x, ops.weight_rows(self.wqkv, 0, self.q_dim), torch.float32)
        return ops.qk_store(rows, self.q_bias, None, None, self.num_heads, self.num_kv_heads, self.head_dim, None, None, self.dtype)

    def _project_extended(self, x, ctx, cache, rot):
        """q of a projection with a norm per head and/or values of their own size: the float32 rows are normed in
        place, then rotated (if the position part rotates) and stored by the cache-write kernel."""
        if rot is None and type(self.position).__name__ != "NoPosition":
            raise ValueError("attention: qk_norm, value_dim, sink and keep_first need a rotary position part or none")
        writes = cache.writes
        w = self.wqkv if writes else ops.weight_rows(self.wqkv, 0, self.q_dim)
        qkv = ops.linear(x, w, torch.float32)
        if self.qk_norm is not None:
            ops.head_rmsnorm(qkv, 0, self.num_heads, self.q_norm_w, self.q_dim, self.num_kv_heads if writes else 0, self.k_norm_w,
                             self.head_dim, float(self.qk_norm["eps"]))
        inv_freq, rotary_dim, factor, table = None, 0, 1.0, None
        if rot is not None:
            inv_freq, rotary_dim, factor = rot
            table = self.position.table(ctx) if hasattr(self.position, "table") else None
        return ops.rope_kv_write(qkv, ctx.positions, ctx.slot_mapping[cache.group] if writes else None, inv_freq, rotary_dim, factor,
                                 self.num_heads, self.num_kv_heads, self.head_dim, cache.k if writes else None,
                                 cache.v if writes else None, self.dtype, table, value_dim=self.value_dim, pad_dim=self.key_dim)

    def _project_and_rotate(self, x, ctx, cache, rot):
        """q (rotated, [n, heads, head_dim]) of the projection; k and v go to the cache."""
        # (with a rotary position the next kernel may add the projection's partial sums itself)
        if self.extended:
            return self._project_extended(x, ctx, cache, rot)
        if cache.writes:
            qkv = ops.linear(x, self.wqkv, torch.float32, partial_ok=rot is not None)
        else:
            # A call that reads another call's cache needs queries only.
            qkv = ops.linear(x, ops.weight_rows(self.wqkv, 0, self.q_dim), torch.float32, partial_ok=rot is not None)
        if rot is None:
            q = qkv[:, : self.q_dim]
            k = qkv[:, self.q_dim: self.q_dim + self.kv_dim] if cache.writes else None
            q2, k2 = self.position.apply(q, k, ctx.positions)
            if cache.writes:
                qkv = torch.cat([q2, k2, qkv[:, self.q_dim + self.kv_dim:]], dim=1).contiguous()
            else:
                qkv = q2.contiguous()
            inv_freq, rotary_dim, factor, table = None, 0, 1.0, None
        else:
            inv_freq, rotary_dim, factor = rot
            table = self.position.table(ctx) if hasattr(self.position, "table") else None
        q = ops.rope_kv_write(
            qkv, ctx.positions, ctx.slot_mapping[cache.group] if cache.writes else None,
            inv_freq, rotary_dim, factor, self.num_heads, self.num_kv_heads, self.head_dim,
            cache.k if cache.writes else None, cache.v if cache.writes else None, self.dtype, table)
        return q


register_part("mixer", "attention", PagedAttention)


@dataclass(frozen=True)
class SizedValueCacheSpec(CacheSpec):
    """Keys of ``head_dim`` and values of ``value_dim``: keys [kv_heads, page_size, head_dim] as ever, values
    transposed [kv_heads, value_dim, page_size]."""
    value_dim: int = 0
    #: with kind ``"window_keep_first"``: the request's first keys that stay visible (and held) under the window
    keep_first: int = 0

    def planes(self, page_size: int):
        return {"k": (self.num_kv_heads, page_size, self.head_dim), "v": (self.num_kv_heads, self.value_dim, page_size)}


class ConvAttention(BranchMixer):
    """Grouped-query softmax attention over the paged cache as a branch (``branch_attention``; ``conv_attention`` where the
    convolution below is part of the design).  q, k and v may pass a short causal convolution per
    channel right behind their projections (``conv_taps`` taps, no bias, no activation, zeros before a request's
    start; before any norm and rotation; 0 or left out: no convolution), the values may have another size than the keys
    (``value_dim``), with ``qk_norm`` (``{"eps"}``, tensors ``q_norm``, ``k_norm`` of [head_dim]) every head of q and of k is
    divided by its root mean square and multiplied by the weight before any rotation, and the
    concatenated heads are multiplied by sigmoid(W_g x) before the output projection (``gate``: True, a number per
    element, or ``"head"``, one number per head).  The position
    encoding, the scale and an optional window are parameters as for ``attention``.

    The columns of its input product are [q | k | v | gate]; a request's state is the convolution's last
    ``conv_taps - 1`` inputs [conv_taps - 1, q | k | v], float32."""
    preferred_portion_align = 8      # (the value cache is transposed: see ``PagedAttention``)

    def __init__(self, spec, hidden_size, dtype, device):
        super().__init__(spec, hidden_size, dtype, device)
        p = spec.params
        self.num_heads = int(p["num_heads"])
        self.num_kv_heads = int(p["num_kv_heads"])
        self.head_dim = int(p["head_dim"])
        self.value_dim = int(p.get("value_dim") or self.head_dim)
        if self.num_heads % self.num_kv_heads != 0:
            raise ValueError("conv_attention: heads must be a multiple of kv heads")
        self.scale = float(p["scale"])
        self.window = p.get("window")
        self.taps = int(p.get("conv_taps") or 0)
        if self.taps < 0:
            raise ValueError("conv_attention: conv_taps must not be negative")
        gate = p.get("gate", False)
        if gate not in (True, False, None, "head"):
            raise ValueError(f"conv_attention: gate {gate!r} unknown (known: True, head)")
        self.gate = bool(gate)
        #: columns that share a gate
        self.gate_per = self.value_dim if gate == "head" else 1
        self.qk_norm = p.get("qk_norm")
        self.position = build_part("position", p["position"], hidden_size, dtype, device)
        if self.position.rotary() is None and type(self.position).__name__ != "NoPosition":
            raise ValueError("conv_attention: the position part must rotate or be none")
        #: one kernel takes the float32 rows to q and the cache: norm per head, rotation, cache write
        self.rows_path = self.qk_norm is not None or self.taps == 0
        self.q_dim = self.num_heads * self.head_dim
        self.k_dim = self.num_kv_heads * self.head_dim
        self.v_dim = self.num_kv_heads * self.value_dim
        self.channels = self.q_dim + self.k_dim + self.v_dim
        self.inner = self.num_heads * self.value_dim
        # values wider than keys, of a size the matrix-core attention kernels take: q and the cached keys get zeros
        # behind their own elements up to the values' size (no score changes; the key pages are that much wider),
        # so that those kernels serve; every other pair of sizes runs the general kernel
        self.key_dim = self.head_dim
        if self.rows_path:
            pair = ops.fast_pair(self.head_dim, self.value_dim) if dtype == torch.bfloat16 and self.head_dim % 2 == 0 else None
            self.key_dim = pair[0] if pair is not None else self.head_dim
        elif dtype == torch.bfloat16 and self.head_dim < self.value_dim <= 128 and self.value_dim % 32 == 0 and self.head_dim % 2 == 0:
            self.key_dim = self.value_dim
        self.conv_w = self.norms = None

    @classmethod
    def expected_weights(cls, spec, hidden_size):
        p, w = spec.params, spec.weights
        vd = int(p.get("value_dim") or p["head_dim"])
        q_dim, k_dim, v_dim = p["num_heads"] * p["head_dim"], p["num_kv_heads"] * p["head_dim"], p["num_kv_heads"] * vd
        taps = int(p.get("conv_taps") or 0)
        out = {
            w["q"]: WeightInfo((q_dim, hidden_size)), w["k"]: WeightInfo((k_dim, hidden_size)), w["v"]: WeightInfo((v_dim, hidden_size)),
            w["o"]: WeightInfo((hidden_size, p["num_heads"] * vd)),
        }
        if taps:
            out.update({w["q_conv"]: WeightInfo((q_dim, taps)), w["k_conv"]: WeightInfo((k_dim, taps)), w["v_conv"]: WeightInfo((v_dim, taps))})
        if p.get("qk_norm") is not None:
            out.update({w["q_norm"]: WeightInfo((p["head_dim"],), "ones"), w["k_norm"]: WeightInfo((p["head_dim"],), "ones")})
        if p.get("gate", False):
            out[w["gate"]] = WeightInfo((p["num_heads"] * (1 if p["gate"] == "head" else vd), hidden_size))
        out.update(part_class("position", p["position"].kind).expected_weights(p["position"], hidden_size))
        return out

    def state_floats(self) -> int:
        return max(0, self.taps - 1) * self.channels

    def cache_spec(self):
        kind = "window" if self.window is not None else "full"
        if self.value_dim == self.key_dim:
            return CacheSpec(kind, self.num_kv_heads, self.key_dim, self.window)
        return SizedValueCacheSpec(kind, self.num_kv_heads, self.key_dim, self.window, self.value_dim)

    def _paired(self, t: torch.Tensor) -> torch.Tensor:
        """Rows of a q or k tensor (projection, convolution or a norm's weight) with every head's rotary elements in paired order
        (see ``PagedAttention._paired``: the rotation kernels take neighbours as pairs)."""
        rot = self.position.rotary()
        if rot is None or rot[1] == 0:
            return t
        rd, half, d = rot[1], rot[1] // 2, self.head_dim
        order = torch.arange(d)
        order[0:rd:2] = torch.arange(half)
        order[1:rd:2] = torch.arange(half) + half
        return t.view(t.shape[0] // d, d, -1)[:, order.to(t.device), :].reshape(t.shape)

    def load_branch(self, get):
        w = self.spec.weights
        rows = [self._paired(get(w["q"])), self._paired(get(w["k"])), get(w["v"])]
        if self.gate:
            rows.append(get(w["gate"]))
        if self.taps:
            conv = torch.cat([self._paired(get(w["q_conv"])), self._paired(get(w["k_conv"])), get(w["v_conv"])], dim=0)
            self.conv_w = self._to_device(conv, torch.float32).t().contiguous()      # tap-major for the kernel
        if self.qk_norm is not None:
            self.norms = tuple(self._to_device(self._paired(get(w[name])), torch.float32) for name in ("q_norm", "k_norm"))
        self.position.load_weights(get)
        return torch.cat([self._to_device(t) for t in rows], dim=0).contiguous(), self._to_device(get(w["o"]))

    def run(self, proj, col0, ctx, cache, out, out_col0, scale):
        if not cache.writes:
            raise ValueError("conv_attention: a call that reads another call's cache is not supported")
        qkv, qkv_col0 = proj, col0
        if self.taps:
            qkv_col0 = 0
            qkv = ops.causal_conv(proj, col0, self.channels, self.conv_w, None, cache.state, ctx.cu_seqlens, ctx.token_req,
                                  ctx.state_slots, ctx.num_requests, state_off=self.state_off, act=False)
        rot = self.position.rotary()
        inv_freq, rotary_dim, factor, table = None, 0, 1.0, None
        if rot is not None:
            inv_freq, rotary_dim, factor = rot
            table = self.position.table(ctx) if hasattr(self.position, "table") else None
        if self.rows_path:
            q = ops.qkv_rows(qkv, ctx.positions, ctx.slot_mapping[cache.group], self.num_heads, self.num_kv_heads, self.head_dim,
                             self.value_dim, cache.k, cache.v, inv_freq, rotary_dim, factor, table, norms=self.norms,
                             eps=float(self.qk_norm["eps"]) if self.qk_norm is not None else 0.0, pad_dim=self.key_dim, col0=qkv_col0,
                             norm_over="head")
        else:
            q = ops.rope_kv_write(qkv, ctx.positions, ctx.slot_mapping[cache.group], inv_freq, rotary_dim, factor, self.num_heads,
                                  self.num_kv_heads, self.head_dim, cache.k, cache.v, self.dtype, table, value_dim=self.value_dim,
                                  pad_dim=self.key_dim)
        a = ops.paged_attention(q, cache.k, cache.v, ctx.block_tables[cache.group], ctx.cu_seqlens, ctx.context_lens,
                                ctx.token_req, self.scale, int(self.window or 0), ctx.max_q_len, ctx.max_context_len, ctx.num_single)
        ops.sigmoid_gate(a, proj if self.gate else None, col0 + self.channels, scale, out, out_col0, self.gate_per if self.gate else 1)


register_part("mixer", "conv_attention", ConvAttention)
register_part("mixer", "branch_attention", ConvAttention)


class LatentAttention(BranchMixer):
    """Softmax attention whose keys and values are expanded from one compressed vector per token.  With H =
    ``num_heads``, per head D = ``head_dim`` unrotated and R = ``rotary_dim`` rotated query/key elements, values of
    ``value_dim`` and a latent of L = ``latent_dim``: q = W_q x, per head [D unrotated | R rotated]; W_down x has L + R
    rows: the first L, RMS-normed (``norm_eps``) with a weight, are the latent c, the last R (not normed) are ONE rotated
    key part shared by all heads.  Head h's unrotated key is W_uk[h] c, its value W_uv[h] c; the score is
    (q_plain . k_plain + q_rot . k_rot) * ``scale``.  The position part rotates neighbouring pairs (2i, 2i + 1) of the R
    rotated elements of q and of the shared key part.  ``window``, ``gate`` (sigmoid(W_g x) on the concatenated heads) as
    for ``conv_attention``.

    The cache holds expanded keys and values per head: keys [rotated | unrotated] of R + D, values of ``value_dim``.
    Every model of this kind here runs under a sliding window, which bounds what a request holds, and a decode step
    then needs no products with the expansion weights for the keys it reads.  At load the rows of W_q are brought into
    the cache's order per head, [rotated | unrotated]; q and k are ordered alike, so no score changes.

    The columns of its input product are [q | down | gate]; it keeps no per-request state."""
    preferred_portion_align = 8      # (the value cache is transposed: see ``PagedAttention``)

    def __init__(self, spec, hidden_size, dtype, device):
        super().__init__(spec, hidden_size, dtype, device)
        p = spec.params
        self.num_heads = int(p["num_heads"])
        self.head_dim = int(p["head_dim"])
        self.rotary_dim = int(p["rotary_dim"])
        self.value_dim = int(p["value_dim"])
        self.latent_dim = int(p["latent_dim"])
        self.scale = float(p["scale"])
        self.window = p.get("window")
        self.norm_eps = float(p["norm_eps"])
        self.gate = bool(p.get("gate", False))
        self.position = build_part("position", p["position"], hidden_size, dtype, device)
        rot = self.position.rotary()
        if (rot[1] if rot is not None else 0) != self.rotary_dim:
            raise ValueError("latent_attention: the position part must rotate exactly the rotated elements")
        self.key_dim = self.head_dim + self.rotary_dim
        self.q_dim = self.num_heads * self.key_dim
        self.down_dim = self.latent_dim + self.rotary_dim
        self.inner = self.num_heads * self.value_dim

    @classmethod
    def expected_weights(cls, spec, hidden_size):
        p, w = spec.params, spec.weights
        H, D, R, Dv, L = (int(p[k]) for k in ("num_heads", "head_dim", "rotary_dim", "value_dim", "latent_dim"))
        out = {w["q"]: WeightInfo((H * (D + R), hidden_size)), w["down"]: WeightInfo((L + R, hidden_size)),
               w["latent_norm"]: WeightInfo((L,), "ones"), w["up_k"]: WeightInfo((H * D, L)), w["up_v"]: WeightInfo((H * Dv, L)),
               w["o"]: WeightInfo((hidden_size, H * Dv))}
        if p.get("gate", False):
            out[w["gate"]] = WeightInfo((H * Dv, hidden_size))
        out.update(part_class("position", p["position"].kind).expected_weights(p["position"], hidden_size))
        return out

    def cache_spec(self):
        kind = "window" if self.window is not None else "full"
        if self.value_dim == self.key_dim:
            return CacheSpec(kind, self.num_heads, self.key_dim, self.window)
        return SizedValueCacheSpec(kind, self.num_heads, self.key_dim, self.window, self.value_dim)

    def load_branch(self, get):
        from .base import pad_rows
        w = self.spec.weights
        H, D, R = self.num_heads, self.head_dim, self.rotary_dim
        q = get(w["q"])
        q = torch.cat([q.view(H, D + R, -1)[:, D:], q.view(H, D + R, -1)[:, :D]], dim=1).reshape(q.shape)      # per head [rotated | unrotated]
        rows = [q, get(w["down"])]
        if self.gate:
            rows.append(get(w["gate"]))
        self.latent_norm_w = self._to_device(get(w["latent_norm"]), torch.float32)
        self.w_up = ops.tile_weight(pad_rows(torch.cat([self._to_device(get(w["up_k"])), self._to_device(get(w["up_v"]))], dim=0), 16))
        self.position.load_weights(get)
        return torch.cat([self._to_device(t) for t in rows], dim=0).contiguous(), self._to_device(get(w["o"]))

    def run(self, proj, col0, ctx, cache, out, out_col0, scale):
        if not cache.writes:
            raise ValueError("latent_attention: a call that reads another call's cache is not supported")
        H = self.num_heads
        c = ops.rmsnorm_cols(proj, col0 + self.q_dim, self.latent_dim, self.latent_norm_w, self.norm_eps, self.dtype)
        up = ops.linear(c, self.w_up, torch.float32)
        rows = ops.latent_rows(proj, col0, col0 + self.q_dim + self.latent_dim, up, H, self.head_dim, self.rotary_dim, self.value_dim)
        inv_freq, rotary_dim, factor = self.position.rotary()
        table = self.position.table(ctx) if hasattr(self.position, "table") else None
        q = ops.rope_kv_write(rows, ctx.positions, ctx.slot_mapping[cache.group], inv_freq, rotary_dim, factor, H, H, self.key_dim,
                              cache.k, cache.v, self.dtype, table, value_dim=self.value_dim)
        a = ops.paged_attention(q, cache.k, cache.v, ctx.block_tables[cache.group], ctx.cu_seqlens, ctx.context_lens,
                                ctx.token_req, self.scale, int(self.window or 0), ctx.max_q_len, ctx.max_context_len, ctx.num_single)
        ops.sigmoid_gate(a, proj if self.gate else None, col0 + self.q_dim + self.down_dim, scale, out, out_col0)


register_part("mixer", "latent_attention", LatentAttention)


class LatentCacheAttention(BranchMixer):
    """Softmax attention without positions whose cache holds ONE compressed vector a token, the latent c, from which
    every head's keys and values are linear maps.  With H = ``num_heads``, per head D = ``head_dim`` query/key elements
    and Dv = ``value_dim`` values, a latent of L = ``latent_dim`` and a query latent of ``query_rank``:

        c_q = rmsnorm(W_dq x) * w_dq      q_h = W_uq[h] c_q                       (queries through a latent of their own)
        c   = rmsnorm(W_dkv x) * w_dkv    k_h = W_uk[h] c    v_h = W_uv[h] c      score = (q_h . k_h) * ``scale``

    causal (or under a ``window``), optionally with a ``sink`` per head in the softmax's denominator, then W_o on the
    concatenated heads.  ``own_latent`` False: the layer has no W_dkv; its call of the run order names the cache slot of
    the layer whose latents it reads (with its own W_uk, W_uv and everything else).

    The maps are folded into the two ends: q_h . (W_uk[h] c) = (W_uk[h]^T q_h) . c and W_o[:, h] W_uv[h] (sum_j p_j c_j), so
    the attention itself is one shared key/value head of L elements whose values are its keys, read straight from the
    cache: a step expands nothing of what it reads, however long the context.  The folded weights W_uk[h]^T W_uq[h]
    [H L, query_rank] and W_o[:, h] W_uv[h] [hidden, H L] are formed once at load (in float64, then rounded to the
    compute dtype); per token they cost H L (query_rank + hidden) multiply-adds against H (D query_rank + Dv hidden) plus
    H L (D + Dv) for the maps one after the other, which is the price of a cache and a decode step that stay small.

    The columns of its input product are [dq | dkv]; it keeps no per-request state.  A page holds the latents as keys
    [1, page_size, L] and once more transposed as values [1, L, page_size], the layout every attention kernel reads."""
    preferred_portion_align = 8      # (the value cache is transposed: see ``PagedAttention``)

    def __init__(self, spec, hidden_size, dtype, device):
        super().__init__(spec, hidden_size, dtype, device)
        p = spec.params
        self.num_heads = int(p["num_heads"])
        self.head_dim = int(p["head_dim"])
        self.value_dim = int(p["value_dim"])
        self.latent_dim = int(p["latent_dim"])
        #: the query latent's size: the configuration's, or (None) the checkpoint's own, known once the tensors are loaded
        self.query_rank = int(p["query_rank"]) if p.get("query_rank") is not None else None
        self.scale = float(p["scale"])
        self.norm_eps = float(p["norm_eps"])
        self.window = p.get("window")
        self.has_sink = bool(p.get("sink", False))
        self.own_latent = bool(p.get("own_latent", True))
        self.inner = self.num_heads * self.latent_dim
        self.sink_w = None

    @classmethod
    def expected_weights(cls, spec, hidden_size):
        p, w = spec.params, spec.weights
        H, D, Dv, L = (int(p[k]) for k in ("num_heads", "head_dim", "value_dim", "latent_dim"))
        Q = int(p["query_rank"]) if p.get("query_rank") is not None else None      # (None: the checkpoint says it)
        out = {w["dq"]: WeightInfo((Q, hidden_size)), w["dq_norm"]: WeightInfo((Q,), "ones"), w["uq"]: WeightInfo((H * D, Q)),
               w["uk"]: WeightInfo((H * D, L)), w["uv"]: WeightInfo((H * Dv, L)), w["o"]: WeightInfo((hidden_size, H * Dv))}
        if p.get("own_latent", True):
            out[w["dkv"]] = WeightInfo((L, hidden_size))
            out[w["dkv_norm"]] = WeightInfo((L,), "ones")
        if p.get("sink", False):
            out[w["sink"]] = WeightInfo((H,))
        return out

    def cache_spec(self):
        return CacheSpec("window" if self.window is not None else "full", 1, self.latent_dim, self.window)

    def load_branch(self, get):
        w = self.spec.weights
        H, D, Dv, L = self.num_heads, self.head_dim, self.value_dim, self.latent_dim
        f64 = lambda name: get(w[name]).to(torch.float64)
        dq = get(w["dq"])
        if self.query_rank is None:
            self.query_rank = int(dq.shape[0])
        if get(w["uq"]).shape[1] != self.query_rank or dq.shape[0] != self.query_rank:
            raise ValueError("latent_cache_attention: the two halves of the query projection disagree on its latent's size")
        uq, uk, uv, o = f64("uq").view(H, D, -1), f64("uk").view(H, D, L), f64("uv").view(H, Dv, L), f64("o").view(-1, H, Dv)
        # queries into the latent's space: rows h L .. (h + 1) L are W_uk[h]^T W_uq[h]
        q_fold = torch.einsum("hdl,hdq->hlq", uk, uq).reshape(H * L, -1)
        self.w_q = ops.tile_weight(self._to_device(q_fold))
        # and the heads' sums over the latents back out: columns h L .. (h + 1) L are W_o[:, h] W_uv[h]
        o_fold = torch.einsum("whv,hvl->whl", o, uv).reshape(-1, H * L)
        self.dq_norm_w = self._to_device(get(w["dq_norm"]), torch.float32)
        rows = [dq]
        if self.own_latent:
            rows.append(get(w["dkv"]))
            self.dkv_norm_w = self._to_device(get(w["dkv_norm"]), torch.float32)
        if self.has_sink:
            self.sink_w = self._to_device(get(w["sink"]), torch.float32)
        return torch.cat([self._to_device(t) for t in rows], dim=0).contiguous(), self._to_device(o_fold)

    def run(self, proj, col0, ctx, cache, out, out_col0, scale):
        if cache.writes != self.own_latent:
            raise ValueError("latent_cache_attention: a layer with a latent of its own writes its cache slot, one without reads another's")
        n = proj.shape[0]
        if cache.writes:
            c = ops.rmsnorm_cols(proj, col0 + self.query_rank, self.latent_dim, self.dkv_norm_w, self.norm_eps, cache.k.dtype)
            ops.vector_store(c, ctx.slot_mapping[cache.group], cache.k, cache.v)
        cq = ops.rmsnorm_cols(proj, col0, self.query_rank, self.dq_norm_w, self.norm_eps, self.dtype)
        q = ops.linear(cq, self.w_q, self.dtype).view(n, self.num_heads, self.latent_dim)
        a = ops.paged_attention(q, cache.k, cache.v, ctx.block_tables[cache.group], ctx.cu_seqlens, ctx.context_lens, ctx.token_req,
                                self.scale, int(self.window or 0), ctx.max_q_len, ctx.max_context_len, ctx.num_single, sink=self.sink_w)
        ops.sigmoid_gate(a, None, 0, scale, out, out_col0)


register_part("mixer", "latent_cache_attention", LatentCacheAttention)


class RotaryLatentAttention(BranchMixer):
    """Softmax attention over one cached latent a token (as ``LatentCacheAttention``) beside a rotated key part that all
    heads share.  With H = ``num_heads``, per head D = ``head_dim`` unrotated and R = ``rotary_dim`` rotated query/key
    elements, values of Dv = ``value_dim`` and a latent of L = ``latent_dim``:

        q = W_q x, per head [D unrotated | R rotated]      (no latent of the queries' own)
        W_dkv x has L + R rows: c = rmsnorm(rows 0 .. L - 1) * w_dkv; rows L .. L + R - 1 stay unnormed and, turned, end every head's key
        k_h = W_uk[h] c    v_h = W_uv[h] c    score = (q_plain . k_h + q_rot . k_rot) * ``scale``

    causal, or under a ``window``; ``gate: "head"`` multiplies head h's output by sigmoid(W_g x)_h; then W_o on the
    concatenated heads.  The position part turns the R rotated elements.

    Only c and the rotated part are cached: keys [R rotated | L latent] of one head, values [L latent], both with zeros
    behind up to a pair of sizes that the matrix-core attention kernels take (bfloat16).  The attention itself is one shared
    key/value head over the latents, q_plain . (W_uk[h] c) = (W_uk[h]^T q_plain) . c and sum_j p_j W_uv[h] c_j =
    W_uv[h] sum_j p_j c_j, so a step expands nothing of what it reads.  The two maps run in one of two ways:

    * ``folded`` into the ends, formed once at load in float64: the queries' rows are W_uk[h]^T W_q[h, :D] (L a head,
      beside the R rotated ones), the output's columns W_o[:, h] W_uv[h].  No more launches; a head's gate is one number,
      so it may multiply the sum over the latents;
    * as a product per head each (``ops.head_linear``, bfloat16): W_uk[h]^T on the projection's plain queries, straight
      into the attention's rows, and W_uv[h] with the gate on the attention's outputs.  With latents wider than the heads
      this is less arithmetic and far fewer weight bytes: per token H L (D + Dv) + H (D + Dv) hidden multiply-adds against
      2 H L hidden.

    The part takes whichever has fewer multiply-adds among those whose sizes fit (float32: folded).

    The columns of its input product are [q | latent | rotated key part | gate]; it keeps no per-request state."""

    def __init__(self, spec, hidden_size, dtype, device):
        super().__init__(spec, hidden_size, dtype, device)
        p = spec.params
        self.num_heads = int(p["num_heads"])
        self.head_dim = int(p["head_dim"])
        self.rotary_dim = int(p["rotary_dim"])
        self.value_dim = int(p["value_dim"])
        self.latent_dim = int(p["latent_dim"])
        self.scale = float(p["scale"])
        self.norm_eps = float(p["norm_eps"])
        self.window = p.get("window")
        gate = p.get("gate")
        if gate not in (None, "head"):
            raise ValueError(f"rotary_latent_attention: gate {gate!r} unknown (known: head)")
        self.gate = gate == "head"
        self.position = build_part("position", p["position"], hidden_size, dtype, device)
        rot = self.position.rotary()
        if (rot[1] if rot is not None else 0) != self.rotary_dim:
            raise ValueError("rotary_latent_attention: the position part must turn exactly the rotated elements")
        if self.rotary_dim <= 0 or self.rotary_dim % 2 != 0 or self.latent_dim % 2 != 0:
            raise ValueError("rotary_latent_attention: rotary_dim and latent_dim must be positive and even")
        key = self.rotary_dim + self.latent_dim
        pair = ops.fast_pair(key, self.latent_dim, exact_values=False) if dtype == torch.bfloat16 else None
        #: sizes of a cached key and of a cached value
        self.cached_key, self.cached_value = pair if pair is not None else (key, self.latent_dim)
        H, D, Dv, L = self.num_heads, self.head_dim, self.value_dim, self.latent_dim
        self.folded = not (ops.head_linear_ok(L, D, dtype) and ops.head_linear_ok(Dv, self.cached_value, dtype) and self.rotary_dim % 4 == 0
                           and L * (D + Dv) + (D + Dv) * hidden_size < 2 * L * hidden_size)
        self.q_cols = H * (key if self.folded else D + self.rotary_dim)
        self.inner = H * (self.cached_value if self.folded else Dv)

    @classmethod
    def expected_weights(cls, spec, hidden_size):
        p, w = spec.params, spec.weights
        H, D, R, Dv, L = (int(p[k]) for k in ("num_heads", "head_dim", "rotary_dim", "value_dim", "latent_dim"))
        out = {w["q"]: WeightInfo((H * (D + R), hidden_size)), w["dkv"]: WeightInfo((L + R, hidden_size)), w["dkv_norm"]: WeightInfo((L,), "ones"),
               w["uk"]: WeightInfo((H * D, L)), w["uv"]: WeightInfo((H * Dv, L)), w["o"]: WeightInfo((hidden_size, H * Dv))}
        if p.get("gate") is not None:
            out[w["gate"]] = WeightInfo((H, hidden_size))
        out.update(part_class("position", p["position"].kind).expected_weights(p["position"], hidden_size))
        return out

    def cache_spec(self):
        kind = "window" if self.window is not None else "full"
        if self.cached_value == self.cached_key:
            return CacheSpec(kind, 1, self.cached_key, self.window)
        return SizedValueCacheSpec(kind, 1, self.cached_key, self.window, self.cached_value)

    def load_branch(self, get):
        w = self.spec.weights
        H, D, R, Dv, L = self.num_heads, self.head_dim, self.rotary_dim, self.value_dim, self.latent_dim
        f64 = lambda name: get(w[name]).to(torch.float64)
        order = paired_order(R, R, getattr(self.position, "layout", "halves"))
        pad = (0, self.cached_value - L)
        if self.folded:
            q, uk, uv, o = f64("q").view(H, D + R, -1), f64("uk").view(H, D, L), f64("uv").view(H, Dv, L), f64("o").view(-1, H, Dv)
            latent_q = torch.matmul(uk.transpose(1, 2).contiguous(), q[:, :D].contiguous())
            rot_q = reorder_heads(q[:, D:].reshape(H * R, -1), R, order).view(H, R, -1)
            rows = [self._to_device(torch.cat([rot_q, latent_q], dim=1).reshape(H * (R + L), -1))]
            # columns h V .. (h + 1) V, V the cached values' size: W_o[:, h] W_uv[h], zeros for the padding
            out = torch.matmul(o.transpose(0, 1).contiguous(), uv)                      # [H, hidden, L]
            out = torch.nn.functional.pad(out, pad).transpose(0, 1).reshape(-1, self.inner)
        else:
            q = get(w["q"]).view(H, D + R, -1)
            rot_q = reorder_heads(q[:, D:].reshape(H * R, -1), R, order).view(H, R, -1)
            rows = [self._to_device(torch.cat([q[:, :D], rot_q], dim=1).reshape(H * (D + R), -1))]
            self.w_uk = self._to_device(get(w["uk"]).view(H, D, L).transpose(1, 2))               # [H, L, D]
            self.w_uv = self._to_device(torch.nn.functional.pad(get(w["uv"]).view(H, Dv, L), pad))     # [H, Dv, V]
            out = get(w["o"])
        dkv = get(w["dkv"])
        rows.append(self._to_device(torch.cat([dkv[:L], reorder_heads(dkv[L:], R, order)], dim=0)))
        if self.gate:
            rows.append(self._to_device(get(w["gate"])))
        self.latent_norm_w = self._to_device(get(w["dkv_norm"]), torch.float32)
        self.position.load_weights(get)
        return torch.cat(rows, dim=0).contiguous(), self._to_device(out)

    def run(self, proj, col0, ctx, cache, out, out_col0, scale):
        if not cache.writes:
            raise ValueError("rotary_latent_attention: a call that reads another call's cache is not supported")
        rot = self.position.rotary()
        inv_freq, _, factor = rot if rot is not None else (None, 0, 1.0)
        table = self.position.table(ctx) if hasattr(self.position, "table") else None
        d_col0 = col0 + self.q_cols
        q = ops.latent_rows_write(proj, col0, d_col0, self.latent_norm_w, self.norm_eps, ctx.positions, ctx.slot_mapping[cache.group],
                                  inv_freq, factor, self.num_heads, self.rotary_dim, self.latent_dim, cache.k, cache.v, table,
                                  None if self.folded else self.head_dim)
        n, gate_col0 = proj.shape[0], d_col0 + self.latent_dim + self.rotary_dim
        if not self.folded:
            ops.head_linear(proj, col0, self.head_dim + self.rotary_dim, self.w_uk, q.view(n, -1), self.rotary_dim, self.cached_key)
        a = ops.paged_attention(q, cache.k, cache.v, ctx.block_tables[cache.group], ctx.cu_seqlens, ctx.context_lens, ctx.token_req,
                                self.scale, int(self.window or 0), ctx.max_q_len, ctx.max_context_len, ctx.num_single)
        if not self.folded:
            ops.head_linear(a, 0, self.cached_value, self.w_uv, out, out_col0, self.value_dim, proj if self.gate else None, gate_col0, scale)
            return
        ops.sigmoid_gate(a, proj if self.gate else None, gate_col0, scale, out, out_col0, self.cached_value if self.gate else 1)


register_part("mixer", "rotary_latent_attention", RotaryLatentAttention)
