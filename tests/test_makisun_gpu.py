"""The Makisun design on the GPU: every new or changed kernel alone against its plain PyTorch version
(tests/emu_ops.py), and the model through the engine's own step function, cache manager, graphs and scheduler against
the plain implementation (tests/plain_makisun.py), in float32 and bfloat16."""
import copy
import json

import pytest
import torch

import helpers
import makisun_cases as cases
import plain_makisun as plain
from emu_ops import EmuOps

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
# plain.logit_error of a whole model: the largest difference of any logit, in units of the logits' spread.
TOL = {"float32": 1e-4}
# Models with sharpened queries amplify float32 rounding (scores of several tens); a key that is lost or wrongly seen
# costs at least 0.05 there (each such test asserts that first), 25 times this bound.
SHARP_TOL = 2e-3
emu = EmuOps()


def _ops():
    from tempura_amd.kernels import ops
    return ops


def _assert_logits(got, ref, dtype, what):
    """float32: every logit within TOL.  bfloat16: a bound on the distribution of the positions' errors (the median and
    the worst): the rounding of stored activations moves single positions more than the typical one."""
    if dtype == "float32":
        err = plain.logit_error(got, ref)
        assert err < TOL[dtype], f"{what}: error {err:.3e}"
        return
    g, r = got.double().cpu(), ref.double()
    d = (g - g.mean(-1, keepdim=True)) - (r - r.mean(-1, keepdim=True))
    per = (d.abs().max(-1).values / r.std()).sort().values
    n = per.numel()
    assert float(per[n // 2]) < 0.15 and float(per[-1]) < 0.6, f"{what}: median {float(per[n // 2]):.3f}, worst {float(per[-1]):.3f}"


class _Folders:
    """Model folders by case; in bfloat16 every expert is used by every token (no choice for a rounding to flip)."""

    def __init__(self, root):
        self.root = root

    def get(self, name, dtype="float32"):
        folder = self.root / f"{name}_{dtype}"
        if not folder.exists():
            cases.write_model(name, str(folder), config=_config(name, dtype))
        return str(folder)


def _config(name, dtype):
    return cases.config_json(name, every_expert=dtype == "bfloat16")


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    return _Folders(tmp_path_factory.mktemp("makisun_gpu"))


def _close(got, want, tol):
    got, want = got.double().cpu(), want.double().cpu()
    assert got.shape == want.shape
    err = float((got - want).abs().max() / max(1e-30, float(want.abs().max())))
    assert err <= tol, f"relative error {err:.3e} > {tol:.1e}"


def _dev(*ts):
    return [None if t is None else t.to(DEV) for t in ts]


def _batch(runs):
    """cu_seqlens and token_req of a batch of runs."""
    cu = torch.tensor([0] + list(torch.tensor(runs).cumsum(0)), dtype=torch.int32)
    return cu, torch.tensor([i for i, l in enumerate(runs) for _ in range(l)], dtype=torch.int32)


# ---- kernels alone ------------------------------------------------------------------------------
@pytest.mark.parametrize("H,D,E", [(2, 64, 64), (3, 7, 5), (1, 1, 1), (2, 16, 130), (4, 33, 20), (2, 40, 40), (1, 128, 128), (2, 128, 40), (1, 130, 33),
                                   (1, 256, 64), (1, 300, 12), (1, 1000, 3), (5, 8, 300), (2, 64, 32)])
@pytest.mark.parametrize("with_bonus", [False, True])
def test_linear_recurrence(H, D, E, with_bonus):
    """Three steps of unequal runs (long ones in pieces beside single tokens) that carry the state, from columns of wider
    rows, slots in any order, with and without the bonus; then one step of single tokens."""
    ops = _ops()
    g = torch.Generator().manual_seed(H * 1000 + D + E)
    R, off, slots_n = 4, 3, 6
    hd, he = H * D, H * E
    state = torch.zeros(slots_n, off + hd * E + 2)
    state_d = state.clone().to(DEV)
    slots = torch.tensor([4, 1, 0, 5], dtype=torch.int32)
    bonus = torch.randn(hd, generator=g) if with_bonus else None
    for runs in ([1, 70, 3, 17], [200, 1, 1, 64], [1, 1, 1, 1], [2, 33, 129, 5]):
        n = sum(runs)
        cu, _ = _batch(runs)
        qk, v = torch.randn(n, 2 * hd + 5, generator=g), torch.randn(n, he + 3, generator=g)
        decay = torch.sigmoid(torch.randn(n, hd, generator=g) * 2 + 2)
        want = emu.linear_scan((qk, 1), (qk, hd + 4), (v, 2), decay, state, off, cu, slots, R, H, D, E, bonus, 0.7)
        qd, vd, wd, cd, sd, bd = _dev(qk, v, decay, cu, slots, bonus)
        got = ops.linear_scan((qd, 1), (qd, hd + 4), (vd, 2), wd, state_d, off, cd, sd, R, H, D, E, bd, 0.7, max(runs))
        _close(got, want, 2e-5)
        _close(state_d, state, 2e-5)
    assert float(state_d[2].abs().max()) == 0.0 and float(state_d[:, :off].abs().max()) == 0.0      # (nobody else's row)


def test_pieces_of_a_run_change_rounding_only():
    """One run of 1,000 tokens in pieces of several lengths, uncut, and token by token: the same read-outs and state."""
    ops = _ops()
    g = torch.Generator().manual_seed(5)
    H, D, E, n = 3, 64, 64, 1000
    rows = torch.randn(n, H * (2 * D + E), generator=g).to(DEV)
    decay = torch.exp(-torch.exp(torch.randn(n, H * D, generator=g) * 1.5 - 3)).to(DEV)
    bonus = torch.randn(H * D, generator=g).to(DEV)
    cu, slots = _dev(torch.tensor([0, n], dtype=torch.int32), torch.zeros(1, dtype=torch.int32))

    def run(cuts):
        state, out = torch.zeros(1, H * D * E, device=DEV), []
        for a, b in zip(cuts[:-1], cuts[1:]):
            x = rows[a:b].contiguous()
            c = torch.tensor([0, b - a], dtype=torch.int32, device=DEV)
            out.append(ops.linear_scan((x, 0), (x, H * D), (x, 2 * H * D), decay[a:b].contiguous(), state, 0, c, slots, 1, H, D, E, bonus, 1.0, b - a))
        return torch.cat(out), state
    keep = ops.scan_min_piece, ops.scan_target_blocks
    try:
        ops.scan_min_piece = 2000
        ref = run([0, n])
        assert ops.scan_piece(n, n, H, D, E) == 0
        ops.scan_target_blocks = 1 << 30
        for piece in (16, 48, 64, 496, 512):
            ops.scan_min_piece = piece
            assert ops.scan_piece(n, n, H, D, E) == piece
            for got, want in zip(run([0, n]), ref):
                _close(got, want, 2e-5)
        for got, want in zip(run([0, 2, 501, 503, 700, 999, 1000]), ref):
            _close(got, want, 2e-5)
    finally:
        ops.scan_min_piece, ops.scan_target_blocks = keep
    few = run(list(range(0, 41)))[0]
    _close(few, ref[0][:40], 2e-5)


@pytest.mark.parametrize("width", [48, 32, 7, 130, 256, 1024, 4096])
@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
def test_mixes_with_the_row_before(width, out_dtype):
    ops = _ops()
    g = torch.Generator().manual_seed(width)
    off, mixes = 5, 5
    state = torch.randn(5, off + width + 1, generator=g)
    state_d = state.clone().to(DEV)
    mu = torch.rand(mixes, width, generator=g)
    slots = torch.tensor([3, 0, 4], dtype=torch.int32)
    for runs in ([5, 1, 12], [1, 1, 1], [1, 2, 40], [1, 1, 1]):
        cu, tr = _batch(runs)
        x = torch.randn(sum(runs), width, generator=g)
        want = emu.token_shift(x, mu, state, off, cu, tr, slots, 3, out_dtype)
        xd, md, cd, td, sd = _dev(x, mu, cu, tr, slots)
        got = ops.token_shift(xd, md, state_d, off, cd, td, sd, 3, out_dtype, max(runs))
        assert len(got) == mixes
        for a, b in zip(got, want):
            _close(a, b, 1e-6 if out_dtype == torch.float32 else 8e-3)
        assert torch.equal(state_d.cpu(), state)


@pytest.mark.parametrize("n", [1, 8, 9, 64, 65, 300])
@pytest.mark.parametrize("rank,cols", [(1, 5), (16, 208), (64, 130), (100, 1000), (3, 64)])
def test_decays_of_low_rank_projections(rank, cols, n):
    """Every function of the second product, at the row counts of both kernels."""
    ops = _ops()
    g = torch.Generator().manual_seed(rank + cols)
    x = torch.randn(n, rank + 7, generator=g) * 2
    wt = torch.randn(rank, cols, generator=g) * rank ** -0.5
    bias, a_log = torch.randn(cols, generator=g) - 1.0, torch.randn(cols, generator=g)
    xd, wd, bd, ad = _dev(x, wt, bias, a_log)
    for mode, kw in (("exp_exp", {"in_act": "tanh"}), ("root_sigmoid", {"rate": 1.0 / 16.0}), ("root_sigmoid", {"rate": 1.0}), ("exp_exp", {}), ("plain", {}),
                     ("sigmoid", {"in_act": "tanh"}), ("rate_sigmoid", {"rate": 0.6}), ("decay", {"per_head": 1})):
        want = emu.lowrank_up(x, 4, wt, mode, a_log, bias, kw.get("per_head", 0), kw.get("rate", 0.0), kw.get("in_act"))
        got = ops.lowrank_up(xd, 4, wd, mode, ad, bd, kw.get("per_head", 0), kw.get("rate", 0.0), kw.get("in_act"))
        _close(got, want, 1e-5)


@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [1, 37])
@pytest.mark.parametrize("H,E,col0,shared", [(3, 10, 0, False), (4, 64, 8, False), (2, 128, 4, True), (5, 3, 1, True), (1, 260, 0, False), (8, 32, 4, True)])
def test_norm_per_head_with_a_gate(H, E, col0, shared, n, out_dtype):
    ops = _ops()
    g = torch.Generator().manual_seed(H * E)
    o = torch.randn(n, H * E, generator=g) * 3
    w = torch.randn(E if shared else H * E, generator=g)
    rows = torch.randn(n, H * E + 12, generator=g)
    for act in ("silu", "sigmoid"):
        want = torch.zeros(n, col0 + H * E + 4, dtype=out_dtype)
        got = want.clone().to(DEV)
        emu.head_norm_gate(o, w, None, 1e-5, 0.8, H, want, col0, rows, 8, act)
        od, wd, rd = _dev(o, w, rows)
        ops.head_norm_gate(od, wd, None, 1e-5, 0.8, H, got, col0, rd, 8, act)
        _close(got, want, 1e-5 if out_dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [48, 1024, 1028, 4096, 9000])
def test_scaled_and_added(width, out_dtype):
    """The closing kernel without the norm on the sublayer's result: with and without the next norm, with a gate."""
    ops = _ops()
    g = torch.Generator().manual_seed(width)
    n = 9
    h, y = torch.randn(n, width, generator=g), torch.randn(n, width, generator=g)
    w, nw = torch.randn(width, generator=g), torch.randn(width, generator=g)
    rows, bias = torch.randn(n, width + 8, generator=g), torch.randn(width, generator=g)
    for next_w in (None, nw):
        for gate in (None, rows):
            mine, theirs = h.clone(), h.clone().to(DEV)
            want = emu.scale_add(mine, y, w, next_w, 1e-5, out_dtype, gate, 4, bias if gate is not None else None)
            yd, wd, nd, gd, bd = _dev(y, w, next_w, gate, bias if gate is not None else None)
            got = ops.scale_add(theirs, yd, wd, nd, 1e-5, out_dtype, gd, 4, bd)
            _close(theirs, mine, 2e-6)
            assert (got is None) == (want is None)
            if want is not None:
                _close(got, want, 2e-5 if out_dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [1, 37, 300])
@pytest.mark.parametrize("H,G,D,E,rot,pad,col0", [(4, 2, 12, 10, 8, 12, 0), (3, 3, 6, 6, 2, 6, 2), (6, 2, 64, 32, 64, 64, 12), (2, 1, 48, 128, 24, 128, 3),
                                                (16, 4, 128, 128, 128, 128, 0), (1, 1, 10, 200, 0, 10, 1), (2, 2, 96, 128, 64, 128, 4)])
def test_rows_into_queries_and_cache_with_a_norm_per_head(H, G, D, E, rot, pad, col0, n, dtype):
    """Norm per head, rotation of part of a head and the store, with and without the norm and biases, from columns that do
    not start at zero; with the angles computed and from a table."""
    ops = _ops()
    g = torch.Generator().manual_seed(H * 100 + D + n)
    ps = 16
    pages = (n + ps - 1) // ps + 3
    widths = (H * D, G * D, G * E)
    extra = 6 + (col0 + sum(widths)) % 2
    rows = torch.randn(n, col0 + sum(widths) + extra, generator=g) * 3
    order = torch.randperm(pages, generator=g)
    slots = (order[:, None] * ps + torch.arange(ps)[None, :]).reshape(-1)[3: 3 + n].to(torch.int32)
    positions = torch.randint(0, 5000, (n,), generator=g).to(torch.int32)
    norms = (torch.randn(D, generator=g), torch.randn(D, generator=g))
    biases = tuple(torch.randn(w, generator=g) for w in widths)
    f = torch.pow(torch.tensor(5000.0, dtype=torch.float64), -2.0 * torch.arange(rot // 2, dtype=torch.float64) / max(rot, 1)) if rot else None
    tol = 2e-5 if dtype == torch.float32 else 8e-3
    for nw, bs in ((norms, (None,) * 3), (None, (None,) * 3), (norms, biases)):
        k, v = torch.randn(pages, G, ps, pad, generator=g).to(dtype), torch.randn(pages, G, E, ps, generator=g).to(dtype)
        kd, vd = _dev(k, v)
        want = emu.qkv_rows(rows, positions, slots, H, G, D, E, k, v, f, rot, 1.0, bs, nw, 1e-5, None, pad, col0, "head")
        rd, pd, sd, fd = _dev(rows, positions, slots, f)
        for table in [None] + ([ops.rope_table(pd, fd, rot, 1.0)] if n >= 256 and rot else []):
            got = ops.qkv_rows(rd, pd, sd, H, G, D, E, kd, vd, fd, rot, 1.0, table, tuple(_dev(*bs)), None if nw is None else tuple(_dev(*nw)), 1e-5,
                               None, None, pad, col0, "head")
            assert got.dtype == dtype
            _close(got, want, tol)
            _close(kd, k, tol)
            _close(vd, v, tol)
        if pad > D:
            assert float(got[..., D:].abs().max()) == 0.0


@pytest.mark.parametrize("m", [1, 3, 8, 16])
@pytest.mark.parametrize("k,sizes", [(64, (16, 32, 16)), (128, (48,)), (256, (16, 16, 32, 64, 16)), (1088, (64, 128, 16, 16)), (4096, (256, 256, 64)),
                                     (192, (16,) * 8)])
def test_products_in_groups(m, k, sizes):
    """Every group's rows times its own weight, in one launch; a row's result does not depend on the other rows."""
    ops = _ops()
    g = torch.Generator().manual_seed(m * 10 + k)
    n = sum(sizes)
    w = (torch.randn(n, k, generator=g) * k ** -0.5).to(torch.bfloat16).to(DEV)
    x = torch.randn(len(sizes), m, k, generator=g).to(torch.bfloat16).to(DEV)
    blocked = x.reshape(len(sizes), m, k // 8, 8).transpose(1, 2).contiguous()
    ends = torch.tensor(sizes).cumsum(0).tolist()
    tiled = ops.tile_weight(w)
    assert ops.group_linear_ok(m, tiled)
    got = ops.group_linear(blocked, tiled, ends)
    want = torch.cat([x[i].float() @ w[e - c: e].float().T for i, (c, e) in enumerate(zip(sizes, ends))], dim=1)
    _close(got, want, 2e-5)
    alone = ops.group_linear(blocked[:, :, :1].contiguous(), tiled, ends)
    assert torch.equal(alone, got[:1])


@pytest.mark.parametrize("m", [1, 2, 8, 16])
@pytest.mark.parametrize("E,top,ff,k,n", [(4, 1, 64, 64, 32), (8, 2, 128, 128, 48), (16, 3, 192, 64, 64), (100, 4, 64, 128, 16), (3, 3, 640, 256, 128), (8, 2, 1088, 512, 256),
                                          (1, 1, 64, 64, 16)])
@pytest.mark.parametrize("activation", ["relu2", "gelu_erf", "gelu_tanh", "silu", None])
def test_routed_experts_of_a_few_rows(m, E, top, ff, k, n, activation):
    """Ungated and gated experts, some used by no row, into a new tensor and added to another; a row's result has the
    same bits alone and beside rows that use other experts."""
    ops = _ops()
    g = torch.Generator().manual_seed(E * 100 + m + ff)
    bf = lambda *s, std=1.0: (torch.randn(*s, generator=g) * std).to(torch.bfloat16).to(DEV)
    up, down = bf(E, ff, k, std=k ** -0.5), bf(E, n, ff, std=ff ** -0.5)
    gate = bf(E, ff, k, std=k ** -0.5)
    x = bf(m, k)
    dense = torch.zeros(m, E)
    for t in range(m):
        dense[t, torch.randperm(E, generator=g)[:top]] = torch.rand(top, generator=g) + 0.1
    dense = dense.to(DEV)
    rows = up if activation is not None else torch.stack([ops.interleave_gate_up(gate[e], up[e]) for e in range(E)])
    w_up = ops.tile_weight(rows.reshape(-1, k).contiguous())
    w_down = ops.tile_weight(down.reshape(-1, ff).contiguous())
    assert ops.moe_few_ok(m, E, ff, w_up, w_down)
    xd, want = x.double(), torch.zeros(m, n, dtype=torch.float64, device=DEV)
    for e in range(E):
        u = xd @ up[e].double().T
        a = u * torch.nn.functional.silu(xd @ gate[e].double().T) if activation is None else emu.activation(u.cpu(), activation, torch.float64).to(DEV)
        want += ((a * dense[:, e:e + 1].double()).to(torch.bfloat16).double()) @ down[e].double().T
    got = ops.moe_few(ops.block_rows(x), w_up, w_down, dense, ff, activation)
    _close(got, want, 6e-3)
    y = torch.randn(m, n, generator=g).to(DEV)
    more = ops.moe_few(ops.block_rows(x), w_up, w_down, dense, ff, activation, y.clone())
    _close(more, want + y.double(), 6e-3)
    alone = ops.moe_few(ops.block_rows(x[-1:].contiguous()), w_up, w_down, dense[-1:].contiguous(), ff, activation)
    assert torch.equal(alone, got[-1:])


@pytest.mark.parametrize("m", [1, 7, 16])
def test_rows_that_leave_k_blocked(m):
    """The closing kernel, the mixes, activations and the up product with the squared ReLU: k-blocked rows hold the bits of
    the plain ones, in and out."""
    ops = _ops()
    g = torch.Generator().manual_seed(m)
    for width in (64, 128, 1024, 4096):
        h, y = torch.randn(m, width, generator=g).to(DEV), torch.randn(m, width, generator=g).to(DEV)
        w, nw = torch.rand(width, generator=g).to(DEV), torch.rand(width, generator=g).to(DEV)
        for op in (lambda h, **kw: ops.scale_add(h, y, w, nw, 1e-5, torch.bfloat16, **kw), lambda h, **kw: ops.norm_add(h, y, w, 1e-5, nw, 1e-5, torch.bfloat16, **kw)):
            plain_rows, blocked = op(h.clone()), op(h.clone(), blocked=True)
            assert isinstance(blocked, ops.KBlocked) and torch.equal(blocked.row_major(), plain_rows)
        assert torch.equal(ops.block_rows(plain_rows).row_major(), plain_rows)
        for kind in ("gelu_erf", "relu2"):
            assert torch.equal(ops.activation(h, kind, torch.bfloat16, blocked=True).row_major(), ops.activation(h, kind, torch.bfloat16))
        wt = ops.tile_weight((torch.randn(256, width, generator=g) * width ** -0.5).to(torch.bfloat16).to(DEV))
        a, side = ops.linear_relu2(plain_rows, wt, 128)
        b, side2 = ops.linear_relu2(blocked, wt, 128)
        _close(b, a.float(), 8e-3)
        _close(side2, side, 2e-5)
        cu, tr = _dev(*_batch([1] * m))
        slots = torch.arange(m, dtype=torch.int32, device=DEV)
        mu, state = torch.rand(5, width, generator=g).to(DEV), torch.randn(m, width, generator=g).to(DEV)
        shift = lambda **kw: ops.token_shift(h, mu, state.clone(), 0, cu, tr, slots, m, torch.bfloat16, 1, **kw)
        rows, stacked = shift(), shift(blocked=True)
        for i in range(5):
            assert torch.equal(ops.KBlocked(stacked[i], m, width).row_major(), rows[i])


def test_sizes_the_kernels_do_not_take_are_refused():
    ops = _ops()
    z = lambda *s: torch.zeros(*s, device=DEV)
    i32 = lambda *x: torch.tensor(x, dtype=torch.int32, device=DEV)
    with pytest.raises(ops.KernelError, match="state rows too short"):
        ops.linear_scan((z(2, 8), 0), (z(2, 8), 0), (z(2, 8), 0), z(2, 8), z(1, 31), 0, i32(0, 2), i32(0), 1, 2, 4, 4)
    with pytest.raises(ops.KernelError, match="bad v rows"):
        ops.linear_scan((z(2, 8), 0), (z(2, 8), 0), (z(2, 8), 4), z(2, 8), z(1, 32), 0, i32(0, 2), i32(0), 1, 2, 4, 4)
    with pytest.raises(ops.KernelError, match="key size 1028"):
        ops.linear_scan((z(1, 1028), 0), (z(1, 1028), 0), (z(1, 1), 0), z(1, 1028), z(1, 1028), 0, i32(0, 1), i32(0), 1, 1, 1028, 1)
    with pytest.raises(ops.KernelError, match="not 1 runs of one"):
        ops.token_shift(z(2, 8), z(5, 8), z(1, 8), 0, i32(0, 2), i32(0, 0), i32(0), 1, torch.float32, 1)
    with pytest.raises(ops.KernelError, match="q norm must be"):
        ops.qkv_rows(z(1, 48), i32(0), i32(0), 1, 1, 16, 16, z(1, 1, 16, 16), z(1, 1, 16, 16), norms=(z(8), z(8)), norm_over="head")
    w = ops.tile_weight(torch.zeros(32, 64, dtype=torch.bfloat16, device=DEV))
    with pytest.raises(ops.KernelError, match="disagree"):
        ops.group_linear(torch.zeros(2, 8, 1, 8, dtype=torch.bfloat16, device=DEV), w, [16, 48])
    with pytest.raises(ops.KernelError, match="group borders"):
        ops.group_linear(torch.zeros(2, 8, 1, 8, dtype=torch.bfloat16, device=DEV), w, [8, 32])
    assert not ops.group_linear_ok(17, w)
    with pytest.raises(ops.KernelError, match="disagree"):
        ops.moe_few(ops.block_rows(torch.zeros(1, 64, dtype=torch.bfloat16, device=DEV)), w, w, z(1, 2), 64, "relu2")
    with pytest.raises(ops.KernelError, match="decay biases"):
        ops.lowrank_up(z(1, 4), 0, z(4, 8), "exp_exp")


# ---- the model through the step function --------------------------------------------------------
def _runner(folder, dtype, max_tokens, page_size=16, max_requests=4, use_graph=False):
    from tempura_amd.engine.loading import load_model
    from tempura_amd.engine.runner import ModelRunner
    model = load_model(folder, dtype, DEV)
    return ModelRunner(model, page_size, (max_tokens + page_size - 1) // page_size, max_requests=max_requests, use_graph=use_graph)


_REFS = {}


def _ref(name, rid, dtype):
    if (name, rid, dtype) not in _REFS:
        _REFS[(name, rid, dtype)] = plain.forward(_config(name, dtype), cases.make_weights(name), cases.requests(name)[rid])
    return _REFS[(name, rid, dtype)]


@pytest.mark.parametrize("name", ["mix", "one", "wide"])
def test_each_part_alone_matches_its_plain_function(dirs, name):
    import makisun_mechanisms
    makisun_mechanisms.check(dirs.get(name), name, DEV, 3e-5, cuts=(0, 21, 23, 110, 111))


@pytest.mark.parametrize("name", ["mix", "one", "wide"])
def test_each_part_alone_in_bfloat16(dirs, name):
    """The parts over the bfloat16 kernels (the matrix-core attention and the fused activation where they serve), every
    expert used."""
    import makisun_mechanisms
    makisun_mechanisms.check(dirs.get(name, "bfloat16"), name, DEV, 6e-2, dtype="bfloat16", cfg=_config(name, "bfloat16"))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mix", "one", "wide"])
@pytest.mark.parametrize("mode", ["whole", "bulk_tail", "portions", "mixed"])
def test_every_cutting_matches_plain(dirs, name, mode, dtype):
    reqs = cases.requests(name)
    lengths = cases.LENGTHS[name]
    if mode == "mixed":
        max_tokens = sum(sorted(helpers.roundup(n, 64) for n in lengths.values())[-2:]) + 64
        steps = helpers.schedule_mixed(lengths, max_tokens, seed=11)
    else:
        max_tokens = max(helpers.roundup(n, 64) for n in lengths.values())
        steps = {"whole": helpers.schedule_whole, "bulk_tail": lambda l: helpers.schedule_bulk_tail(l, tail=40),
                 "portions": lambda l: helpers.schedule_portions(l, sizes=(7, 2, 16, 3, 2, 31, 5, 2, 64, 9, 2, 17))}[mode](lengths)
    runner = _runner(dirs.get(name, dtype), dtype, max_tokens)
    got = helpers.run_schedule(runner, reqs, steps)
    for rid in reqs:
        _assert_logits(got[rid], _ref(name, rid, dtype), dtype, f"{name}/{mode}/{dtype}: request {rid}")
    assert not runner.cache.live_requests()
    assert runner.cache.free_pages() == [p.num_pages for p in runner.cache.pools]


def test_cutting_changes_rounding_only(dirs):
    """The same request whole, in portions and beside others, in float32: summation order only."""
    reqs = cases.requests("wide")
    lengths = cases.LENGTHS["wide"]
    runs = []
    for steps in (helpers.schedule_whole(lengths), helpers.schedule_portions(lengths, sizes=(2, 9, 33, 2, 16, 5)),
                  helpers.schedule_mixed(lengths, 512, seed=3)):
        runs.append(helpers.run_schedule(_runner(dirs.get("wide"), "float32", 512), reqs, steps))
    for rid in reqs:
        for other in runs[1:]:
            assert plain.logit_error(other[rid], runs[0][rid]) < 1e-4, rid


@pytest.mark.parametrize("window", [16, 33, 50])
def test_the_edges_of_the_window_on_the_gpu(tmp_path, window):
    """Queries many times larger than drawn (a softmax that rests on one or two keys): a prompt whole, then in portions that
    end at and beside page and window borders with decoding behind them.  The premise first: a window one longer or one
    shorter gives other logits."""
    from tempura_amd.engine.runner import StepEntry
    cfg = cases.config_json("wide")
    cfg["layers"] = [cfg["layers"][1], cfg["layers"][4]]
    cfg["layers"][0]["mixer"]["left"]["mask"] = {"size": window}
    W = cases.make_weights("wide", sharp=6.0, cfg=cfg)
    folder = cases.write_model("wide", str(tmp_path / "sharp"), weights=W, config=cfg)
    toks = cases.tokens("wide", 200, 5)
    ref = plain.forward(cfg, W, toks)
    for other in (window - 1, window + 1):
        c2 = copy.deepcopy(cfg)
        c2["layers"][0]["mixer"]["left"]["mask"]["size"] = other
        assert plain.logit_error(plain.forward(c2, W, toks), ref) > 0.05, other
    runner = _runner(folder, "float32", 256)
    runner.add_request("w")
    whole = runner.step([StepEntry("w", toks, list(range(200)))]).cpu()
    assert plain.logit_error(whole, ref) < SHARP_TOL
    runner.end_request("w")
    runner.add_request("r")
    rows, at = [], 0
    for c in (16, 15, 2, 31, 57, 40, 3):
        rows.append(runner.step([StepEntry("r", toks[at: at + c], list(range(c)))]).cpu())
        at += c
    rows += [runner.step([StepEntry("r", [t], [0])]).cpu() for t in toks[at:]]
    assert plain.logit_error(torch.cat(rows), ref) < SHARP_TOL


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_token_decides_on_the_gpu(tmp_path, dtype):
    """Slow decays over 450 tokens, so that the recurrences' pieces carry what far tokens left behind; portions cut anywhere,
    then decoding.  The premise first: the first tokens matter at the end."""
    from tempura_amd.engine.runner import StepEntry
    cfg = cases.config_json("wide", every_expert=dtype == "bfloat16")
    cfg["layers"] = [cfg["layers"][0], cfg["layers"][5], cfg["layers"][2]]
    W = cases.make_weights("wide", slow=5.0, cfg=cfg)
    folder = cases.write_model("wide", str(tmp_path / "far"), weights=W, config=cfg)
    toks = cases.tokens("wide", 450, 17)
    ref = plain.forward(cfg, W, toks)
    other = [(t + 1) % 96 for t in toks[:20]] + toks[20:]
    assert plain.logit_error(plain.forward(cfg, W, other)[-5:], ref[-5:]) > (0.05 if dtype == "float32" else 0.2)
    runner = _runner(folder, dtype, 512)
    runner.add_request("r")
    rows, at = [], 0
    for c in (130, 2, 161, 100, 7):
        rows.append(runner.step([StepEntry("r", toks[at: at + c], list(range(c)))]).cpu())
        at += c
    rows += [runner.step([StepEntry("r", [t], [0])]).cpu() for t in toks[at:]]
    _assert_logits(torch.cat(rows), ref, dtype, "far token")


@pytest.mark.parametrize("name,dtype", [("wide", "float32"), ("wide", "bfloat16"), ("mix", "float32")])
def test_long_decoding_through_a_captured_step(dirs, name, dtype):
    """Two requests decoded token by token for 150 steps through the graph path: pages, states and rows before move along."""
    from tempura_amd.engine.runner import StepEntry
    cfg, W = _config(name, dtype), cases.make_weights(name)
    runner = _runner(dirs.get(name, dtype), dtype, 512, use_graph=True)
    assert runner.use_graph, "every part of the design may be captured"
    seqs = {"p": cases.tokens(name, 170, 41), "q": cases.tokens(name, 158, 42)}
    start = {"p": 20, "q": 8}
    got = {rid: [] for rid in seqs}
    for rid in seqs:
        runner.add_request(rid)
        got[rid].append(runner.step([StepEntry(rid, seqs[rid][: start[rid]], list(range(start[rid])))]).cpu())
    for i in range(150):
        logits = runner.step([StepEntry(rid, [seqs[rid][start[rid] + i]], [0]) for rid in seqs]).cpu()
        for k, rid in enumerate(seqs):
            got[rid].append(logits[k: k + 1].clone())
    assert runner.graph_steps >= 149
    for rid in seqs:
        _assert_logits(torch.cat(got[rid]), plain.forward(cfg, W, seqs[rid]), dtype, f"captured {name} {dtype} {rid}")


def test_a_captured_step_gives_the_bits_of_the_eager_one(dirs):
    """Three requests (a graph of four rows, the fourth on the spare state row), bfloat16."""
    from tempura_amd.engine.runner import StepEntry
    runs = []
    for use_graph in (False, True):
        runner = _runner(dirs.get("wide", "bfloat16"), "bfloat16", 512, use_graph=use_graph)
        seqs = {r: cases.tokens("wide", 30 + 7 * i, 60 + i) for i, r in enumerate("abc")}
        out = []
        for r in seqs:
            runner.add_request(r)
            runner.step([StepEntry(r, seqs[r][:20], [])])
        for i in range(10):
            out.append(runner.step([StepEntry(r, [seqs[r][20 + i]], [0]) for r in seqs]).cpu().clone())
        runs.append(torch.stack(out))
    assert torch.equal(runs[0], runs[1])


@pytest.mark.parametrize("name", ["mix", "wide"])
@pytest.mark.parametrize("use_graph", [False, True])
def test_engine_generates_what_plain_greedy_generates(dirs, name, use_graph):
    from tempura_amd.engine import Engine
    from tempura_amd.sampling import SamplingParams
    cfg, W = cases.config_json(name), cases.make_weights(name)
    prompts = [cases.tokens(name, n, 20 + i) for i, n in enumerate((3, 18, 9, 40, 1))]
    eng = Engine(dirs.get(name), dtype="float32", page_size=16, kv_pages=24, max_batch_size=3, max_num_batched_tokens=32,
                 prefill_chunk_size=7, device=DEV, use_graph=use_graph)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=12))
    for p, o in zip(prompts, outs):
        assert o == plain.greedy(cfg, W, p, 12)
    if use_graph:
        assert eng.runner.graph_steps > 0


@pytest.mark.parametrize("kind", ["wkv", "parallel"])
def test_models_of_one_mixer_alone(tmp_path, kind):
    """Recurrences alone (a model that has no paged cache) and branches alone, captured steps included."""
    from tempura_amd.engine import Engine
    from tempura_amd.sampling import SamplingParams
    cfg = cases.config_json("wide")
    cfg["layers"] = [layer for layer in cfg["layers"] if layer["type"] == kind]
    W = cases.make_weights("wide", 3, cfg=cfg)
    eng = Engine(cases.write_model("wide", str(tmp_path / kind), weights=W, config=cfg), dtype="float32", page_size=16, kv_pages=40, max_batch_size=3,
                 max_num_batched_tokens=128, prefill_chunk_size=70, device=DEV, use_graph=True)
    prompts = [cases.tokens("wide", n, 40 + i) for i, n in enumerate((90, 2, 33, 8))]
    for p, o in zip(prompts, eng.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=8))):
        assert o == plain.greedy(cfg, W, p, 8)
    assert eng.runner.graph_steps > 0


def test_replay_program_on_a_model_folder(dirs, tmp_path):
    """bin/trace_run on a small folder: steps on standard input, logits files out, against the plain result."""
    import os
    import subprocess
    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    toks = cases.tokens("mix", 30, 5)
    out = tmp_path / "out"
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:11], "want": [0, 10]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[11:13], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[13:], "want": [16]}, {"id": "b", "tokens": toks[:4], "want": [3]}], "end": ["a", "b"]}]
    p = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", dirs.get("mix"), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    ref = plain.forward(cases.config_json("mix"), cases.make_weights("mix"), toks)
    vocab = ref.shape[1]
    a = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(-1, vocab))
    c = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(-1, vocab))
    assert plain.logit_error(torch.cat([a, c]), torch.stack([ref[0], ref[10], ref[29], ref[3]])) < TOL["float32"]
