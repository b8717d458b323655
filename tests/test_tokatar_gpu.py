"""The Tokatar design on the GPU: every new or changed kernel alone against its plain PyTorch version
(tests/emu_ops.py), and the model through the engine's own step function, cache manager, graphs and scheduler against
the plain implementation (tests/plain_tokatar.py), in float32 and bfloat16."""
import copy
import json

import pytest
import torch

import helpers
import plain_tokatar as plain
import tokatar_cases as cases
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


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("tokatar_gpu")
    return {name: cases.write_model(name, str(root / name)) for name in cases.CASES}


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


def _places(n, pages, ps, g, runs=False):
    """Distinct cache places: scattered, or mostly runs of neighbours from a multiple of eight on."""
    if not runs:
        return torch.randperm(pages * ps, generator=g)[:n].to(torch.int32)
    order = torch.randperm(pages, generator=g)
    flat = (order[:, None] * ps + torch.arange(ps)[None, :]).reshape(-1)
    return flat[3: 3 + n].to(torch.int32)


# ---- kernels alone ------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [1, 37, 300])
@pytest.mark.parametrize("H,G,D,E,rot,pad,extra", [(4, 2, 12, 10, 8, 12, 6), (3, 3, 6, 6, 2, 6, 0), (6, 2, 64, 32, 64, 64, 12), (2, 1, 48, 128, 24, 128, 4),
                                                 (16, 4, 128, 128, 128, 128, 20), (1, 1, 10, 200, 0, 10, 2)])
def test_rows_of_a_projection_into_queries_and_cache(H, G, D, E, rot, pad, extra, n, dtype):
    """Biases, the norm over the whole projection, both rotations and the store, each alone and together, at a handful of
    rows and at the row counts where values go sixteen tokens at a time; with the angles computed and from a table."""
    ops = _ops()
    g = torch.Generator().manual_seed(H * 100 + D + n)
    ps = 16
    pages = (n + ps - 1) // ps + 3
    widths = (H * D, G * D, G * E)
    rows = torch.randn(n, sum(widths) + extra, generator=g) * 3
    slots = _places(n, pages, ps, g, runs=n > 100)
    positions = torch.randint(0, 5000, (n,), generator=g).to(torch.int32)
    biases = tuple(torch.randn(w, generator=g) for w in widths)
    norms = tuple(torch.randn(w, generator=g) for w in widths[:2])
    f = torch.pow(torch.tensor(5000.0, dtype=torch.float64), -2.0 * torch.arange(rot // 2, dtype=torch.float64) / max(rot, 1)) if rot else None
    fv = torch.pow(torch.tensor(700.0, dtype=torch.float64), -2.0 * torch.arange(E // 2, dtype=torch.float64) / E)
    tol = 2e-5 if dtype == torch.float32 else 8e-3
    for bs, nw, vf in ((biases, norms, fv), ((None, None, None), norms, None), ((biases[0], None, biases[2]), None, fv), ((None,) * 3, None, None)):
        k, v = torch.randn(pages, G, ps, pad, generator=g).to(dtype), torch.randn(pages, G, E, ps, generator=g).to(dtype)
        kd, vd = _dev(k, v)
        want = emu.qkv_rows(rows, positions, slots, H, G, D, E, k, v, f, rot, 1.0, bs, nw, 1e-5, vf, pad)
        rd, pd, sd, fd, vfd = _dev(rows, positions, slots, f, vf)
        tables = [(None, None)]
        if n >= 256:
            tables.append((ops.rope_table(pd, fd, rot, 1.0) if rot else None, None if vf is None else ops.rope_table(pd, vfd, E, 1.0)))
        for table, vtable in tables:
            got = ops.qkv_rows(rd, pd, sd, H, G, D, E, kd, vd, fd, rot, 1.0, table, tuple(_dev(*bs)), None if nw is None else tuple(_dev(*nw)), 1e-5,
                               vfd, vtable, pad)
            assert got.dtype == dtype
            _close(got, want, tol)
            _close(kd, k, tol)
            _close(vd, v, tol)
        if pad > D:
            assert float(got[..., D:].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [1, 23, 270])
@pytest.mark.parametrize("H,R,L,key,value,col0", [(3, 4, 20, 24, 20, 0), (1, 12, 8, 20, 8, 2), (4, 32, 96, 128, 128, 8), (32, 64, 128, 192, 128, 0), (2, 6, 10, 32, 32, 0)])
def test_latent_rows_into_queries_and_cache(H, R, L, key, value, col0, n, dtype):
    """Queries with a rotated part beside a latent, the normed latent and the shared rotated part; padded key and value
    sizes; columns that do not start at zero."""
    ops = _ops()
    g = torch.Generator().manual_seed(H * 10 + L + n)
    ps = 16
    pages = (n + ps - 1) // ps + 2
    q_cols = H * (R + L)
    rows = torch.randn(n, col0 + q_cols + L + R + 4, generator=g) * 2
    w = torch.randn(L, generator=g)
    slots = _places(n, pages, ps, g)
    positions = torch.randint(0, 5000, (n,), generator=g).to(torch.int32)
    f = torch.pow(torch.tensor(900.0, dtype=torch.float64), -2.0 * torch.arange(R // 2, dtype=torch.float64) / R)
    k, v = torch.randn(pages, 1, ps, key, generator=g).to(dtype), torch.randn(pages, 1, value, ps, generator=g).to(dtype)
    kd, vd = _dev(k, v)
    want = emu.latent_rows_write(rows, col0, col0 + q_cols, w, 1e-5, positions, slots, f, 1.0, H, R, L, k, v)
    rd, wd, pd, sd, fd = _dev(rows, w, positions, slots, f)
    tol = 2e-5 if dtype == torch.float32 else 8e-3
    for table in (None, ops.rope_table(pd, fd, R, 1.0)):
        got = ops.latent_rows_write(rd, col0, col0 + q_cols, wd, 1e-5, pd, sd, fd, 1.0, H, R, L, kd, vd, table)
        _close(got, want, tol)
        _close(kd, k, tol)
        _close(vd, v, tol)


@pytest.mark.parametrize("n", [1, 30, 258])
def test_rotated_queries_whose_latent_part_comes_from_elsewhere(n):
    """The queries' rows hold [plain | rotated]: only the rotated part and the padding are written."""
    ops = _ops()
    g = torch.Generator().manual_seed(n)
    for H, D, R, L, key, value in ((4, 32, 32, 256, 288, 256), (3, 48, 8, 20, 32, 32), (2, 10, 6, 10, 16, 10)):
        rows = torch.randn(n, H * (D + R) + L + R + 6, generator=g)
        w = torch.randn(L, generator=g)
        pages = (n + 15) // 16 + 2
        slots = _places(n, pages, 16, g)
        positions = torch.randint(0, 3000, (n,), generator=g).to(torch.int32)
        f = torch.pow(torch.tensor(900.0, dtype=torch.float64), -2.0 * torch.arange(R // 2, dtype=torch.float64) / R)
        k, v = torch.zeros(pages, 1, 16, key, dtype=torch.bfloat16), torch.zeros(pages, 1, value, 16, dtype=torch.bfloat16)
        kd, vd = _dev(k, v)
        d_col0 = H * (D + R)
        want = emu.latent_rows_write(rows, 0, d_col0, w, 1e-5, positions, slots, f, 1.0, H, R, L, k, v, D)
        rd, wd, pd, sd, fd = _dev(rows, w, positions, slots, f)
        got = ops.latent_rows_write(rd, 0, d_col0, wd, 1e-5, pd, sd, fd, 1.0, H, R, L, kd, vd, None, D)
        _close(got[..., :R], want[..., :R], 8e-3)
        assert key == R + L or float(got[..., R + L:].abs().max()) == 0.0
        _close(kd, k, 8e-3)
        _close(vd, v, 8e-3)


@pytest.mark.parametrize("m", [1, 8, 17, 64, 65, 300, 1000])
@pytest.mark.parametrize("H,N,K", [(3, 16, 32), (4, 256, 32), (18, 512, 64), (5, 48, 256), (8, 128, 512), (2, 80, 96)])
def test_product_per_head(m, H, N, K):
    """Strided float32 and bfloat16 rows in, pieces of wider bfloat16 rows out, with and without a gate per head; nothing
    beside the pieces is touched."""
    ops = _ops()
    g = torch.Generator().manual_seed(H * N + K + m)
    w = (torch.randn(H, N, K, generator=g) * K ** -0.5).to(torch.bfloat16)
    x_head, out_head = K + 8, N + 4
    x = torch.randn(m, 8 + H * x_head + 8, generator=g)
    gate = torch.randn(m, 3 + H + 2, generator=g)
    for xt in (x, x.to(torch.bfloat16)):
        for gt in (None, gate):
            out = torch.full((m, 4 + H * out_head + 4), 7.0, dtype=torch.bfloat16)
            dev = out.to(DEV)
            emu.head_linear(xt, 8, x_head, w, out, 4, out_head, gt, 3, 1.5)
            ops.head_linear(xt.to(DEV), 8, x_head, w.to(DEV), dev, 4, out_head, None if gt is None else gt.to(DEV), 3, 1.5)
            _close(dev, out, 8e-3)
            same = torch.ones(out.shape[1], dtype=torch.bool)
            for h in range(H):
                same[4 + h * out_head: 4 + h * out_head + N] = False
            assert bool((dev.cpu()[:, same] == 7.0).all())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_outputs_turned_back_and_gated(dtype):
    ops = _ops()
    g = torch.Generator().manual_seed(5)
    for n, H, E, col0 in ((1, 3, 6, 2), (40, 2, 64, 0), (260, 4, 128, 8), (7, 1, 10, 5)):
        a = torch.randn(n, H * E, generator=g).to(dtype)
        gate = torch.randn(n, col0 + H * E + 4, generator=g) * 2
        positions = torch.randint(0, 9000, (n,), generator=g).to(torch.int32)
        f = torch.pow(torch.tensor(300.0, dtype=torch.float64), -2.0 * torch.arange(E // 2, dtype=torch.float64) / E)
        ad, gd, pd, fd = _dev(a, gate, positions, f)
        tol = 2e-6 if dtype == torch.float32 else 8e-3
        for rows in (gate, None):
            want = emu.turn_gate(a, positions, f, E, rows, col0)
            for table in (None, ops.rope_table(pd, fd, E, 1.0)):
                _close(ops.turn_gate(ad, pd, fd, E, gd if rows is not None else None, col0, table), want, tol)
        # turned by its position and back again: the value
        back = ops.turn_gate(ops.turn_gate(ad, -pd, fd, E), pd, fd, E)
        _close(back, a, 2e-6 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,col0", [(48, 3), (128, 4), (1024, 8), (1028, 2), (4096, 4096), (7168, 0), (9000, 1)])
def test_gated_norm_and_add(width, col0, out_dtype):
    """A sublayer's result times the sigmoid of gate rows, normed, scaled, added, and the stream normed for what follows."""
    ops = _ops()
    g = torch.Generator().manual_seed(width)
    n = 5
    h, y = torch.randn(n, width, generator=g) * 2, torch.randn(n, width, generator=g) * 3
    w, w2, b = (torch.randn(width, generator=g) for _ in range(3))
    gate = torch.randn(n, col0 + width + 4, generator=g) * 2
    hd, yd, wd, w2d, bd, gd = _dev(h, y, w, w2, b, gate)
    tol = 2e-6 if out_dtype == torch.float32 else 8e-3
    for bias, bias_d in ((b, bd), (None, None)):
        h_ref, h_dev = h.clone(), hd.clone()
        emu.norm_add(h_ref, y, w, 1e-5, gate=gate, gate_col0=col0, gate_bias=bias)
        assert ops.norm_add(h_dev, yd, wd, 1e-5, gate=gd, gate_col0=col0, gate_bias=bias_d) is None
        _close(h_dev, h_ref, 2e-6)
        want = emu.norm_add(h_ref, y, w, 1e-5, w2, 1e-6, out_dtype, gate, col0, bias)
        _close(ops.norm_add(h_dev, yd, wd, 1e-5, w2d, 1e-6, out_dtype, gd, col0, bias_d), want, tol)
        _close(h_dev, h_ref, 3e-6)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_one_gate_for_a_run_of_columns(dtype):
    ops = _ops()
    g = torch.Generator().manual_seed(9)
    for n, width, per, col0, out0 in ((11, 60, 20, 1, 0), (5, 64, 32, 3, 4), (300, 96, 6, 0, 2), (4, 7, 7, 2, 1), (9, 24, 1, 4, 8)):
        a = torch.randn(n, width, generator=g).to(dtype)
        proj = torch.randn(n, col0 + width // per + 3, generator=g)
        ref = torch.zeros(n, out0 + width + 4, dtype=dtype)
        dev = ref.to(DEV)
        emu.sigmoid_gate(a, proj, col0, 1.25, ref, out0, per)
        ops.sigmoid_gate(a.to(DEV), proj.to(DEV), col0, 1.25, dev, out0, per)
        _close(dev, ref, 2e-6 if dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
def test_square_of_relu(out_dtype):
    ops = _ops()
    g = torch.Generator().manual_seed(2)
    for n, wide, col0, width in ((37, 45, 3, 30), (8, 64, 0, 48), (260, 1024, 512, 256)):
        u = torch.randn(n, wide, generator=g) * 2.5
        tol = 2e-6 if out_dtype == torch.float32 else 8e-3
        _close(ops.activation(u.to(DEV), "relu2", out_dtype), emu.activation(u, "relu2", out_dtype), tol)
        for kind in ("relu2", "silu"):
            _close(ops.activation(u.to(DEV), kind, out_dtype, col0, width), emu.activation(u, kind, out_dtype, col0, width), tol)
    assert ops.activation(torch.tensor([[-2.0, 0.0, 3.0]], device=DEV), "relu2", torch.float32).tolist() == [[0.0, 0.0, 9.0]]


def _paged(ctx_lens, kvh, d, vd, ps, dtype, g, spare=3):
    """Random keys and values of requests with the given context lengths, spread over shuffled pages."""
    pages_of = [(c + ps - 1) // ps for c in ctx_lens]
    total = sum(pages_of) + spare
    order = torch.randperm(total, generator=g).tolist()
    k = torch.randn(total + 1, kvh, ps, d, generator=g).to(dtype)
    v = torch.randn(total + 1, kvh, vd, ps, generator=g).to(dtype)
    bt = torch.full((len(ctx_lens), max(pages_of)), total, dtype=torch.int32)
    at = 0
    for r, n in enumerate(pages_of):
        bt[r, :n] = torch.tensor(order[at: at + n], dtype=torch.int32)
        at += n
    return k, v, bt


def _attend(q, k, v, bt, cu, cl, scale, chunk, cap, sink, ps):
    """The attention of every request as whole matrices in float64 (for contexts the stand-in's loops are slow for)."""
    n, H, d = q.shape
    G, vd = k.shape[1], v.shape[2]
    out = torch.zeros(n, H, vd, dtype=torch.float64)
    for r in range(bt.shape[0]):
        lo, hi, ctx = int(cu[r]), int(cu[r + 1]), int(cl[r])
        j = torch.arange(ctx)
        pages = bt[r].long()[j // ps]
        K, V = k[pages, :, j % ps].double(), v[pages, :, :, j % ps].double()
        i = ctx - (hi - lo) + torch.arange(hi - lo)
        ok = j[None, :] <= i[:, None]
        if chunk:
            ok = ok & (j[None, :] // chunk == i[:, None] // chunk)
        for h in range(H):
            s = (q[lo:hi, h].double() @ K[:, h // (H // G)].T) * scale
            s = (cap * torch.tanh(s / cap) if cap else s).masked_fill(~ok, float("-inf"))
            if sink is not None:
                s = torch.cat([s, sink[h].double().expand(hi - lo, 1)], dim=1)
            out[lo:hi, h] = torch.softmax(s, dim=1)[:, :ctx] @ V[:, h // (H // G)]
    return out.reshape(n, H * vd)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kvh,d,vd,chunk,cap", [(4, 2, 12, 10, 9, 2.0), (1, 1, 20, 28, 16, 0.0), (3, 3, 6, 6, 1, 5.0), (4, 2, 64, 64, 50, 6.0),
                                                     (8, 1, 32, 32, 33, 0.0), (4, 4, 64, 32, 72, 3.0), (4, 4, 64, 32, 0, 0.0), (16, 1, 128, 128, 100, 4.0),
                                                     (4, 1, 128, 64, 0, 8.0), (2, 2, 128, 64, 64, 0.0), (5, 1, 160, 96, 0, 0.0), (4, 1, 192, 128, 0, 0.0),
                                                     (32, 1, 192, 128, 90, 7.0), (4, 1, 288, 256, 0, 0.0), (18, 1, 576, 512, 0, 0.0),
                                                     (3, 1, 320, 256, 40, 4.0), (33, 1, 576, 512, 77, 3.0), (2, 1, 96, 96, 48, 2.5), (6, 2, 32, 32, 32, 9.0)])
def test_attention_with_chunks_and_capped_scores(dtype, heads, kvh, d, vd, chunk, cap):
    """Portions behind cached prefixes and single tokens in one batch, every pair of sizes the matrix-core kernels take and
    some that they do not; with and without a sink of a constant score."""
    ops = _ops()
    g = torch.Generator().manual_seed(heads * 100 + d)
    q_lens, ctx_lens = [1, 37, 5, 1, 70], [150, 37, 120, 3, 200]
    k, v, bt = _paged(ctx_lens, kvh, d, vd, 16, dtype, g)
    n = sum(q_lens)
    q = (torch.randn(n, heads, d, generator=g) * 2).to(dtype)
    cu, token_req = _batch(q_lens)
    cl = torch.tensor(ctx_lens, dtype=torch.int32)
    tol = 2e-5 if dtype == torch.float32 else 1.6e-2
    scale = 2.0 * d ** -0.5
    dev = _dev(k, v, bt)
    for sink in (None, torch.zeros(heads)):
        want = emu.paged_attention(q, k, v, bt, cu, cl, token_req, scale, 0, max(q_lens), max(ctx_lens), None, None, sink, 0, chunk, cap)
        _close(_attend(q, k, v, bt, cu, cl, scale, chunk, cap, sink, 16), want, 1e-6 if dtype == torch.float32 else 8e-3)
        for singles in (0, 2):      # (the single tokens as portions of one, and through the kernels for decoding)
            got = ops.paged_attention(q.to(DEV), *dev, *_dev(cu, cl, token_req), scale, 0, max(q_lens), max(ctx_lens), singles,
                                      sink=None if sink is None else sink.to(DEV), chunk=chunk, softcap=cap)
            _close(got, want, tol)
        # a step of single tokens only (split over the context and combined, where the matrix-core kernels serve)
        q1 = (torch.randn(5, heads, d, generator=g) * 2).to(dtype)
        cu1, tr1 = _batch([1] * 5)
        want = emu.paged_attention(q1, k, v, bt, cu1, cl, tr1, scale, 0, 1, max(ctx_lens), None, None, sink, 0, chunk, cap)
        got = ops.paged_attention(q1.to(DEV), *dev, *_dev(cu1, cl, tr1), scale, 0, 1, max(ctx_lens), 5,
                                  sink=None if sink is None else sink.to(DEV), chunk=chunk, softcap=cap)
        _close(got, want, tol)


@pytest.mark.parametrize("heads,kvh,d,vd,chunk,cap", [(4, 1, 192, 128, 0, 0.0), (20, 1, 576, 512, 0, 0.0), (4, 2, 128, 128, 1500, 5.0), (2, 1, 128, 64, 0, 4.0), (8, 2, 64, 64, 700, 0.0)])
def test_long_contexts_in_parts_and_tiles(heads, kvh, d, vd, chunk, cap):
    """bfloat16, a portion behind 2,400 cached keys whose keys are split over blocks, a prompt beside it, and the kernels
    of 16 and of 32 query rows a wave and of per-wave loads forced in turn."""
    import ctypes
    ops = _ops()
    g = torch.Generator().manual_seed(d)
    q_lens, ctx_lens = [130, 1, 300], [2530, 2200, 300]
    k, v, bt = _paged(ctx_lens, kvh, d, vd, 16, torch.bfloat16, g)
    q = (torch.randn(sum(q_lens), heads, d, generator=g) * 2).to(torch.bfloat16)
    cu, token_req = _batch(q_lens)
    cl = torch.tensor(ctx_lens, dtype=torch.int32)
    scale = 1.5 * d ** -0.5
    want = _attend(q, k, v, bt, cu, cl, scale, chunk, cap, torch.zeros(heads), 16)
    args = _dev(q, k, v, bt, cu, cl, token_req)
    lib = ops.library()
    lib.tp_attention_tune.argtypes = [ctypes.c_int]
    keep = ops.portion_min_keys
    try:
        for tune, min_keys in ((0, 512), (0, 1 << 20), (1, 1 << 20), (2, 1 << 20), (3, 1 << 20)):
            ops.portion_min_keys = min_keys
            lib.tp_attention_tune(tune)
            got = ops.paged_attention(*args, scale, 0, max(q_lens), max(ctx_lens), 1, sink=torch.zeros(heads, device=DEV), chunk=chunk, softcap=cap)
            _close(got, want, 1.6e-2)
    finally:
        ops.portion_min_keys = keep
        lib.tp_attention_tune(0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("chunk", [16, 40, 47, 64])
def test_a_key_that_stands_out_at_every_edge_of_a_chunk(dtype, chunk):
    """One query whose score for ONE key is far above the rest: the first key of its chunk, the one before it, its own, a
    page's first and last place, at positions just inside and just outside an edge.  The output is that key's value when
    the query sees it and something else when it does not."""
    ops = _ops()
    g = torch.Generator().manual_seed(3)
    heads, kvh, d, vd, ps = 2, 1, 64, 64, 16
    for ctx in (3 * chunk, 3 * chunk + 1, 3 * chunk + 2, 200):
        k, v, bt = _paged([ctx], kvh, d, vd, ps, dtype, g)
        pos = ctx - 1
        start = pos // chunk * chunk
        cu, token_req = _batch([1])
        cl = torch.tensor([ctx], dtype=torch.int32)
        for needle in sorted({start, max(0, start - 1), pos, (pos + start) // 2, 0, 15, 16, max(0, pos - chunk)}):
            if needle > pos:
                continue
            page, off = int(bt[0, needle // ps]), needle % ps
            q = torch.zeros(1, heads, d)
            q[0, :] = k[page, 0, off].float() * 3.0
            q = q.to(dtype)
            want = emu.paged_attention(q, k, v, bt, cu, cl, token_req, 1.0, 0, 1, ctx, None, None, None, 0, chunk, 150.0)
            for singles in (1, 0):
                got = ops.paged_attention(*_dev(q, k, v, bt, cu, cl, token_req), 1.0, 0, 1, ctx, singles, chunk=chunk, softcap=150.0)
                _close(got, want, 2e-5 if dtype == torch.float32 else 1.6e-2)
            is_value = torch.allclose(want.float().reshape(heads, vd)[0], v[page, 0, :, off].float(), atol=0.05)
            assert is_value == (needle >= start), (ctx, needle)


def test_sizes_the_kernels_do_not_take_are_refused():
    ops = _ops()
    q = torch.zeros(1, 2, 32, device=DEV)
    k, v = torch.zeros(2, 1, 16, 32, device=DEV), torch.zeros(2, 1, 32, 16, device=DEV)
    i32 = lambda *x: torch.tensor(x, dtype=torch.int32, device=DEV)
    with pytest.raises(ops.KernelError, match="exclude"):
        ops.paged_attention(q, k, v, i32(0).view(1, 1), i32(0, 1), i32(1), i32(0), 1.0, 8, 1, 1, 1, chunk=8)
    with pytest.raises(ops.KernelError, match="exclude"):
        ops.paged_attention(q, k, v, i32(0).view(1, 1), i32(0, 1), i32(1), i32(0), 1.0, 0, 1, 1, 1, softcap=2.0, dist_bias=torch.zeros(2, 4, device=DEV))
    with pytest.raises(ops.KernelError, match="even"):
        ops.qkv_rows(torch.zeros(1, 15, device=DEV), i32(0), i32(0), 1, 1, 5, 5, torch.zeros(1, 1, 16, 5, device=DEV), torch.zeros(1, 1, 5, 16, device=DEV))
    with pytest.raises(ops.KernelError, match="caches"):
        ops.qkv_rows(torch.zeros(1, 96, device=DEV), i32(0), i32(0), 1, 1, 32, 32, k, torch.zeros(2, 1, 16, 16, device=DEV))


# ---- the model through the step function --------------------------------------------------------
def _runner(folder, dtype, max_tokens, page_size=16, max_requests=4, use_graph=False):
    from tempura_amd.engine.loading import load_model
    from tempura_amd.engine.runner import ModelRunner
    model = load_model(folder, dtype, DEV)
    return ModelRunner(model, page_size, (max_tokens + page_size - 1) // page_size, max_requests=max_requests, use_graph=use_graph)


_REFS = {}


def _ref(name, rid):
    if (name, rid) not in _REFS:
        _REFS[(name, rid)] = plain.forward(cases.config_json(name), cases.make_weights(name), cases.requests(name)[rid])
    return _REFS[(name, rid)]


@pytest.mark.parametrize("name", ["mix", "one", "wide", "deep"])
@pytest.mark.parametrize("dtype,tol", [("float32", 3e-5), ("bfloat16", 6e-2)])
def test_each_part_alone_matches_its_plain_function(dirs, name, dtype, tol):
    import tokatar_mechanisms
    tokatar_mechanisms.check(dirs[name], name, DEV, tol, dtype=dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mix", "one", "wide", "deep"])
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
    runner = _runner(dirs[name], dtype, max_tokens)
    got = helpers.run_schedule(runner, reqs, steps)
    for rid in reqs:
        _assert_logits(got[rid], _ref(name, rid), dtype, f"{name}/{mode}/{dtype}: request {rid}")
    assert not runner.cache.live_requests()
    assert runner.cache.free_pages() == [p.num_pages for p in runner.cache.pools]


def test_cutting_changes_rounding_only(dirs):
    """The same request whole, in portions and beside others, in float32: summation order only."""
    reqs = cases.requests("wide")
    lengths = cases.LENGTHS["wide"]
    runs = []
    for steps in (helpers.schedule_whole(lengths), helpers.schedule_portions(lengths, sizes=(2, 9, 33, 2, 16, 5)),
                  helpers.schedule_mixed(lengths, 512, seed=3)):
        runs.append(helpers.run_schedule(_runner(dirs["wide"], "float32", 512), reqs, steps))
    for rid in reqs:
        for other in runs[1:]:
            assert plain.logit_error(other[rid], runs[0][rid]) < 1e-4, rid


@pytest.mark.parametrize("chunk", [16, 33, 50, 64])
@pytest.mark.parametrize("layer", [0, 1])
def test_the_edges_of_the_chunks_on_the_gpu(tmp_path, chunk, layer):
    """Queries many times larger than drawn (a softmax that rests on one or two keys of its chunk): a prompt whole, then in
    portions that end at and beside page and chunk borders with decoding behind them.  The premise first: a chunk one
    longer or one shorter gives other logits.  (float32: in bfloat16 the rounding of q and k decides between near-equal keys
    of such a softmax; the kernels' own tests plant their keys in both types.)"""
    from tempura_amd.engine.runner import StepEntry
    cfg = cases.config_json("wide")
    cfg["layers"] = cfg["layers"][layer: layer + 1] + cfg["layers"][2:3]
    cfg["layers"][0]["mixer"].update({"mask": {"size": chunk}})
    if layer == 0:
        cfg["layers"][0]["mixer"]["softcap"] = 25.0
    W = cases.make_weights("wide", sharp=6.0, cfg=cfg)
    folder = cases.write_model("wide", str(tmp_path / "sharp"), weights=W, config=cfg)
    toks = cases.tokens("wide", 200, 5)
    ref = plain.forward(cfg, W, toks)
    for other in (chunk - 1, chunk + 1):
        c2 = copy.deepcopy(cfg)
        c2["layers"][0]["mixer"]["mask"]["size"] = other
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


def test_a_far_latent_decides_on_the_gpu(tmp_path):
    """Sharp queries over the cached latents, 450 tokens, in a prompt cut anywhere, then in decoding."""
    from tempura_amd.engine.runner import StepEntry
    cfg = cases.config_json("wide")
    cfg["layers"] = [cfg["layers"][2], cfg["layers"][4]]
    W = cases.make_weights("wide", sharp=6.0, cfg=cfg)
    folder = cases.write_model("wide", str(tmp_path / "far"), weights=W, config=cfg)
    toks = cases.tokens("wide", 450, 17)
    ref = plain.forward(cfg, W, toks)
    runner = _runner(folder, "float32", 512)
    runner.add_request("r")
    rows, at = [], 0
    for c in (130, 2, 161, 100, 7):
        rows.append(runner.step([StepEntry("r", toks[at: at + c], list(range(c)))]).cpu())
        at += c
    rows += [runner.step([StepEntry("r", [t], [0])]).cpu() for t in toks[at:]]
    assert plain.logit_error(torch.cat(rows), ref) < SHARP_TOL


@pytest.mark.parametrize("name,dtype", [("wide", "float32"), ("wide", "bfloat16"), ("deep", "bfloat16")])
def test_long_decoding_through_a_captured_step(dirs, name, dtype):
    """Two requests decoded token by token for 150 steps through the graph path: pages, latents and chunks move along."""
    from tempura_amd.engine.runner import StepEntry
    cfg, W = cases.config_json(name), cases.make_weights(name)
    runner = _runner(dirs[name], dtype, 512, use_graph=True)
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


@pytest.mark.parametrize("name", ["mix", "wide"])
@pytest.mark.parametrize("use_graph", [False, True])
def test_engine_generates_what_plain_greedy_generates(dirs, name, use_graph):
    from tempura_amd.engine import Engine
    from tempura_amd.sampling import SamplingParams
    cfg, W = cases.config_json(name), cases.make_weights(name)
    prompts = [cases.tokens(name, n, 20 + i) for i, n in enumerate((3, 18, 9, 40, 1))]
    eng = Engine(dirs[name], dtype="float32", page_size=16, kv_pages=24, max_batch_size=3, max_num_batched_tokens=32,
                 prefill_chunk_size=7, device=DEV, use_graph=use_graph)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=12))
    for p, o in zip(prompts, outs):
        assert o == plain.greedy(cfg, W, p, 12)
    if use_graph:
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
    p = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", dirs["mix"], "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    ref = plain.forward(cases.config_json("mix"), cases.make_weights("mix"), toks)
    vocab = ref.shape[1]
    a = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(-1, vocab))
    c = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(-1, vocab))
    assert plain.logit_error(torch.cat([a, c]), torch.stack([ref[0], ref[10], ref[29], ref[3]])) < TOL["float32"]


@pytest.mark.parametrize("m", [1, 2, 8, 16, 17, 40, 64, 65, 100, 128, 129, 200, 300, 700, 2049])
@pytest.mark.parametrize("n,act,k", [(384, 128, 128), (384, 384, 192), (640, 512, 256), (2576, 1536, 2048), (1168, 1024, 64), (4608, 3584, 512)])
def test_up_product_that_leaves_squared_relu_beside_plain_columns(m, n, act, k):
    """Every product kernel that a number of rows selects, weights tiled and row-major: the activated columns in bfloat16
    (a few rows also k-blocked), the side columns in float32."""
    ops = _ops()
    g = torch.Generator().manual_seed(n + k)
    w = (torch.randn(n, k, generator=g) * k ** -0.5).to(torch.bfloat16).to(DEV)
    x = torch.randn(m, k, generator=torch.Generator().manual_seed(m)).to(torch.bfloat16).to(DEV)
    y = x.float() @ w.float().T
    want = torch.clamp(y[:, :act], min=0.0) ** 2
    for weight in (w, ops.tile_weight(w)):
        out, side = ops.linear_relu2(x, weight, act)
        assert out.dtype == torch.bfloat16 and side.shape == (m, n - act)
        _close(out, want, 6e-3)
        if n > act:
            _close(side, y[:, act:], 3e-5)
        blocked, side2 = ops.linear_relu2(x, weight, act, blocked_out=True)
        if m <= 16:
            assert isinstance(blocked, ops.KBlocked) and torch.equal(blocked.row_major(), out)
        assert torch.equal(side2, side)
