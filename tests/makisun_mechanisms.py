"""Each mechanism of the Makisun design alone: the framework's part, taken out of a loaded model and run on random
rows through the step's own context, cache and state, against the plain function of tests/plain_makisun.py for it.
Used by the host tests (over the stand-in operations) and by the GPU tests (over the kernels)."""
from __future__ import annotations

import torch

import makisun_cases as cases
import plain_makisun as plain


def _err(got, ref):
    got, ref = got.double().cpu(), ref.double()
    return float((got - ref).abs().max() / ref.abs().max())


def check(folder: str, name: str, device: str, tol: float, seed: int = 0, cuts=(0, 21, 23, 37, 38), dtype: str = "float32", cfg=None) -> None:
    """Asserts, for every layer of case ``name``: the mixer and the feed-forward alone and the whole block (norms and
    scales) on a stream of its own, and, for two mixers side by side, each of them alone, as a prompt cut at ``cuts`` (so
    that cached keys, states and carried rows cross the steps' borders, the last step being one token); then the embedding
    and the last norm."""
    from tempura_amd.engine.loading import load_model
    from tempura_amd.engine.runner import ModelRunner, StepEntry
    from tempura_amd.kernels import ops
    cfg = cfg if cfg is not None else cases.config_json(name)
    W = cases.make_weights(name)
    W64 = {k: v.double() for k, v in W.items()}
    model = load_model(folder, dtype, device)
    runner = ModelRunner(model, 16, 2 * ((cuts[-1] + 15) // 16) + 2, max_requests=2)
    g = torch.Generator().manual_seed(seed)
    n, width = cuts[-1], cfg["width"]
    toks = cases.tokens(name, n, 3)
    eps = float(cfg["norm"]["eps"])
    x = torch.randn(n, width, generator=g)
    if dtype == "bfloat16":
        x = x.to(torch.bfloat16).float()
    stream = torch.randn(n, width, generator=g) * 3
    outs = {}
    for phase in ("parts", "left", "right", "blocks"):
        runner.add_request(phase)
        for slot_state in runner.pools.state.values():
            slot_state.zero_()      # (the step function clears a new request's state; the parts are called without it)
        for lo, hi in zip(cuts[:-1], cuts[1:]):
            tok_dev, ctx = runner._pack_step([StepEntry(phase, toks[lo:hi], [])])
            if phase == "parts":
                outs.setdefault("embed", []).append(model.embedding.forward(tok_dev, ctx.positions, 1, ctx=ctx).cpu())
                outs.setdefault("norm", []).append(model.final_norm.forward(stream[lo:hi].to(device)).cpu())
            rows = x[lo:hi].to(device=device)
            for i, block in enumerate(model.layers):
                ctx.shared.clear()
                cache = runner.layer_caches[i]
                if phase == "blocks":
                    h = stream[lo:hi].to(device).clone()
                    assert block.forward(h, ctx, cache) is None
                    outs.setdefault((i, "block"), []).append(h.cpu())
                elif phase == "parts":
                    mine = rows.to(block.mixer.input_dtype or model.dtype)
                    outs.setdefault((i, "mixer"), []).append(block.mixer.forward(mine, ctx, cache, None).cpu())
                    if block.ffn is not None:
                        outs.setdefault((i, "ffn"), []).append(block.ffn.forward(rows.to(model.dtype), ctx, None).cpu())
                elif cfg["layers"][i]["type"] == "parallel":
                    k = ("left", "right").index(phase)
                    mixer = block.mixer
                    act = torch.zeros((hi - lo, mixer.inner), dtype=model.dtype, device=device)
                    proj = ops.linear(rows.to(model.dtype), mixer.w_in, torch.float32)
                    mixer.branches[k].run(proj, mixer.in_cols[k], ctx, cache, act, mixer.out_cols[k], 1.0)
                    outs.setdefault((i, phase), []).append(ops.linear(act, mixer.w_out, torch.float32).cpu())
            runner.cache.commit_many([phase], ctx.q_lens)
        runner.end_request(phase)
    got = {k: torch.cat(v) for k, v in outs.items()}
    xd = x.double()
    assert _err(got["embed"], W64["embed"][torch.tensor(toks)] * cfg["embedding"]["scale"]) < min(tol, 1e-6), "embedding"
    assert _err(got["norm"], plain.norm_around_zero(stream.double(), W64["final.norm"], eps)) < min(tol, 1e-2), "last norm"
    for i, layer in enumerate(cfg["layers"]):
        p, c = f"l{i}", layer["mixer"]
        mixer = plain.MIXERS[layer["type"]]
        assert _err(got[(i, "mixer")], mixer(xd, W64, p + ".mix", c, eps)) < tol, f"layer {i}: {layer['type']}"
        if layer["type"] == "parallel":
            assert _err(got[(i, "left")], plain.left(xd, W64, p + ".mix.left", c["left"], eps)) < tol, f"layer {i}: left"
            assert _err(got[(i, "right")], plain.right(xd, W64, p + ".mix.right", c["right"], eps)) < tol, f"layer {i}: right"
        h = stream.double()
        h = h + W64[p + ".ls1"] * mixer(plain.norm_around_zero(h, W64[p + ".norm1"], eps), W64, p + ".mix", c, eps)
        if layer["mlp"] is not None:
            assert _err(got[(i, "ffn")], plain.feed_forward(xd, W64, p + ".mlp", layer["mlp"])) < tol, f"layer {i}: feed-forward"
            h = h + W64[p + ".ls2"] * plain.feed_forward(plain.norm_around_zero(h, W64[p + ".norm2"], eps), W64, p + ".mlp", layer["mlp"])
        assert _err(got[(i, "block")], h) < tol, f"layer {i}: block"
