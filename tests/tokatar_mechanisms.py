"""Each mechanism of the Tokatar design alone: the framework's part, taken out of a loaded model and run on random
rows through the step's own context, cache and state, against the plain function of tests/plain_tokatar.py for it.
Used by the host tests (over the stand-in operations) and by the GPU tests (over the kernels)."""
from __future__ import annotations

import torch

import plain_tokatar as plain
import tokatar_cases as cases


def _err(got, ref):
    got, ref = got.double().cpu(), ref.double()
    return float((got - ref).abs().max() / ref.abs().max())


def check(folder: str, name: str, device: str, tol: float, seed: int = 0, cuts=(0, 21, 23, 37, 38), dtype: str = "float32") -> None:
    """Asserts, for every layer of case ``name``: the mixer and the feed-forward alone with the rows of the gates that
    ride along, and the whole block (norms, gates, scales) on a stream of its own, as a prompt cut at ``cuts`` (so that
    cached keys cross the steps' borders, the last step being one token); then the embedding and the last norm."""
    from tempura_amd.engine.loading import load_model
    from tempura_amd.engine.runner import ModelRunner, StepEntry
    cfg, W = cases.config_json(name), cases.make_weights(name)
    W64 = {k: v.double() for k, v in W.items()}
    model = load_model(folder, dtype, device)
    runner = ModelRunner(model, 16, 8, max_requests=2)
    g = torch.Generator().manual_seed(seed)
    n, width = cuts[-1], cfg["width"]
    toks = cases.tokens(name, n, 3)
    eps = float(cfg["norm"]["eps"])
    x = torch.randn(n, width, generator=g)
    if dtype == "bfloat16":
        x = x.to(torch.bfloat16).float()
    stream = torch.randn(n, width, generator=g) * 3
    outs = {}
    for phase in ("parts", "blocks"):
        runner.add_request(phase)
        for lo, hi in zip(cuts[:-1], cuts[1:]):
            tok_dev, ctx = runner._pack_step([StepEntry(phase, toks[lo:hi], [])])
            if phase == "parts":
                outs.setdefault("embed", []).append(model.embedding.forward(tok_dev, ctx.positions, 1, ctx=ctx).cpu())
                outs.setdefault("norm", []).append(model.final_norm.forward(stream[lo:hi].to(device)).cpu())
            rows = x[lo:hi].to(device=device, dtype=model.dtype)
            for i, block in enumerate(model.layers):
                ctx.shared.clear()
                cache = runner.layer_caches[i]
                if phase == "blocks":
                    h = stream[lo:hi].to(device).clone()
                    assert block.forward(h, ctx, cache) is None
                    outs.setdefault((i, "block"), []).append(h.cpu())
                    continue
                for part, args in (("mixer", (rows, ctx, cache, None)), ("ffn", (rows, ctx))):
                    p = getattr(block, part)
                    if p is None:
                        continue
                    y, (side, col0) = p.forward(*args)
                    outs.setdefault((i, part), []).append(y.cpu())
                    outs.setdefault((i, part + " gate"), []).append(side[:, col0: col0 + width].cpu())
            runner.cache.commit_many([phase], ctx.q_lens)
        runner.end_request(phase)
    got = {k: torch.cat(v) for k, v in outs.items()}
    xd = x.double()
    assert _err(got["embed"], W64["embed"][torch.tensor(toks)] * cfg["embedding"]["scale"]) < min(tol, 1e-6), "embedding"
    assert _err(got["norm"], plain.scalar_norm(stream.double(), W64["final.norm"], eps)) < min(tol, 1e-2), "last norm"
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        mixer = plain.MIXERS[layer["type"]]
        assert _err(got[(i, "mixer")], mixer(xd, W64, p + ".mix", layer["mixer"], eps)) < tol, f"layer {i}: {layer['type']}"
        assert _err(got[(i, "mixer gate")], xd @ W64[p + ".rg1"].T) < min(tol, 1e-4), f"layer {i}: gate rows"
        h = stream.double()
        u = plain.scalar_norm(h, W64[p + ".norm1"], eps)
        h = plain.closing(h, mixer(u, W64, p + ".mix", layer["mixer"], eps), u, W64, p, 1, eps)
        if layer["mlp"] is not None:
            assert _err(got[(i, "ffn")], plain.dense_ff(xd, W64, p + ".mlp")) < tol, f"layer {i}: feed-forward"
            assert _err(got[(i, "ffn gate")], xd @ W64[p + ".rg2"].T) < min(tol, 1e-4), f"layer {i}: gate rows"
            u = plain.scalar_norm(h, W64[p + ".norm2"], eps)
            h = plain.closing(h, plain.dense_ff(u, W64, p + ".mlp"), u, W64, p, 2, eps)
        assert _err(got[(i, "block")], h) < tol, f"layer {i}: block"
