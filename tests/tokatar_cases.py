"""Small Tokatar configurations and random weights of the tests' own making (stored as bfloat16 values, so that the
float32 and the bfloat16 engine and the plain implementation all read the same numbers)."""
from __future__ import annotations

import json
import os
from typing import Dict, List

import torch


def _rot(dims, base, scaling=None):
    d = {"dims": dims, "base": base}
    if scaling is not None:
        d["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return d


def _attention(heads, kv, dim, vdim, scale, rot, chunk=None, cap=None, kind="attention"):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    if chunk is not None:
        m["mask"] = {"size": chunk}
    if cap is not None:
        m["softcap"] = cap
    return kind, m


def _attention_2(*args, **kw):
    return _attention(*args, **kw, kind="attention_2")


def _latent(heads, dim, rot_dim, vdim, rank, scale, base):
    return "latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale,
                                "rot": _rot(rot_dim, base)}


def _layer(mixer, ff):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _case(vocab, width, layers, eps, scale):
    return {"architecture": "Tokatar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}


#: name -> config.json content
CASES: Dict[str, dict] = {
    # the three mixers; grouped key heads, values narrower and wider than keys, part of a head rotated, scaled frequencies
    # of every kind (kept, blended, divided), chunks shorter than the prompts, a cap that bends every score; an
    # attention without chunks, cap or scaling; layers without a feed-forward
    "mix": _case(90, 48, [_layer(_attention(4, 2, 12, 10, 0.3, _rot(8, 300.0, (4.0, 1.0, 4.0, 64)), chunk=9, cap=2.0), 40),
                          _layer(_attention_2(4, 2, 10, 6, 0.35, _rot(6, 90.0), chunk=21), 24),
                          _layer(_latent(3, 8, 4, 6, 20, 0.3, 50.0), None),
                          _layer(_attention_2(2, 1, 8, 12, 0.4, _rot(8, 500.0)), 32),
                          _layer(_latent(2, 10, 6, 14, 10, 0.25, 200.0), 24),
                          _layer(_attention(2, 2, 8, 8, 0.35, _rot(8, 100.0)), None)], 1e-5, 2.5),
    # values that a model may happen to make 1 or equal: one head, one key head, a chunk of exactly one page, of one
    # position and of five, two rotated elements, sizes that fill no power of two, a latent narrower than its rotated part
    "one": _case(40, 32, [_layer(_attention(1, 1, 20, 28, 0.25, _rot(20, 100.0), chunk=16, cap=1.0), 16),
                          _layer(_attention_2(3, 3, 6, 6, 0.4, _rot(2, 10.0), chunk=5), 8),
                          _layer(_latent(1, 7, 12, 5, 8, 0.3, 40.0), 16),
                          _layer(_attention_2(1, 1, 6, 10, 0.5, _rot(6, 30.0), chunk=1), None),
                          _layer(_attention(3, 1, 6, 6, 0.4, _rot(4, 20.0, (8.0, 2.0, 2.0, 32)), cap=30.0), 8)], 1e-6, 1.0),
    # sizes the matrix-core kernels take (also keys wider than values, and latents with a rotated part that are padded up
    # to such sizes), chunks that are no multiple of a page
    "wide": _case(96, 128, [_layer(_attention(4, 2, 64, 64, 0.125, _rot(64, 10000.0, (8.0, 1.0, 4.0, 256)), chunk=50, cap=6.0), 128),
                            _layer(_attention_2(4, 4, 64, 32, 0.125, _rot(32, 5000.0), chunk=72), 256),
                            _layer(_latent(4, 32, 32, 48, 96, 0.125, 1000.0), 128),
                            _layer(_attention(8, 1, 32, 32, 0.2, _rot(16, 3000.0), chunk=33), None),
                            _layer(_latent(2, 64, 64, 32, 128, 0.09, 8000.0), 64),
                            _layer(_attention_2(2, 1, 128, 128, 0.09, _rot(128, 20000.0)), 128)], 1e-5, 1.75),
    # latents much wider than the heads: the matrix-core kernels for keys of several hundred, maps as products per head
    "deep": _case(70, 64, [_layer(_latent(4, 32, 32, 32, 256, 0.125, 1000.0), 64),
                           _layer(_latent(3, 32, 64, 48, 256, 0.1, 3000.0), None),
                           _layer(_latent(18, 64, 64, 32, 512, 0.09, 8000.0), 128)], 1e-5, 2.0),
}


def config_json(name: str) -> dict:
    """The case as config.json would hold it."""
    return json.loads(json.dumps(CASES[name]))


def make_weights(name: str, seed: int = 0, sharp: float = 1.0, cfg: dict = None) -> Dict[str, torch.Tensor]:
    """bfloat16 tensors by checkpoint name, drawn so that every mechanism matters to the logits.  ``sharp`` multiplies
    the queries: with large values a query's softmax rests on one or two keys somewhere among those it sees, far ones
    as often as near ones."""
    cfg = cfg if cfg is not None else CASES[name]
    g = torch.Generator().manual_seed(seed)
    W: Dict[str, torch.Tensor] = {}

    def normal(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=g, dtype=torch.float64) * std + mean

    width = cfg["width"]
    W["embed"] = normal(cfg["vocab"], width, std=0.6)
    W["final.norm"] = normal(1, std=0.2, mean=1.1).reshape(())
    W["head"] = normal(cfg["vocab"], width, std=width ** -0.5)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        for n in (1, 2) if layer["mlp"] is not None else (1,):
            W[f"{p}.norm{n}"] = normal(1, std=0.2, mean=1.2).reshape(())
            W[f"{p}.norm{n}b"] = normal(1, std=0.2, mean=0.8).reshape(())
            W[f"{p}.ls{n}"] = normal(width, std=0.3, mean=1.0)
            W[f"{p}.rg{n}"] = normal(width, width, std=1.5 * width ** -0.5)
            W[f"{p}.rg{n}.b"] = normal(width, std=0.7)
        m, q = layer["mixer"], f"{p}.mix"
        H, D, E = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "latent_attention":
            R, L = m["rot_dim"], m["kv_rank"]
            W[q + ".q"] = normal(H * (D + R), width, std=sharp * 1.5 * width ** -0.5)
            W[q + ".dkv"] = normal(L + R, width, std=width ** -0.5)
            W[q + ".dkv.norm"] = normal(L, std=0.2, mean=1.0)
            W[q + ".uk"] = normal(H * D, L, std=1.5 * L ** -0.5)
            W[q + ".uv"] = normal(H * E, L, std=L ** -0.5)
            W[q + ".g"] = normal(H, width, std=1.5 * width ** -0.5)
        else:
            G = m["kv_heads"]
            two = layer["type"] == "attention_2"
            W[q + ".q"] = normal(H * D, width, std=(1.0 if two else 1.5 * sharp) * width ** -0.5)
            W[q + ".k"] = normal(G * D, width, std=(1.0 if two else 1.5) * width ** -0.5)
            W[q + ".v"] = normal(G * E, width, std=width ** -0.5)
            W[q + ".g"] = normal(H * E, width, std=1.5 * width ** -0.5)
            if two:
                W[q + ".q.b"] = normal(H * D, std=0.5)
                W[q + ".k.b"] = normal(G * D, std=0.5)
                W[q + ".v.b"] = normal(G * E, std=0.5)
                W[q + ".q.norm"] = normal(H * D, std=0.3, mean=sharp * 1.5)
                W[q + ".k.norm"] = normal(G * D, std=0.3, mean=1.5)
        W[q + ".o"] = normal(width, H * E, std=(H * E) ** -0.5)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            W[f"{p}.mlp.up"] = normal(ff, width, std=1.5 * width ** -0.5)
            W[f"{p}.mlp.down"] = normal(width, ff, std=ff ** -0.5)
    return {k: v.to(torch.bfloat16) for k, v in W.items()}


def write_model(name: str, folder: str, seed: int = 0, weights=None, config=None) -> str:
    from tempura_amd.weights import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(config if config is not None else config_json(name), f)
    W = weights if weights is not None else make_weights(name, seed)
    write_safetensors(os.path.join(folder, "model.safetensors"), W.items(), metadata={"format": "pt"})
    return folder


def tokens(name: str, n: int, seed: int) -> List[int]:
    g = torch.Generator().manual_seed(8765 + seed)
    return torch.randint(0, CASES[name]["vocab"], (n,), generator=g).tolist()


#: request lengths per case: one token, a few, around pages' and chunks' edges, long
LENGTHS = {"mix": {"m0": 1, "m1": 6, "m2": 23, "m3": 49, "m4": 33, "m5": 16},
           "one": {"o0": 2, "o1": 31, "o2": 17, "o3": 1, "o4": 40},
           "wide": {"w0": 5, "w1": 74, "w2": 33, "w3": 160, "w4": 50},
           "deep": {"d0": 3, "d1": 90, "d2": 17, "d3": 140, "d4": 64}}


def requests(name: str) -> Dict[str, List[int]]:
    return {rid: tokens(name, n, i) for i, (rid, n) in enumerate(LENGTHS[name].items())}
