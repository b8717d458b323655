"""Small Makisun configurations and random weights of the tests' own making (stored as bfloat16 values, so that the
float32 and the bfloat16 engine and the plain implementation all read the same numbers)."""
from __future__ import annotations

import json
import os
from typing import Dict, List

import torch


def _wkv(heads, dim):
    return "wkv", {"heads": heads, "dim": dim}


def _left(heads, kv, dim, vdim, scale, rot, base, window=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"dims": rot, "base": base}}
    if window is not None:
        m["mask"] = {"size": window}
    return m


def _right(heads, dim, vdim, tau):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def _parallel(left, right, left_scale, right_scale):
    return "parallel", {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def _layer(mixer, mlp):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def _case(vocab, width, layers, eps, scale):
    return {"architecture": "Makisun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}


#: ranks of the decays' low-rank projections (the tensors' own: no configuration names them), by case
RANKS = {"mix": (6, 5), "one": (1, 3), "wide": (16, 24)}

#: name -> config.json content
CASES: Dict[str, dict] = {
    # both mixers and every feed-forward; grouped key heads, values narrower and wider than keys, part of a head rotated,
    # windows shorter than the prompts and none, a router with and without a shared expert
    "mix": _case(90, 48, [_layer(_wkv(3, 10), _dense(40)),
                          _layer(_parallel(_left(4, 2, 12, 10, 0.3, 8, 300.0, window=9), _right(3, 6, 14, 8.0), 0.7, 1.2), _moe(24, 6, 2, shared=20)),
                          _layer(_wkv(2, 16), _moe(12, 5, 3)),
                          _layer(_parallel(_left(2, 1, 8, 14, 0.4, 8, 90.0), _right(2, 12, 5, 2.5), 1.3, 0.6), None),
                          _layer(_wkv(4, 7), None)], 1e-5, 2.5),
    # values that a model may happen to make 1 or equal: one head, one key head, one expert a token, scales and a root of
    # 1, a window of exactly a page and of one position, two rotated elements, ranks of 1, sizes that fill no power of two
    "one": _case(40, 32, [_layer(_parallel(_left(1, 1, 20, 28, 0.25, 20, 100.0, window=16), _right(1, 7, 5, 1.0), 1.0, 1.0), _moe(8, 4, 1, shared=8)),
                          _layer(_wkv(1, 9), _dense(16)),
                          _layer(_parallel(_left(3, 3, 6, 6, 0.4, 2, 10.0, window=1), _right(5, 3, 3, 20.0), 1.0, -0.5), _moe(16, 3, 3)),
                          _layer(_wkv(5, 4), _moe(7, 1, 1, shared=9))], 1e-6, 1.0),
    # sizes the matrix-core kernels and the fused products take, recurrences of 64 x 64 to 128 x 32, windows that are no
    # multiple of a page
    "wide": _case(96, 128, [_layer(_wkv(2, 64), _dense(256)),
                            _layer(_parallel(_left(4, 2, 64, 64, 0.125, 32, 10000.0, window=50), _right(2, 128, 64, 16.0), 0.8, 0.9), _moe(128, 16, 3, shared=128)),
                            _layer(_wkv(1, 128), _moe(64, 8, 2)),
                            _layer(_parallel(_left(8, 1, 32, 32, 0.2, 16, 3000.0, window=33), _right(4, 32, 128, 12.0), 1.1, 0.7), None),
                            _layer(_wkv(8, 16), _dense(192)),
                            _layer(_parallel(_left(2, 2, 96, 128, 0.1, 64, 500.0, window=80), _right(3, 40, 32, 9.0), 0.9, 1.2), _dense(64))], 1e-5, 1.75),
}


def config_json(name: str, every_expert: bool = False) -> dict:
    """The case as config.json would hold it.  ``every_expert``: each token uses all experts, so that no choice is
    there for a rounding to flip (for runs in bfloat16; the logits still weigh the experts)."""
    cfg = json.loads(json.dumps(CASES[name]))
    for layer in cfg["layers"]:
        if every_expert and layer["mlp"] is not None and layer["mlp"]["kind"] == "moe":
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return cfg


def make_weights(name: str, seed: int = 0, sharp: float = 1.0, slow: float = 0.0, cfg: dict = None) -> Dict[str, torch.Tensor]:
    """bfloat16 tensors by checkpoint name, drawn so that every mechanism matters to the logits.  ``sharp`` multiplies
    the queries of the attentions: with large values a query's softmax rests on one or two keys somewhere among those
    it sees.  ``slow`` moves the recurrences' decays towards one (a step's loss shrinks by e^-slow), so that their states
    remember hundreds of tokens."""
    cfg = cfg if cfg is not None else CASES[name]
    g = torch.Generator().manual_seed(seed)
    W: Dict[str, torch.Tensor] = {}

    def normal(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=g, dtype=torch.float64) * std + mean

    width = cfg["width"]
    rank_w, rank_a = RANKS[name]
    W["embed"] = normal(cfg["vocab"], width, std=0.6)
    W["final.norm"] = normal(width, std=0.2)
    W["head"] = normal(cfg["vocab"], width, std=width ** -0.5)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        for n in (1, 2) if layer["mlp"] is not None else (1,):
            W[f"{p}.norm{n}"] = normal(width, std=0.2)
            W[f"{p}.ls{n}"] = normal(width, std=0.3, mean=1.0)
        m, q = layer["mixer"], f"{p}.mix"
        if layer["type"] == "wkv":
            H, D = m["heads"], m["dim"]
            for s in "rkvgw":
                W[f"{q}.mu.{s}"] = normal(width, std=0.3, mean=0.5)
            for s in "rkvg":
                W[f"{q}.{s}"] = normal(H * D, width, std=1.3 * width ** -0.5)
            W[q + ".w1"] = normal(rank_w, width, std=1.5 * width ** -0.5)
            W[q + ".w2"] = normal(H * D, rank_w, std=1.2 * rank_w ** -0.5)
            W[q + ".w0"] = normal(H * D, std=1.0, mean=-1.5 - slow)
            W[q + ".u"] = normal(H, D, std=1.0)
            W[q + ".norm"] = normal(H * D, std=0.2, mean=1.0)
            W[q + ".o"] = normal(width, H * D, std=(H * D) ** -0.5)
        else:
            a, r = m["left"], m["right"]
            H, G, D, E = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            W[q + ".left.q"] = normal(H * D, width, std=width ** -0.5)
            W[q + ".left.k"] = normal(G * D, width, std=width ** -0.5)
            W[q + ".left.v"] = normal(G * E, width, std=width ** -0.5)
            W[q + ".left.q.norm"] = normal(D, std=0.3, mean=sharp * 1.6)
            W[q + ".left.k.norm"] = normal(D, std=0.3, mean=1.6)
            W[q + ".left.g"] = normal(H, width, std=2.0 * width ** -0.5)
            W[q + ".left.o"] = normal(width, H * E, std=(H * E) ** -0.5)
            H, D, E = r["heads"], r["dim"], r["vdim"]
            for s, rows in (("q", H * D), ("k", H * D), ("v", H * E), ("g", H * E)):
                W[f"{q}.right.{s}"] = normal(rows, width, std=1.3 * width ** -0.5)
            W[q + ".right.a1"] = normal(rank_a, width, std=1.5 * width ** -0.5)
            W[q + ".right.a2"] = normal(H * D, rank_a, std=1.5 * rank_a ** -0.5)
            W[q + ".right.a2.b"] = normal(H * D, std=1.0, mean=slow)
            W[q + ".right.norm"] = normal(E, std=0.2, mean=1.0)
            W[q + ".right.o"] = normal(width, H * E, std=(H * E) ** -0.5)
        mlp = layer["mlp"]
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            W[f"{p}.mlp.up"] = normal(mlp["ff"], width, std=1.5 * width ** -0.5)
            W[f"{p}.mlp.down"] = normal(width, mlp["ff"], std=mlp["ff"] ** -0.5)
            continue
        experts, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        W[f"{p}.mlp.router"] = normal(experts, width, std=2.0 * width ** -0.5)
        W[f"{p}.mlp.router.b"] = normal(experts, std=1.0)
        names = [(f"{p}.mlp.e{e}", ff) for e in range(experts)] + ([] if mlp.get("shared") is None else [(f"{p}.mlp.shared", mlp["shared"]["ff"])])
        for base, n in names:
            W[base + ".up"] = normal(n, width, std=1.3 * width ** -0.5)
            W[base + ".down"] = normal(width, n, std=n ** -0.5)
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
    g = torch.Generator().manual_seed(2468 + seed)
    return torch.randint(0, CASES[name]["vocab"], (n,), generator=g).tolist()


#: request lengths per case: one token, a few, around pages' and windows' edges, long enough for pieces of a recurrence
LENGTHS = {"mix": {"m0": 1, "m1": 6, "m2": 23, "m3": 49, "m4": 33, "m5": 16},
           "one": {"o0": 2, "o1": 31, "o2": 17, "o3": 1, "o4": 40},
           "wide": {"w0": 5, "w1": 74, "w2": 33, "w3": 210, "w4": 50}}


def requests(name: str) -> Dict[str, List[int]]:
    return {rid: tokens(name, n, i) for i, (rid, n) in enumerate(LENGTHS[name].items())}
