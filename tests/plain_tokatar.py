"""The Tokatar design written out plainly in float64, one function per mechanism.  It shares no code with the product:
tensors come as a dict name -> tensor, the configuration as the dict that config.json holds.  Slow on purpose.

Notation: x is the residual stream [T, W]; u is a sublayer's input, the normed stream.  A sublayer f with the gate
r = sigmoid(R u + b), the norm behind it and the vector s does  x <- x + s * norm(r * f(u)).
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def over_rms(x, eps):
    """x over the root of (mean of squares + eps), along the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def scalar_norm(x, g, eps):
    """RMS norm whose weight is one number for the whole row."""
    return over_rms(x, eps) * g.reshape(())


def stream_gate(u, R, b):
    """What multiplies a sublayer's result, element by element."""
    return torch.sigmoid(u @ R.T + b)


# ---- rotations ----------------------------------------------------------------------------------------------
def frequencies(dims, base):
    return torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)


def stretched(freq, factor, low, high, original):
    """The rule that keeps short wavelengths, divides the frequencies of long ones by ``factor`` and blends between."""
    out = freq.clone()
    for i, f in enumerate(freq.tolist()):
        wave = 2.0 * math.pi / f
        if wave < original / high:
            continue
        if wave > original / low:
            out[i] = f / factor
        else:
            s = (original / wave - low) / (high - low)
            out[i] = (1.0 - s) * f / factor + s * f
    return out


def key_frequencies(rot):
    f = frequencies(int(rot["dims"]), float(rot["base"]))
    s = rot.get("scaling")
    return f if s is None else stretched(f, float(s["factor"]), float(s["low"]), float(s["high"]), float(s["original"]))


def pair_places(dims, layout):
    """The two element indices of every pair: ``halves`` (i, i + dims / 2) or ``neighbours`` (2 i, 2 i + 1)."""
    i = torch.arange(dims // 2)
    return (i, i + dims // 2) if layout == "halves" else (2 * i, 2 * i + 1)


def turn(x, freq, layout, sign=1.0):
    """x [T, heads, D]: pair i of the first 2 len(freq) elements turned by sign * position * freq[i]; the rest as it is."""
    T = x.shape[0]
    a, b = pair_places(2 * len(freq), layout)
    angle = sign * torch.arange(T, dtype=F64)[:, None, None] * freq[None, None, :]
    out = x.clone()
    out[..., a] = x[..., a] * torch.cos(angle) - x[..., b] * torch.sin(angle)
    out[..., b] = x[..., b] * torch.cos(angle) + x[..., a] * torch.sin(angle)
    return out


# ---- scores and softmax ---------------------------------------------------------------------------------------
def visible(T, chunk=None):
    """Boolean [T, T]: query i sees key j when j <= i and, with chunks, both lie in the same chunk of positions."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    if chunk is not None:
        ok = ok & (i // chunk == j // chunk)
    return ok


def capped(scores, cap):
    return scores if cap is None else float(cap) * torch.tanh(scores / float(cap))


def softmax_plus(scores, mask, extra):
    """Weights exp(s_j) / (extra + sum of exp(s_j)) over the visible keys; ``extra`` 0: the ordinary softmax."""
    s = scores.masked_fill(~mask[None], -math.inf)
    top = s.amax(dim=-1, keepdim=True)
    if extra:
        top = torch.clamp(top, min=0.0)
    e = torch.exp(s - top)
    return e / (e.sum(dim=-1, keepdim=True) + extra * torch.exp(-top))


def attend(q, k, v, scale, mask, cap=None, extra=0.0):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]."""
    H, G = q.shape[1], k.shape[1]
    out = torch.zeros(q.shape[0], H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        scores = capped((q[:, h] @ k[:, g].T) * scale, cap)
        out[:, h] = softmax_plus(scores[None], mask, extra)[0] @ v[:, g]
    return out


# ---- mixers -----------------------------------------------------------------------------------------------------
def attention(u, W, p, c, eps):
    T = u.shape[0]
    H, G, D, E = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = (u @ W[p + ".q"].T).reshape(T, H, D)
    k = (u @ W[p + ".k"].T).reshape(T, G, D)
    v = (u @ W[p + ".v"].T).reshape(T, G, E)
    if c.get("rot") is not None:
        f = key_frequencies(c["rot"])
        q, k = turn(q, f, "halves"), turn(k, f, "halves")
    mask = visible(T, None if c.get("mask") is None else int(c["mask"]["size"]))
    o = attend(q, k, v, float(c["scale"]), mask, c.get("softcap")).reshape(T, H * E)
    return (o * torch.sigmoid(u @ W[p + ".g"].T)) @ W[p + ".o"].T


def attention_2(u, W, p, c, eps):
    T = u.shape[0]
    H, G, D, E = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = over_rms(u @ W[p + ".q"].T + W[p + ".q.b"], eps) * W[p + ".q.norm"]
    k = over_rms(u @ W[p + ".k"].T + W[p + ".k.b"], eps) * W[p + ".k.norm"]
    v = (u @ W[p + ".v"].T + W[p + ".v.b"]).reshape(T, G, E)
    q, k = q.reshape(T, H, D), k.reshape(T, G, D)
    f = key_frequencies(c["rot"])
    q, k = turn(q, f, "neighbours"), turn(k, f, "neighbours")
    fv = frequencies(E, float(c["rot"]["base"]))
    v = turn(v, fv, "neighbours")
    mask = visible(T, None if c.get("mask") is None else int(c["mask"]["size"]))
    o = attend(q, k, v, float(c["scale"]), mask, c.get("softcap"), extra=1.0)
    o = turn(o, fv, "neighbours", sign=-1.0).reshape(T, H * E)
    return (o * torch.sigmoid(u @ W[p + ".g"].T)) @ W[p + ".o"].T


def latent_attention(u, W, p, c, eps):
    T = u.shape[0]
    H, D, R, E, L = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    q = (u @ W[p + ".q"].T).reshape(T, H, D + R)
    down = u @ W[p + ".dkv"].T
    latent = over_rms(down[:, :L], eps) * W[p + ".dkv.norm"]
    f = key_frequencies(c["rot"])
    shared = turn(down[:, None, L:], f, "halves")
    k = torch.cat([(latent @ W[p + ".uk"].T).reshape(T, H, D), shared.expand(T, H, R)], dim=-1)
    q = torch.cat([q[..., :D], turn(q[..., D:], f, "halves")], dim=-1)
    v = (latent @ W[p + ".uv"].T).reshape(T, H, E)
    o = attend(q, k, v, float(c["scale"]), visible(T))
    o = o * torch.sigmoid(u @ W[p + ".g"].T)[:, :, None]
    return o.reshape(T, H * E) @ W[p + ".o"].T


MIXERS = {"attention": attention, "attention_2": attention_2, "latent_attention": latent_attention}


def dense_ff(u, W, p):
    return torch.clamp(u @ W[p + ".up"].T, min=0.0) ** 2 @ W[p + ".down"].T


# ---- the model ----------------------------------------------------------------------------------------------
def closing(x, y, u, W, p, n, eps):
    """The stream after sublayer ``n`` (1: the mixer, 2: the feed-forward) of layer ``p`` with input u and result y."""
    y = y * stream_gate(u, W[f"{p}.rg{n}"], W[f"{p}.rg{n}.b"])
    return x + W[f"{p}.ls{n}"] * scalar_norm(y, W[f"{p}.norm{n}b"], eps)


def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives the stream after every layer."""
    W = {k: (v.to(F64) if v.is_floating_point() else v) for k, v in W.items()}
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.tensor(tokens)] * float(cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        u = scalar_norm(x, W[p + ".norm1"], eps)
        x = closing(x, MIXERS[layer["type"]](u, W, p + ".mix", layer["mixer"], eps), u, W, p, 1, eps)
        if layer.get("mlp") is not None:
            u = scalar_norm(x, W[p + ".norm2"], eps)
            x = closing(x, dense_ff(u, W, p + ".mlp"), u, W, p, 2, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return scalar_norm(x, W["final.norm"], eps) @ W["head"].T


def greedy(config, weights, prompt, n_new):
    """The tokens that greedy decoding appends to ``prompt`` (the whole sequence is run anew for every token)."""
    toks = list(prompt)
    for _ in range(n_new):
        toks.append(int(torch.argmax(forward(config, weights, toks)[-1])))
    return toks[len(prompt):]


def logit_error(got, ref):
    """Largest difference between two sets of logits after taking each row's mean off, relative to the reference's
    spread."""
    g, r = got.to(F64).cpu(), ref.to(F64)
    d = (g - g.mean(-1, keepdim=True)) - (r - r.mean(-1, keepdim=True))
    return float(d.abs().max() / r.std())
