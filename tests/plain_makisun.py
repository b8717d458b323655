"""The Makisun design written out plainly in float64, one function per mechanism, token by token where the design is
recurrent.  It shares no code with the product: tensors come as a dict name -> tensor, the configuration as the dict that
config.json holds.  Slow on purpose.

Notation: x is the residual stream [T, W]; u is a sublayer's input (the normed stream); a layer is
x += ls1 * mixer(norm1(x)), then x += ls2 * ff(norm2(x)) when it has a feed-forward.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def over_rms(x, eps):
    """x over the root of (mean of squares + eps), along the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm_around_zero(x, w, eps):
    """RMS norm whose stored weight is the deviation from one."""
    return over_rms(x, eps) * (1.0 + w)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def relu_squared(z):
    return torch.clamp(z, min=0.0) ** 2


# ---- mixer: wkv ---------------------------------------------------------------------------------------------
def shifted(u):
    """Every row's predecessor in its sequence; zeros in front of the first."""
    return torch.cat([torch.zeros_like(u[:1]), u[:-1]], dim=0)


def blend(u, mu):
    """A mix of a token's row and the row before it: mu 0 is the token's own, mu 1 the one before."""
    return u + (shifted(u) - u) * mu


def wkv_decay(rows, w1, w2, w0):
    """exp(-exp(w2 tanh(w1 x) + w0)), between 0 and 1 for every channel."""
    return torch.exp(-torch.exp(torch.tanh(rows @ w1.T) @ w2.T + w0))


def wkv_chain(r, k, v, w, bonus):
    """r, k, w [T, H, D]; v [T, H, E] (here E = D); bonus [H, D].  Per head, with S [key, value] from zero, a token reads the
    state as the token before left it plus its own k v^T with every key channel times the bonus; then S <- diag(w) S + k v^T."""
    T, H, D = r.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        own = k[t][:, :, None] * v[t][:, None, :]
        out[t] = ((S + bonus[:, :, None] * own) * r[t][:, :, None]).sum(1)
        S = w[t][:, :, None] * S + own
    return out


def wkv(u, W, p, c, eps):
    T = u.shape[0]
    H, D = c["heads"], c["dim"]
    part = lambda name: blend(u, W[f"{p}.mu.{name}"])
    r, k, v = ((part(n) @ W[f"{p}.{n}"].T).reshape(T, H, D) for n in ("r", "k", "v"))
    gate = silu(part("g") @ W[p + ".g"].T)
    w = wkv_decay(part("w"), W[p + ".w1"], W[p + ".w2"], W[p + ".w0"]).reshape(T, H, D)
    o = over_rms(wkv_chain(r, k, v, w, W[p + ".u"]), eps).reshape(T, H * D)
    return (o * W[p + ".norm"] * gate) @ W[p + ".o"].T


# ---- mixer: parallel, left ------------------------------------------------------------------------------------
def frequencies(dims, base):
    return base ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)


def rotate(x, freqs, dims):
    """x [T, heads, D] at positions 0 .. T - 1: element i of the first ``dims`` of a head turns with element i + dims / 2."""
    T, half = x.shape[0], dims // 2
    ang = torch.arange(T, dtype=F64)[:, None] * freqs[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    a, b = x[..., :half], x[..., half:dims]
    return torch.cat([a * c - b * s, b * c + a * s, x[..., dims:]], dim=-1)


def visible(T, window=None):
    """Boolean [T, T]: query i sees key j when 0 <= i - j and (with a window) i - j < window."""
    gap = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (gap >= 0) if window is None else (gap >= 0) & (gap < window)


def attend(q, k, v, scale, ok):
    """Softmax attention of [T, H, D] queries over [T, G, D] keys; query head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        out[:, h] = torch.softmax(s.masked_fill(~ok, -math.inf), dim=-1) @ v[:, h // per]
    return out


def left(u, W, p, c, eps):
    T = u.shape[0]
    H, G, D, E = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = over_rms((u @ W[p + ".q"].T).reshape(T, H, D), eps) * W[p + ".q.norm"]
    k = over_rms((u @ W[p + ".k"].T).reshape(T, G, D), eps) * W[p + ".k.norm"]
    v = (u @ W[p + ".v"].T).reshape(T, G, E)
    rot, mask = c.get("rot"), c.get("mask")
    if rot is not None:
        f = frequencies(rot["dims"], float(rot["base"]))
        q, k = rotate(q, f, rot["dims"]), rotate(k, f, rot["dims"])
    o = attend(q, k, v, float(c["scale"]), visible(T, None if mask is None else int(mask["size"])))
    o = o * torch.sigmoid(u @ W[p + ".g"].T)[:, :, None]
    return o.reshape(T, H * E) @ W[p + ".o"].T


# ---- mixer: parallel, right -----------------------------------------------------------------------------------
def root_decay(u, a1, a2, bias, tau):
    """sigmoid(z) to the power 1 / tau, z = a2 (a1 u) + bias."""
    return torch.sigmoid((u @ a1.T) @ a2.T + bias) ** (1.0 / tau)


def gla_chain(q, k, v, alpha):
    """q, k, alpha [T, H, D]; v [T, H, E].  S <- diag(alpha) S + k v^T, then the token reads S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def right(u, W, p, c, eps):
    T = u.shape[0]
    H, D, E = c["heads"], c["dim"], c["vdim"]
    q = (u @ W[p + ".q"].T).reshape(T, H, D) * D ** -0.5
    k = (u @ W[p + ".k"].T).reshape(T, H, D)
    v = (u @ W[p + ".v"].T).reshape(T, H, E)
    alpha = root_decay(u, W[p + ".a1"], W[p + ".a2"], W[p + ".a2.b"], float(c["tau"])).reshape(T, H, D)
    o = over_rms(gla_chain(q, k, v, alpha), eps) * W[p + ".norm"]
    return (o.reshape(T, H * E) * silu(u @ W[p + ".g"].T)) @ W[p + ".o"].T


def parallel(u, W, p, c, eps):
    return float(c["left_scale"]) * left(u, W, p + ".left", c["left"], eps) + \
        float(c["right_scale"]) * right(u, W, p + ".right", c["right"], eps)


MIXERS = {"wkv": wkv, "parallel": parallel}


# ---- feed-forwards --------------------------------------------------------------------------------------------------
def dense_ff(u, W, p):
    return gelu_erf(u @ W[p + ".up"].T) @ W[p + ".down"].T


def expert(u, W, p):
    return relu_squared(u @ W[p + ".up"].T) @ W[p + ".down"].T


def route(u, W, p, top):
    """(ids [T, top], weights [T, top]): the ``top`` largest logits (the lower index wins a tie) and a softmax over
    those logits alone."""
    z = u @ W[p + ".router"].T + W[p + ".router.b"]
    ids = torch.tensor([sorted(range(z.shape[1]), key=lambda e: (-float(row[e]), e))[:top] for row in z])
    return ids, torch.softmax(torch.gather(z, 1, ids), dim=-1)


def moe_ff(u, W, p, c):
    ids, weights = route(u, W, p, int(c["router"]["top"]))
    y = torch.zeros(u.shape[0], W[p + ".e0.down"].shape[0], dtype=F64)
    for t in range(u.shape[0]):
        for e, w in zip(ids[t].tolist(), weights[t]):
            y[t] += w * expert(u[t], W, f"{p}.e{e}")
    return y if c.get("shared") is None else y + expert(u, W, p + ".shared")


def feed_forward(u, W, p, c):
    return dense_ff(u, W, p) if c["kind"] == "dense" else moe_ff(u, W, p, c)


# ---- the model ----------------------------------------------------------------------------------------------
def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives the stream after every layer."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.tensor(list(tokens))] * float(cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        u = norm_around_zero(x, W[p + ".norm1"], eps)
        x = x + W[p + ".ls1"] * MIXERS[layer["type"]](u, W, p + ".mix", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            u = norm_around_zero(x, W[p + ".norm2"], eps)
            x = x + W[p + ".ls2"] * feed_forward(u, W, p + ".mlp", layer["mlp"])
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm_around_zero(x, W["final.norm"], eps) @ W["head"].T


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
