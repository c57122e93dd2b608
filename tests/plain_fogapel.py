"""A plain, slow implementation of the Fogapel design: whole sequences, no cache, one function a
mechanism, float64 on the CPU by default. It shares no code with the package; the tests compare
the engine with it.

A model is (config dict, tensors dict name -> torch tensor). Notation: h [T, W] is the normed input
that a layer's two sublayers share, rows are positions 0..T-1 of one sequence.
"""
from __future__ import annotations

import torch

# The dtype an engine rounds to where it stores a result between kernels (the normed input and the
# time mixes, queries, keys and values, the heads' results in front of an output projection, a
# feed-forward's hidden values and result); None: nothing is rounded. Set by forward(round_inputs=...).
ROUND_TO = None


def stored(x):
    return x if ROUND_TO is None else x.to(ROUND_TO).to(x.dtype)


def lin(h, w, b=None):
    y = h @ w.T
    return y if b is None else y + b


def silu(z):
    return z * torch.sigmoid(z)


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


# ---- softmax attention inside chunks -----------------------------------------------------------
def short_conv(x, w):
    """x [T, C], w [C, taps]: y[s, c] = sum_j w[c, j] x[s - (taps - 1) + j, c], zeros before 0."""
    T, C = x.shape
    taps = w.shape[1]
    xp = torch.cat([torch.zeros(taps - 1, C, dtype=x.dtype), x], dim=0)
    return sum(xp[j:j + T] * w[:, j] for j in range(taps))


def rotate_pairs(x, dims, base):
    """x [T, H, D]: entries 2i and 2i + 1 (of the first ``dims``) of position p turn by
    p * base^(-2i / dims); the others pass."""
    T = x.shape[0]
    y = x.clone()
    if dims == 0:
        return y
    p = torch.arange(T, dtype=torch.float64)[:, None]
    angle = p * float(base) ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
    c, s = torch.cos(angle).to(x.dtype)[:, None, :], torch.sin(angle).to(x.dtype)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    y[..., 0:dims:2] = u * c - v * s
    y[..., 1:dims:2] = v * c + u * s
    return y


def chunk_mask(T, size):
    """[T, T]: row i sees column j <= i of its own chunk; ``size`` None: every j <= i."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if size is not None:
        seen &= torch.div(i, size, rounding_mode="floor") == torch.div(j, size, rounding_mode="floor")
    return seen


def softmax_with_one(scores, seen):
    """exp(s_j) / (1 + sum exp(s_j)) over the seen columns."""
    s = scores.masked_fill(~seen, float("-inf"))
    top = s.amax(-1, keepdim=True).clamp(min=0.0)           # (the added term has score 0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def softcap(s, cap):
    return s if not cap else cap * torch.tanh(s / cap)


def attention(h, m, t, pre, eps):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    u = {n: lin(h, t[pre + n], t[pre + n + ".b"]) for n in "qkv"}
    if m.get("conv"):
        u = {n: short_conv(x, t[pre + n + ".conv"]) for n, x in u.items()}
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    turned = lambda x, heads: stored(rms(rotate_pairs(x.view(T, heads, D), rot["dims"], rot["base"]), eps))
    q = turned(u["q"], H)
    k = turned(u["k"], G).repeat_interleave(H // G, dim=1)
    v = stored(u["v"]).view(T, G, Dv).repeat_interleave(H // G, dim=1)
    mask = m.get("mask")
    s = softcap(torch.einsum("ihd,jhd->hij", q, k) * m["scale"], m.get("softcap"))
    p = softmax_with_one(s, chunk_mask(T, None if mask is None else mask["size"]))
    o = torch.einsum("hij,jhe->ihe", p, v).reshape(T, H * Dv)
    return lin(stored(o), t[pre + "o"], t[pre + "o.b"])


# ---- the time mixer ----------------------------------------------------------------------------
def time_mix(h, mu):
    """h + (h' - h) mu, h' the row before (zeros in front of the first)."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mu


def wkv_recurrence(r, k, v, log_decay, u):
    """o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t, then S_t = diag(exp(log_decay_t)) S_(t-1) + k_t v_t^T
    from S = 0, head by head: r, k, log_decay [T, H, D], v [T, H, Dv], u [H, D]. Returns o [T, H, Dv]."""
    T, H, D = r.shape
    S = torch.zeros(H, D, v.shape[2], dtype=r.dtype)
    out = torch.zeros(T, H, v.shape[2], dtype=r.dtype)
    for s in range(T):
        kv = k[s][:, :, None] * v[s][:, None, :]
        out[s] = torch.einsum("hde,hd->he", S + u[:, :, None] * kv, r[s])
        S = torch.exp(log_decay[s])[:, :, None] * S + kv
    return out


def wkv(h, m, t, pre, eps):
    T = h.shape[0]
    H, D = m["heads"], m["dim"]
    mix = {n: stored(time_mix(h, t[pre + "mu." + n])) for n in "rkvgw"}
    r, k, v = (lin(mix[n], t[pre + n]).view(T, H, D) for n in "rkv")
    z = lin(torch.tanh(lin(mix["w"], t[pre + "w1"])), t[pre + "w2"], t[pre + "w0"]).view(T, H, D)
    o = rms(wkv_recurrence(r, k, v, -torch.exp(z), t[pre + "u"]), eps).reshape(T, H * D) * t[pre + "norm"]
    return lin(stored(o * silu(lin(mix["g"], t[pre + "g"]))), t[pre + "o"])


# ---- feed-forwards -----------------------------------------------------------------------------
def clamped_ff(h, t, pre, limit):
    g = lin(h, t[pre + "gate"]).clamp(max=limit)
    u = lin(h, t[pre + "up"]).clamp(-limit, limit)
    return lin(stored(g * torch.sigmoid(1.702 * g) * (u + 1.0)), t[pre + "down"])


def silu_ff(h, t, pre):
    return stored(lin(stored(silu(lin(h, t[pre + "gate"])) * lin(h, t[pre + "up"])), t[pre + "down"]))


def routed(h, mlp, t, pre):
    """Every token through its ``top`` experts, weighted by the softmax over their logits alone."""
    top = mlp["router"]["top"]
    z = lin(h, t[pre + "router"], t[pre + "router.b"])
    best, which = torch.topk(z, top, dim=-1)
    weight = torch.softmax(best, dim=-1)
    y = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows, place = (which == e).nonzero(as_tuple=True)
        if len(rows):
            y[rows] += weight[rows, place][:, None] * silu_ff(h[rows], t, pre + f"e{e}.")
    if mlp.get("shared") is not None:
        y = y + silu_ff(h, t, pre + "shared.")
    return y


def feed_forward(h, mlp, t, pre):
    if mlp["kind"] == "dense":
        return clamped_ff(h, t, pre, mlp["limit"])
    return routed(h, mlp, t, pre)


# ---- the model ---------------------------------------------------------------------------------
MIXERS = {"attention": attention, "wkv": wkv}


def forward(config, tensors, tokens, dtype=torch.float64, return_layers=False, round_inputs=None):
    """Logits [T, vocab] of one whole sequence (and the stream after every layer).
    ``round_inputs``: a dtype that every sublayer's input, and what an engine stores between
    kernels (see ROUND_TO), is rounded to, as an engine of that dtype rounds it (the stream itself
    is not rounded)."""
    global ROUND_TO
    ROUND_TO = round_inputs
    try:
        return _forward(config, tensors, tokens, dtype, return_layers)
    finally:
        ROUND_TO = None


def _forward(config, tensors, tokens, dtype, return_layers):
    t = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps = float(config["norm"]["eps"])
    x = t["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(config["embedding"]["scale"])
    after = []
    for i, layer in enumerate(config["layers"]):
        pre = f"l{i}."
        h = stored(rms(x, eps) * t[pre + "norm1"])
        y = MIXERS[layer["type"]](h, layer["mixer"], t, pre + "mix.", eps) * t[pre + "ls1"]
        if layer.get("mlp") is not None:
            y = y + feed_forward(h, layer["mlp"], t, pre + "mlp.") * t[pre + "ls2"]
        x = x + y
        after.append(x)
    logits = lin(stored(rms(x, eps) * t["final.norm"]), t["head"])
    return (logits, torch.stack(after)) if return_layers else logits
