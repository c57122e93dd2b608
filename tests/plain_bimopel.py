"""A plain, slow implementation of the Bimopel design: whole sequences, no cache, one function a
mechanism, float64 on the CPU by default. It shares no code with the package; the tests compare
the engine with it.

A model is (config dict, tensors dict name -> torch tensor). Notation: h [T, W] is a sublayer's
input, rows are positions 0..T-1 of one sequence.
"""
from __future__ import annotations

import math

import torch

# The dtype an engine rounds to where it stores a result between kernels (queries, keys and values,
# the heads' results in front of an output projection, a feed-forward's hidden values and result);
# None: nothing is rounded. Set by forward(round_inputs=...).
ROUND_TO = None


def stored(x):
    return x if ROUND_TO is None else x.to(ROUND_TO).to(x.dtype)


def lin(h, w, b=None):
    y = h @ w.T
    return y if b is None else y + b


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


# ---- in front of the layers --------------------------------------------------------------------
def position_vectors(T, width, dtype=torch.float64):
    """[T, width]: entry 2i is sin(p / 10000^(2i / width)), entry 2i + 1 the cosine of it."""
    p = torch.arange(T, dtype=torch.float64)[:, None]
    e = torch.arange(width)
    angle = p * 10000.0 ** (-(2.0 * torch.div(e, 2, rounding_mode="floor")).double() / width)
    return torch.where(e % 2 == 0, torch.sin(angle), torch.cos(angle)).to(dtype)


def embed(t, tokens, scale):
    rows = t["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    return rows * scale + position_vectors(rows.shape[0], rows.shape[1], rows.dtype)


# ---- softmax attention inside chunks -----------------------------------------------------------
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


def chunk_attention(h, m, t, pre, eps):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms(lin(h, t[pre + "q"], t[pre + "q.b"]), eps) * t[pre + "q.norm"]
    k = rms(lin(h, t[pre + "k"], t[pre + "k.b"]), eps) * t[pre + "k.norm"]
    v = lin(h, t[pre + "v"], t[pre + "v.b"])
    q = stored(q).view(T, H, D)
    k = stored(k).view(T, G, D).repeat_interleave(H // G, dim=1)
    v = stored(v).view(T, G, Dv).repeat_interleave(H // G, dim=1)
    mask = m.get("mask")
    p = softmax_with_one(torch.einsum("ihd,jhd->hij", q, k) * m["scale"],
                         chunk_mask(T, None if mask is None else mask["size"]))
    o = torch.einsum("hij,jhe->ihe", p, v) * torch.sigmoid(lin(h, t[pre + "g"]))[:, :, None]
    return lin(stored(o.reshape(T, H * Dv)), t[pre + "o"])


# ---- matrices carried from token to token --------------------------------------------------------
def linear_recurrence(q, k, v, log_decay):
    """S_t = diag(exp(log_decay_t)) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t from S = 0, head by head:
    q, k [T, H, D], v [T, H, Dv], log_decay [T, H, D] (or [T, H, 1]). Returns o [T, H, Dv]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for s in range(T):
        S = torch.exp(log_decay[s])[:, :, None] * S + k[s][:, :, None] * v[s][:, None, :]
        out[s] = torch.einsum("hde,hd->he", S, q[s])
    return out


def gated_linear_attention(h, m, t, pre, eps):
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    q = lin(h, t[pre + "q"]).view(T, H, D) * D ** -0.5
    k = lin(h, t[pre + "k"]).view(T, H, D)
    v = lin(h, t[pre + "v"]).view(T, H, Dv)
    z = lin(lin(h, t[pre + "a1"]), t[pre + "a2"], t[pre + "a2.b"]).view(T, H, D)
    o = linear_recurrence(q, k, v, torch.nn.functional.logsigmoid(z) / m["tau"])
    o = (rms(o, eps) * t[pre + "norm"]).reshape(T, H * Dv) * silu(lin(h, t[pre + "g"]))
    return lin(stored(o), t[pre + "o"])


def short_conv(x, w, b):
    """x [T, C], w [C, taps]: y[s, c] = b[c] + sum_j w[c, j] x[s - (taps - 1) + j, c], zeros before 0."""
    T, C = x.shape
    taps = w.shape[1]
    xp = torch.cat([torch.zeros(taps - 1, C, dtype=x.dtype), x], dim=0)
    return sum(xp[j:j + T] * w[:, j] for j in range(taps)) + b


def mamba2(h, m, t, pre, eps):
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = torch.split(lin(h, t[pre + "in"]), [inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(short_conv(xbc, t[pre + "conv"], t[pre + "conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=1)
    x = x.reshape(T, H, P)
    B = B.reshape(T, G, N).repeat_interleave(H // G, dim=1)
    C = C.reshape(T, G, N).repeat_interleave(H // G, dim=1)
    dt = torch.nn.functional.softplus(dt + t[pre + "dt_bias"])
    y = linear_recurrence(C, B * dt[:, :, None], x, (-torch.exp(t[pre + "A_log"]) * dt)[:, :, None])
    y = (y + t[pre + "D"][:, None] * x).reshape(T, inner) * silu(z)
    parts = m["norm_groups"]
    y = rms(y.reshape(T, parts, inner // parts), eps).reshape(T, inner) * t[pre + "norm"]
    return lin(stored(y), t[pre + "o"])


def parallel(h, m, t, pre, eps):
    left = rms(chunk_attention(h, m["left"], t, pre + "left.", eps), eps) * t[pre + "left.out"]
    right = rms(gated_linear_attention(h, m["right"], t, pre + "right.", eps), eps) * t[pre + "right.out"]
    return 0.5 * (left + right)


def dense_ff(h, t, pre):
    return stored(lin(stored(gelu_tanh(lin(h, t[pre + "gate"])) * lin(h, t[pre + "up"])), t[pre + "down"]))


# ---- the model ---------------------------------------------------------------------------------
MIXERS = {"mamba2": mamba2, "parallel": parallel}


def softcap(logits, cap):
    return logits if not cap else cap * torch.tanh(logits / cap)


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
    eps, alpha = float(config["norm"]["eps"]), float(config["postln_alpha"])
    x = embed(t, tokens, float(config["embedding"]["scale"]))
    after = []
    for i, layer in enumerate(config["layers"]):
        pre = f"l{i}."
        y = MIXERS[layer["type"]](stored(x), layer["mixer"], t, pre + "mix.", eps)
        x = rms(alpha * x + y, eps) * t[pre + "norm1"]
        if layer.get("mlp") is not None:
            x = rms(alpha * x + dense_ff(stored(x), t, pre + "mlp."), eps) * t[pre + "norm2"]
        after.append(x)
    logits = softcap(lin(stored(rms(x, eps) * t["final.norm"]), t["head"]), config.get("logit_softcap"))
    return (logits, torch.stack(after)) if return_layers else logits
