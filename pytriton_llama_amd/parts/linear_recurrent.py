"""Mixers whose memory is a matrix a head that decays and takes outer products
(csrc/linear_scan.hip): Mamba-2 (one decay a head), gated linear attention (a decay a key
channel) and the time mixer of RWKV (the same with a bonus on the current token)."""
from __future__ import annotations

from typing import List, Optional

import torch

from .. import ops
from .base import ParamSource, Part, StateSpec, as_tensor, place, register_part
from .linear import LINEAR_LIBRARIES, decode_copy, linear
from .normed_attention import pad_rows


class _LinearStateMixer(Part):
    """What the first two mixers below share: one fused first projection whose result is taken in
    float32, a float32 state slot, and an output projection with a float32 result. Sequences of one
    token (the leading ones of a step) take the decode kernel, the others the chunked one."""
    kernel_libraries = ("linear_scan", "prepare") + LINEAR_LIBRARIES

    def make_decode_copies(self) -> int:
        self.proj_blocked, self.o_blocked = decode_copy(self.proj), decode_copy(self.o)
        return sum(t.numel() * t.element_size() for t in (self.proj_blocked, self.o_blocked)
                   if t is not None)

    def forward(self, x, ctx, cache):
        x = as_tensor(x)
        p = linear(x, self.proj, out_dtype=torch.float32, blocked=self.proj_blocked)
        y = torch.empty((x.shape[0], self.num_heads, self.vdim), dtype=torch.float32, device=x.device)
        n = ctx.num_decode_seqs
        if n:
            self.decode(y, p, cache.state, ctx.q_start[:n + 1], ctx.state_slots[:n])
        if n < ctx.num_seqs:
            self.portions(y, p, cache.state, ctx.q_start[n:], ctx.state_slots[n:], max(ctx.q_lens[n:]))
        return linear(self.finish(y, p, x.dtype, ctx, cache.state), self.o, out_dtype=torch.float32,
                      blocked=self.o_blocked)


@register_part("mixer", "mamba2")
class Mamba2(_LinearStateMixer):
    """Mamba-2 (Dao, Gu: "Transformers are SSMs: Generalized Models and Efficient Algorithms Through
    Structured State Space Duality"): W_in x = [z: inner | x: inner | B: G N | C: G N | dt: H], inner =
    H vdim. x, B and C together pass a short causal convolution over time ([channels, taps], the last
    tap is the current token's, with a bias) and SiLU. Per head (head h reads group h / (H / G)), with
    dt <- softplus(dt + dt_bias):

        S <- exp(-exp(A_log) dt) S + dt B x^T  [N, vdim];    y = S^T C + D x

    The heads' y times silu(z), then RMS-normed in ``norm_groups`` equal parts, times a weight
    [inner], then W_o. S and the convolution's last taps - 1 inputs live in the request's state slot
    in float32."""
    kernel_libraries = _LinearStateMixer.kernel_libraries + ("selective", "recurrent")

    def __init__(self, hidden_size: int, num_heads: int, vdim: int, state: int, groups: int, taps: int,
                 norm_groups: int, eps: float, in_name: str = "in", conv_name: str = "conv",
                 conv_bias_name: str = "conv.b", dt_bias_name: str = "dt_bias", A_log_name: str = "A_log",
                 D_name: str = "D", norm_name: str = "norm", o_name: str = "o"):
        if num_heads % groups:
            raise ValueError(f"{num_heads} heads are not a multiple of {groups} groups")
        if (num_heads * vdim) % norm_groups:
            raise ValueError(f"{norm_groups} norm groups do not divide {num_heads} heads of {vdim}")
        if state > ops.LINEAR_MAX_KEYS:
            raise ValueError(f"the recurrence kernels take up to {ops.LINEAR_MAX_KEYS} states, got {state}")
        if taps < 1:
            raise ValueError("a convolution has at least one tap")
        self.hidden_size, self.num_heads, self.vdim = int(hidden_size), int(num_heads), int(vdim)
        self.state, self.groups, self.taps = int(state), int(groups), int(taps)
        self.norm_groups, self.eps = int(norm_groups), float(eps)
        self.names = dict(i=in_name, conv=conv_name, conv_b=conv_bias_name, dt_b=dt_bias_name, A_log=A_log_name,
                          D=D_name, norm=norm_name, o=o_name)
        self.inner = self.num_heads * self.vdim
        self.channels = self.inner + 2 * self.groups * self.state
        self.x_off = self.inner                         # columns of the first projection (z at 0)
        self.b_off = 2 * self.inner
        self.c_off = self.b_off + self.groups * self.state
        self.dt_off = self.c_off + self.groups * self.state
        self.tail_off = ops.linear_state_floats(self.num_heads, self.state, self.vdim)
        self.proj = self.o = self.proj_blocked = self.o_blocked = None
        self.conv_weight = self.conv_bias = self.dt_bias = self.A_log = self.D = self.norm_weight = None

    def cache_spec(self):
        floats = self.tail_off + (self.taps - 1) * self.channels
        return StateSpec((-(-floats // 4) * 4,), torch.float32)

    def param_sources(self) -> List[ParamSource]:
        n, W, H = self.names, self.hidden_size, self.num_heads
        return [ParamSource(n["i"], (self.dt_off + H, W)),
                ParamSource(n["conv"], (self.channels, self.taps), "vector", init=("normal", 0.0, 0.5)),
                ParamSource(n["conv_b"], (self.channels,), "vector", init=("normal", 0.0, 0.1)),
                ParamSource(n["dt_b"], (H,), "vector", init=("uniform", -4.0, -1.0)),
                ParamSource(n["A_log"], (H,), "vector", init=("uniform", -1.0, 2.0)),
                ParamSource(n["D"], (H,), "vector"),
                ParamSource(n["norm"], (self.inner,), "vector"),
                ParamSource(n["o"], (W, self.inner))]

    def load(self, tensors, dtype, device) -> None:
        n = self.names
        self.proj = place(pad_rows(tensors[n["i"]]), "matrix", dtype, device)
        self.o = place(tensors[n["o"]], "matrix", dtype, device)
        for attr, key in (("conv_weight", "conv"), ("conv_bias", "conv_b"), ("dt_bias", "dt_b"), ("A_log", "A_log"),
                          ("D", "D"), ("norm_weight", "norm")):
            setattr(self, attr, place(tensors[n[key]], "vector", dtype, device))

    def decode(self, y, p, state, q_start, slots) -> None:
        ops.linear_decode_conv(y, p, self.x_off, self.b_off, self.c_off, self.dt_off, self.A_log, self.dt_bias,
                               self.D, self.conv_weight, self.conv_bias, self.tail_off, state, q_start, slots,
                               self.groups, self.state)

    def portions(self, y, p, state, q_start, slots, max_q_len) -> None:
        u, _ = ops.selective_conv(p, self.x_off, self.conv_weight, self.conv_bias, state, self.tail_off, q_start,
                                  slots, max_q_len)
        if self.taps > 1:
            ops.conv_tail_update(p, self.x_off, self.channels, self.taps, state, self.tail_off, q_start, slots)
        b = self.inner
        c = b + self.groups * self.state
        ops.linear_scan(y, u[:, c:], u[:, b:], u, self.groups, self.state, state, q_start, slots, max_q_len,
                        dt=p[:, self.dt_off:], A_log=self.A_log, dt_bias=self.dt_bias, skip=self.D)

    def finish(self, y, p, dtype, ctx, state) -> torch.Tensor:
        # (the rows of single tokens also advance their slots' kept inputs: decode() has read the old ones)
        tail = None
        if ctx.num_decode_seqs and self.taps > 1:
            tail = (state, self.tail_off, p[:, self.x_off:], self.channels, self.taps, ctx.state_slots,
                    ctx.num_decode_seqs)
        return ops.gate_group_norm(y.view(y.shape[0], self.inner), p, self.norm_weight, self.norm_groups, self.eps,
                                   dtype, tail)


@register_part("mixer", "gated_linear_attention")
class GatedLinearAttention(_LinearStateMixer):
    """Gated linear attention (Yang, Wang, Shen, Panda, Kim: "Gated Linear Attention Transformers with
    Hardware-Efficient Training"): q = W_q x * dim^-1/2, k = W_k x [heads, dim], v = W_v x [heads, vdim], a
    decay a key channel a = sigmoid(W_a2 (W_a1 x) + b)^(1 / tau), per head

        S <- diag(a) S + k v^T;    o = S^T q

    then each head's o RMS-normed with a weight [vdim] shared by the heads, times silu(W_g x), then
    W_o. S lives in the request's state slot in float32; W_a1 x is taken in float32 and W_a2 held in
    float32. ``rank``: the rows of W_a1; None: the checkpoint says (``rank_from``), and random weights
    are drawn with DEFAULT_RANK."""
    DEFAULT_RANK = 16

    def __init__(self, hidden_size: int, num_heads: int, dim: int, vdim: int, tau: float, eps: float,
                 rank: Optional[int] = None, q_name: str = "q", k_name: str = "k", v_name: str = "v",
                 g_name: str = "g", a1_name: str = "a1", a2_name: str = "a2", norm_name: str = "norm",
                 o_name: str = "o"):
        if dim > ops.LINEAR_MAX_KEYS:
            raise ValueError(f"the recurrence kernels take key sizes up to {ops.LINEAR_MAX_KEYS}, got {dim}")
        if tau <= 0:
            raise ValueError("tau must be positive")
        self.hidden_size, self.num_heads, self.dim, self.vdim = int(hidden_size), int(num_heads), int(dim), int(vdim)
        self.tau, self.eps = float(tau), float(eps)
        self.rank = int(rank) if rank else self.DEFAULT_RANK
        self.names = dict(q=q_name, k=k_name, v=v_name, g=g_name, a1=a1_name, a2=a2_name, norm=norm_name, o=o_name)
        H, D, Dv = self.num_heads, self.dim, self.vdim
        self.k_off, self.v_off = H * D, 2 * H * D
        self.g_off = 2 * H * D + H * Dv
        self.a_off = self.g_off + H * Dv
        self.proj = self.o = self.proj_blocked = self.o_blocked = None
        self.a2 = self.a2_bias = self.norm_weight = None

    def rank_from(self, prefix: str, shape_of) -> None:
        """Take the rank from the shape of the checkpoint's W_a1 (``prefix``: of this mixer's tensors)."""
        self.rank = int(shape_of(prefix + self.names["a1"])[0])

    def cache_spec(self):
        return StateSpec((ops.linear_state_floats(self.num_heads, self.dim, self.vdim),), torch.float32)

    def param_sources(self) -> List[ParamSource]:
        n, W, H, D, Dv, R = self.names, self.hidden_size, self.num_heads, self.dim, self.vdim, self.rank
        return [ParamSource(n["q"], (H * D, W)), ParamSource(n["k"], (H * D, W)), ParamSource(n["v"], (H * Dv, W)),
                ParamSource(n["g"], (H * Dv, W)), ParamSource(n["o"], (W, H * Dv)),
                ParamSource(n["norm"], (Dv,), "vector"), ParamSource(n["a1"], (R, W)),
                ParamSource(n["a2"], (H * D, R), "vector", init=("normal", 0.0, R ** -0.5)),
                ParamSource(n["a2"] + ".b", (H * D,), "vector", init=("normal", 1.0, 1.0))]

    def load(self, tensors, dtype, device) -> None:
        n = self.names
        rows = torch.cat([tensors[n[x]] for x in ("q", "k", "v", "g", "a1")], dim=0)
        self.proj = place(pad_rows(rows), "matrix", dtype, device)
        self.o = place(tensors[n["o"]], "matrix", dtype, device)
        self.a2 = place(tensors[n["a2"]], "vector", dtype, device)
        self.a2_bias = place(tensors[n["a2"] + ".b"], "vector", dtype, device)
        self.norm_weight = place(tensors[n["norm"]], "vector", dtype, device)

    def decode(self, y, p, state, q_start, slots) -> None:
        ops.linear_decode_lowrank(y, p, 0, self.k_off, self.v_off, self.a_off, self.dim ** -0.5, self.a2, self.a2_bias,
                                  self.tau, state, q_start, slots, self.dim)

    def portions(self, y, p, state, q_start, slots, max_q_len) -> None:
        decay = ops.lowrank_decay(p[:, self.a_off:], self.a2, self.a2_bias, self.tau)
        ops.linear_scan(y, p, p[:, self.k_off:], p[:, self.v_off:], self.num_heads, self.dim, state, q_start, slots,
                        max_q_len, qscale=self.dim ** -0.5, decay=decay)

    def finish(self, y, p, dtype, ctx, state) -> torch.Tensor:
        out = torch.empty((y.shape[0], self.num_heads * self.vdim), dtype=dtype, device=y.device)
        ops.head_norm_gate(out, y, 1, 0.0, self.norm_weight, False, 1.0, p, self.g_off, ops.GATE_SILU, self.eps)
        return out


@register_part("mixer", "time_mixer")
class TimeMixer(Part):
    """The time mixer of RWKV-6 (Peng et al.: "Eagle and Finch: RWKV with Matrix-Valued States and
    Dynamic Recurrence"), without its data-dependent mixing: with x' the token's row before (zeros in front of
    the first), each of r, k, v, g, w reads its own mix x + (x' - x) mu; r, k, v [heads, dim] are W_r, W_k,
    W_v of theirs, the decay a key channel is a = exp(-exp(W_w2 tanh(W_w1 mix_w) + w0)), per head

        o = (S + diag(u) k v^T)^T r;    S <- diag(a) S + k v^T

    then each head's o divided by its root mean square, times a weight of all heads' size, times silu(W_g
    mix_g), then W_o. S and the last row x live in the request's state slot in float32; W_w1's result is
    taken in float32 and W_w2 held in float32. ``rank``: the rows of W_w1; None: the checkpoint says
    (``rank_from``), and random weights are drawn with DEFAULT_RANK."""
    kernel_libraries = ("linear_scan", "prepare") + LINEAR_LIBRARIES
    DEFAULT_RANK = 16
    MIXES = ("r", "k", "v", "g", "w")          # the order of the projections' rows (w: those of W_w1)

    def __init__(self, hidden_size: int, num_heads: int, dim: int, eps: float, rank: Optional[int] = None,
                 mu_prefix: str = "mu.", r_name: str = "r", k_name: str = "k", v_name: str = "v", g_name: str = "g",
                 w1_name: str = "w1", w2_name: str = "w2", w0_name: str = "w0", u_name: str = "u",
                 norm_name: str = "norm", o_name: str = "o"):
        if dim > ops.LINEAR_MAX_KEYS:
            raise ValueError(f"the recurrence kernels take key sizes up to {ops.LINEAR_MAX_KEYS}, got {dim}")
        self.hidden_size, self.num_heads, self.dim, self.eps = int(hidden_size), int(num_heads), int(dim), float(eps)
        self.rank = int(rank) if rank else self.DEFAULT_RANK
        self.mu_prefix = mu_prefix
        self.names = dict(r=r_name, k=k_name, v=v_name, g=g_name, w1=w1_name, w2=w2_name, w0=w0_name, u=u_name,
                          norm=norm_name, o=o_name)
        self.size = self.num_heads * self.dim
        self.cols = -(-self.size // 16) * 16   # columns of a projection in their common result (padded)
        self.x_off = ops.linear_state_floats(self.num_heads, self.dim, self.dim)       # the kept row in a slot
        self.proj = self.o = self.proj_blocked = self.o_blocked = None
        self.mu = self.w2 = self.w0 = self.bonus = self.norm_weight = None

    def rank_from(self, prefix: str, shape_of) -> None:
        """Take the rank from the shape of the checkpoint's W_w1 (``prefix``: of this mixer's tensors)."""
        self.rank = int(shape_of(prefix + self.names["w1"])[0])

    def cache_spec(self):
        return StateSpec((-(-(self.x_off + self.hidden_size) // 4) * 4,), torch.float32)

    def param_sources(self) -> List[ParamSource]:
        n, W, C, R = self.names, self.hidden_size, self.size, self.rank
        return [ParamSource(self.mu_prefix + m, (W,), "vector", init=("uniform", 0.0, 1.0)) for m in self.MIXES] + \
               [ParamSource(n[x], (C, W)) for x in ("r", "k", "v", "g")] + \
               [ParamSource(n["w1"], (R, W)), ParamSource(n["w2"], (C, R), "vector", init=("normal", 0.0, R ** -0.5)),
                ParamSource(n["w0"], (C,), "vector", init=("uniform", -6.0, 0.5)),
                ParamSource(n["u"], (self.num_heads, self.dim), "vector", init=("normal", 0.0, 0.5)),
                ParamSource(n["norm"], (C,), "vector"), ParamSource(n["o"], (W, C))]

    def load(self, tensors, dtype, device) -> None:
        n = self.names
        rows = [pad_rows(tensors[n[x]], 16) for x in ("r", "k", "v", "g", "w1")]
        self.proj = place(torch.cat(rows, dim=0), "matrix", dtype, device)
        self.o = place(tensors[n["o"]], "matrix", dtype, device)
        self.mu = place(torch.stack([tensors[self.mu_prefix + m] for m in self.MIXES]), "vector", dtype, device)
        for attr, key in (("w2", "w2"), ("w0", "w0"), ("bonus", "u"), ("norm_weight", "norm")):
            setattr(self, attr, place(tensors[n[key]], "vector", dtype, device))

    def make_decode_copies(self) -> int:
        self.proj_blocked, self.o_blocked = decode_copy(self.proj), decode_copy(self.o)
        return sum(t.numel() * t.element_size() for t in (self.proj_blocked, self.o_blocked)
                   if t is not None)

    def mixes(self, ctx, cache):
        """What the norm in front of this mixer needs to make its inputs as well (ops.TimeMixes), for a step
        that brings single tokens only; None for any other step."""
        if ctx.num_decode_seqs != ctx.num_seqs:
            return None
        return ops.TimeMixes(self.mu, cache.state, self.x_off, ctx.state_slots)

    def forward(self, x, ctx, cache, mixed=None):
        """``mixed``: the inputs [5, T, hidden], when the norm in front has made them (``mixes``)."""
        x, state = as_tensor(x), cache.state
        T, H, D, c = x.shape[0], self.num_heads, self.dim, self.cols
        if mixed is None:
            mixed = ops.time_shift(x, self.mu, state, self.x_off, ctx.q_start, ctx.state_slots)
        p = ops.gemm_groups(mixed, self.proj, c, self.proj_blocked)
        o = torch.empty((T, H, D), dtype=torch.float32, device=x.device)
        out = torch.empty((T, H * D), dtype=x.dtype, device=x.device)
        keep = (x, self.x_off)              # (the recurrences' kernels leave the last rows in the slots)
        n = ctx.num_decode_seqs
        finish = None
        if n == ctx.num_seqs and D <= ops.LINEAR_HEAD_FUSED:
            finish = (out, self.norm_weight, 3 * c, self.eps)
        if n:
            ops.linear_decode_bonus(o, p, 0, c, 2 * c, 4 * c, self.w2, self.w0, self.bonus, state, ctx.q_start[:n + 1],
                                    ctx.state_slots[:n], D, keep, finish)
        if n < ctx.num_seqs:
            decay = ops.lowrank_decay(p[:, 4 * c:], self.w2, self.w0, form=ops.DECAY_EXP)
            ops.linear_scan(o, p, p[:, c:], p[:, 2 * c:], H, D, state, ctx.q_start[n:], ctx.state_slots[n:],
                            max(ctx.q_lens[n:]), decay=decay, bonus=self.bonus, keep=keep)
        if finish is None:
            ops.head_norm_gate(out, o, 1, 0.0, self.norm_weight, True, 1.0, p, 3 * c, ops.GATE_SILU, self.eps)
        return linear(out, self.o, out_dtype=torch.float32, blocked=self.o_blocked)
