"""Each kernel that Bimopel added or widened, alone, against tests/plain_bimopel.py or a few lines of
float64."""
import pytest
import torch

import plain_bimopel as plain

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]


def dev(t, dtype=torch.float32):
    return t.to(dtype).cuda().contiguous()


def i32(values):
    return torch.tensor(values, dtype=torch.int32, device="cuda")


def close(got, want, tol):
    got = got.double().cpu()
    top = max(float(want.abs().max()), 1e-30)
    err = float((got - want).abs().max()) / top
    assert err < tol, err


# ---- linear recurrences ------------------------------------------------------------------------
# (heads, q/k heads, D, Dv); scalar form with groups, channel form with a q/k head a head
SCALAR_SIZES = [(4, 2, 16, 16), (3, 1, 20, 24), (2, 2, 7, 5), (6, 3, 64, 64), (2, 1, 136, 70), (1, 1, 256, 33),
                (4, 1, 128, 64)]
CHANNEL_SIZES = [(2, 16, 16), (3, 20, 28), (1, 13, 9), (2, 64, 64), (2, 128, 130), (1, 200, 40), (1, 256, 16)]


def scalar_case(H, G, D, Dv, T, seed, pad=0, strong=False):
    """Columns of one float32 matrix (v | k | q | dt, ``pad`` columns in front) and the plain result."""
    g = torch.Generator().manual_seed(seed)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    m = rn(T, pad + H * Dv + 2 * G * D + H).float().double()
    A_log = (torch.rand(H, generator=g, dtype=torch.float64) * (6 if strong else 3) - 1).float().double()
    dt_bias, skip = rn(H).float().double(), rn(H).float().double()
    if strong:                             # a few tokens that wipe the state, between ones that keep it
        m[:, -H:] -= 6.0
        m[::7, -H:] += 26.0
    v = m[:, pad:pad + H * Dv].view(T, H, Dv)
    k = m[:, pad + H * Dv:pad + H * Dv + G * D].view(T, G, D).repeat_interleave(H // G, 1)
    q = m[:, pad + H * Dv + G * D:pad + H * Dv + 2 * G * D].view(T, G, D).repeat_interleave(H // G, 1)
    dt = torch.nn.functional.softplus(m[:, -H:] + dt_bias)
    want = plain.linear_recurrence(q, k * dt[:, :, None], v, (-torch.exp(A_log) * dt)[:, :, None])
    return m, A_log, dt_bias, skip, want + skip[:, None] * v


def channel_case(H, D, Dv, T, seed, pad=0, strong=False):
    g = torch.Generator().manual_seed(seed)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    m = rn(T, pad + 2 * H * D + H * Dv).float().double()
    z = rn(T, H * D) * 2
    if strong:                             # decays down to e^-80 a token beside ones near 1
        z = z * 20
    decay = torch.sigmoid(z).pow(1.0 / (1.0 if strong else 8.0)).float().double()
    q = m[:, pad:pad + H * D].view(T, H, D) * D ** -0.5
    k = m[:, pad + H * D:pad + 2 * H * D].view(T, H, D)
    v = m[:, pad + 2 * H * D:].reshape(T, H, Dv)
    log_decay = torch.log(decay.clamp_min(1e-300)).view(T, H, D)
    return m, decay, plain.linear_recurrence(q, k, v, log_decay)


def run_scan(ops, lens, cuts, make_call, H, D, Dv, slots, seg_len=0, max_num=6, extra=0):
    """Sequences of ``lens`` rows advanced together: round i brings cuts[i][s] rows of sequence s.
    ``make_call(rows, out, q_start, slots, max_q_len)`` runs the kernel on the gathered rows."""
    floats = ops.linear_state_floats(H, D, Dv) + extra
    state = torch.full((max_num + 1, -(-floats // 4) * 4), 7.5, dtype=torch.float32, device="cuda")
    for s in slots:
        state[s] = 0
    start = [sum(lens[:i]) for i in range(len(lens))]
    done = [0] * len(lens)
    out = torch.full((sum(lens), H, Dv), float("nan"), device="cuda")
    for cut in cuts:
        rows, q_start, who = [], [0], []
        for s, n in enumerate(cut):
            n = min(n, lens[s] - done[s])
            if n <= 0:
                continue
            rows += list(range(start[s] + done[s], start[s] + done[s] + n))
            q_start.append(len(rows))
            who.append(slots[s])
            done[s] += n
        if not rows:
            continue
        part = torch.full((len(rows), H, Dv), float("nan"), device="cuda")
        make_call(torch.tensor(rows), part, i32(q_start), i32(who), max(b - a for a, b in zip(q_start, q_start[1:])),
                  state)
        out[torch.tensor(rows).cuda()] = part
    assert done == list(lens)
    untouched = [s for s in range(max_num + 1) if s not in slots]
    assert bool((state[untouched] == 7.5).all())
    return out, state


CUTS = {
    "whole": [[10 ** 6] * 4],
    "portions": [[2, 31, 64, 5], [33, 3, 2, 1], [1, 1, 100, 32], [17, 40, 2, 2], [200, 200, 200, 200]],
    "ones": [[5, 1, 30, 16]] + [[1, 1, 1, 1]] * 40 + [[300] * 4],
}


@pytest.mark.parametrize("cut", sorted(CUTS))
@pytest.mark.parametrize("sizes", SCALAR_SIZES, ids=str)
def test_scalar_scan(gpu_device, sizes, cut):
    from pytriton_llama_amd import ops
    H, G, D, Dv = sizes
    lens = [70, 131, 260, 33]
    pad = 3 if D % 4 else 4
    cases = [scalar_case(H, G, D, Dv, n, 100 + i, pad) for i, n in enumerate(lens)]
    m = torch.cat([c[0] for c in cases])
    A_log, dt_bias, skip = cases[0][1:4]
    want = []
    for n, c in zip(lens, cases):           # one set of head constants for all sequences
        v = c[0][:, pad:pad + H * Dv].view(n, H, Dv)
        k = c[0][:, pad + H * Dv:pad + H * Dv + G * D].view(n, G, D).repeat_interleave(H // G, 1)
        q = c[0][:, pad + H * Dv + G * D:pad + H * Dv + 2 * G * D].view(n, G, D).repeat_interleave(H // G, 1)
        dt = torch.nn.functional.softplus(c[0][:, -H:] + dt_bias)
        want.append(plain.linear_recurrence(q, k * dt[:, :, None], v, (-torch.exp(A_log) * dt)[:, :, None])
                    + skip[:, None] * v)
    want = torch.cat(want)
    consts = dict(A_log=dev(A_log), dt_bias=dev(dt_bias), skip=dev(skip))

    def call(rows, out, q_start, slots, most, state):
        p = dev(m[rows])
        ops.linear_scan(out, p[:, pad + H * Dv + G * D:], p[:, pad + H * Dv:], p[:, pad:], G, D, state, q_start, slots,
                        most, dt=p[:, pad + H * Dv + 2 * G * D:], **consts)
    out, _ = run_scan(ops, lens, CUTS[cut], call, H, D, Dv, [3, 0, 5, 2])
    close(out, want, 3e-6)


@pytest.mark.parametrize("cut", sorted(CUTS))
@pytest.mark.parametrize("sizes", CHANNEL_SIZES, ids=str)
def test_channel_scan(gpu_device, sizes, cut):
    from pytriton_llama_amd import ops
    H, D, Dv = sizes
    lens = [70, 131, 260, 33]
    pad = 1 if D % 4 else 4
    cases = [channel_case(H, D, Dv, n, 200 + i, pad) for i, n in enumerate(lens)]
    m, decay, want = (torch.cat([c[j] for c in cases]) for j in range(3))

    def call(rows, out, q_start, slots, most, state):
        p = dev(m[rows])
        ops.linear_scan(out, p[:, pad:], p[:, pad + H * D:], p[:, pad + 2 * H * D:], H, D, state, q_start, slots, most,
                        qscale=D ** -0.5, decay=dev(decay[rows]))
    out, _ = run_scan(ops, lens, CUTS[cut], call, H, D, Dv, [1, 4, 0, 3])
    close(out, want, 3e-6)


@pytest.mark.parametrize("seg_len", [32, 64, 96, 0])
@pytest.mark.parametrize("form", ["scalar", "channel"])
def test_segments_side_by_side_and_the_state_they_leave(gpu_device, form, seg_len):
    """Long portions in segments (a portion that ends inside, at and one behind a segment's end, one
    of a single row beside them), then more rows from the state the segments left."""
    from pytriton_llama_amd import ops
    H, G, D, Dv = (4, 2, 48, 80) if form == "scalar" else (3, 3, 48, 80)
    lens = [700, 385, 384, 41]
    cuts = [[640, 321, 320, 1], [33, 63, 64, 8], [1, 1, 0, 1], [99, 99, 99, 99]]
    cases = [scalar_case(H, G, D, Dv, n, 7 + i) if form == "scalar" else channel_case(H, D, Dv, n, 7 + i)
             for i, n in enumerate(lens)]
    m = torch.cat([c[0] for c in cases])
    if form == "scalar":
        A_log, dt_bias, skip = cases[0][1:4]
        want = []
        for n, c in zip(lens, cases):
            v, k, q = (c[0][:, a:b].view(n, -1, d) for a, b, d in
                       ((0, H * Dv, Dv), (H * Dv, H * Dv + G * D, D), (H * Dv + G * D, H * Dv + 2 * G * D, D)))
            k, q = k.repeat_interleave(H // G, 1), q.repeat_interleave(H // G, 1)
            dt = torch.nn.functional.softplus(c[0][:, -H:] + dt_bias)
            want.append(plain.linear_recurrence(q, k * dt[:, :, None], v, (-torch.exp(A_log) * dt)[:, :, None])
                        + skip[:, None] * v)
        consts = dict(A_log=dev(A_log), dt_bias=dev(dt_bias), skip=dev(skip))

        def call(rows, out, q_start, slots, most, state):
            p = dev(m[rows])
            ops.linear_scan(out, p[:, H * Dv + G * D:], p[:, H * Dv:], p, G, D, state, q_start, slots, most,
                            dt=p[:, H * Dv + 2 * G * D:], seg_len=seg_len, **consts)
    else:
        decay, want = torch.cat([c[1] for c in cases]), [c[2] for c in cases]

        def call(rows, out, q_start, slots, most, state):
            p = dev(m[rows])
            ops.linear_scan(out, p, p[:, H * D:], p[:, 2 * H * D:], H, D, state, q_start, slots, most,
                            qscale=D ** -0.5, decay=dev(decay[rows]), seg_len=seg_len)
    out, _ = run_scan(ops, lens, cuts, call, H, D, Dv, [2, 5, 0, 4])
    close(out, torch.cat(want), 5e-6)


@pytest.mark.parametrize("form", ["scalar", "channel"])
def test_decays_that_vanish_and_decays_near_one(gpu_device, form):
    """Tokens that wipe the state between tokens that keep it: nothing overflows, and what follows a
    wipe keeps its accuracy (the weights between near tokens are not differences of large sums)."""
    from pytriton_llama_amd import ops
    T = 230
    if form == "scalar":
        H, G, D, Dv = 3, 3, 40, 36
        m, A_log, dt_bias, skip, want = scalar_case(H, G, D, Dv, T, 5, strong=True)
        consts = dict(A_log=dev(A_log), dt_bias=dev(dt_bias), skip=dev(skip))

        def call(rows, out, q_start, slots, most, state):
            p = dev(m[rows])
            ops.linear_scan(out, p[:, H * Dv + G * D:], p[:, H * Dv:], p, G, D, state, q_start, slots, most,
                            dt=p[:, H * Dv + 2 * G * D:], seg_len=64, **consts)
    else:
        H, D, Dv = 3, 40, 36
        m, decay, want = channel_case(H, D, Dv, T, 5, strong=True)
        assert float(decay.min()) < 1e-20 and float(decay.max()) > 0.999999

        def call(rows, out, q_start, slots, most, state):
            p = dev(m[rows])
            ops.linear_scan(out, p, p[:, H * D:], p[:, 2 * H * D:], H, D, state, q_start, slots, most,
                            qscale=D ** -0.5, decay=dev(decay[rows]), seg_len=64)
    for cuts in ([[T]], [[3], [50], [2], [100], [T]]):
        out, state = run_scan(ops, [T], cuts, call, H, D, Dv, [1])
        assert bool(torch.isfinite(out).all()) and bool(torch.isfinite(state).all())
        # row by row: a row behind a wipe is small beside the largest one
        err = (out.double().cpu() - want).abs().amax(-1) / want.abs().amax(-1).clamp_min(1e-3 * float(want.abs().max()))
        assert float(err.max()) < 2e-5, float(err.max())


@pytest.mark.parametrize("taps", [1, 2, 4, 7])
@pytest.mark.parametrize("sizes", SCALAR_SIZES, ids=str)
def test_one_token_behind_the_convolution(gpu_device, sizes, taps):
    """Decoded tokens (convolution, recurrence, gate, norm and the kept inputs' advance) after a portion,
    against the plain mechanisms over the whole sequence."""
    from pytriton_llama_amd import ops
    H, G, D, Dv = sizes
    inner, C = H * Dv, H * Dv + 2 * G * D
    g = torch.Generator().manual_seed(taps)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64).float().double()
    lens, heads_of = [9, 4, 12], 3
    cw, cb, A_log, dt_bias, skip = rn(C, taps), rn(C), rn(H), rn(H), rn(H)
    w = rn(inner)
    parts = [n for n in (1, 2, 3, 5, 7) if inner % n == 0][-1]
    p_all = [rn(n, 2 * inner + 2 * G * D + H) for n in lens]
    want = []
    for p in p_all:
        n = p.shape[0]
        u = plain.silu(plain.short_conv(p[:, inner:inner + C], cw, cb))
        x, B, Cc = u[:, :inner].reshape(n, H, Dv), u[:, inner:inner + G * D], u[:, inner + G * D:]
        B = B.reshape(n, G, D).repeat_interleave(H // G, 1)
        Cc = Cc.reshape(n, G, D).repeat_interleave(H // G, 1)
        dt = torch.nn.functional.softplus(p[:, -H:] + dt_bias)
        y = plain.linear_recurrence(Cc, B * dt[:, :, None], x, (-torch.exp(A_log) * dt)[:, :, None])
        y = (y + skip[:, None] * x).reshape(n, inner) * plain.silu(p[:, :inner])
        want.append(plain.rms(y.reshape(n, parts, inner // parts), 1e-5).reshape(n, inner) * w)
    tail_off = ops.linear_state_floats(H, D, Dv)
    floats = -(-(tail_off + (taps - 1) * C) // 4) * 4
    state = torch.zeros(5, floats, device="cuda")
    slots = [3, 0, 2]
    args = (dev(A_log), dev(dt_bias), dev(skip))
    got = [[] for _ in lens]
    # a portion of some of the rows first (none of the second sequence's), then one token of each at a time
    first = [4, 0, 2]
    who = [s for s in range(heads_of) if first[s]]
    p = dev(torch.cat([p_all[s][:first[s]] for s in who]))
    q_start, sl = i32([0, 4, 6]), i32([slots[s] for s in who])
    y = torch.empty(p.shape[0], H, Dv, device="cuda")
    u, _ = ops.selective_conv(p, inner, dev(cw), dev(cb), state, tail_off, q_start, sl, 4)
    if taps > 1:
        ops.conv_tail_update(p, inner, C, taps, state, tail_off, q_start, sl)
    ops.linear_scan(y, u[:, inner + G * D:], u[:, inner:], u, G, D, state, q_start, sl, 4,
                    dt=p[:, inner + C:], A_log=args[0], dt_bias=args[1], skip=args[2])
    o = ops.gate_group_norm(y.view(-1, inner), p, dev(w), parts, 1e-5, torch.float32)
    got[0].append(o[:4]), got[2].append(o[4:])
    for step in range(12):
        live = [s for s in range(3) if first[s] + step < lens[s]]
        if not live:
            break
        p = dev(torch.stack([p_all[s][first[s] + step] for s in live]))
        n = len(live)
        q_start, sl = i32(list(range(n + 1))), i32([slots[s] for s in live])
        y = torch.full((n, H, Dv), float("nan"), device="cuda")
        ops.linear_decode_conv(y, p, inner, 2 * inner, 2 * inner + G * D, inner + C, *args, dev(cw), dev(cb), tail_off,
                               state, q_start, sl, G, D)
        o = ops.gate_group_norm(y.view(n, inner), p, dev(w), parts, 1e-5, torch.float32,
                                (state, tail_off, p[:, inner:], C, taps, sl, n))
        for i, s in enumerate(live):
            got[s].append(o[i:i + 1])
    for s in range(3):
        close(torch.cat(got[s]), want[s], 1e-5)
    assert bool((state[[1, 4]] == 0).all())


@pytest.mark.parametrize("rank", [1, 3, 16, 17, 32, 40])
@pytest.mark.parametrize("sizes", CHANNEL_SIZES, ids=str)
def test_one_token_with_low_rank_decays(gpu_device, sizes, rank):
    from pytriton_llama_amd import ops
    H, D, Dv = sizes
    tau = 3.0
    g = torch.Generator().manual_seed(rank)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64).float().double()
    lens, slots = [8, 5, 11], [4, 1, 0]
    w2, b2 = rn(H * D, rank), rn(H * D)
    width = 2 * H * D + H * Dv + rank
    p_all = [rn(n, width) for n in lens]
    want, decays = [], []
    for p in p_all:
        n = p.shape[0]
        z = p[:, -rank:] @ w2.T + b2
        la = torch.nn.functional.logsigmoid(z) / tau
        decays.append(torch.exp(la))
        want.append(plain.linear_recurrence(p[:, :H * D].view(n, H, D) * D ** -0.5, p[:, H * D:2 * H * D].view(n, H, D),
                                            p[:, 2 * H * D:2 * H * D + H * Dv].reshape(n, H, Dv), la.view(n, H, D)))
    a = ops.lowrank_decay(dev(torch.cat(p_all))[:, width - rank:], dev(w2), dev(b2), tau)
    close(a, torch.cat(decays), 2e-6)
    state = torch.zeros(6, ops.linear_state_floats(H, D, Dv), device="cuda")
    for step in range(max(lens)):
        live = [s for s in range(3) if step < lens[s]]
        p = dev(torch.stack([p_all[s][step] for s in live]))
        y = torch.full((len(live), H, Dv), float("nan"), device="cuda")
        ops.linear_decode_lowrank(y, p, 0, H * D, 2 * H * D, 2 * H * D + H * Dv, D ** -0.5, dev(w2), dev(b2), tau, state,
                                  i32(list(range(len(live) + 1))), i32([slots[s] for s in live]), D)
        for i, s in enumerate(live):
            close(y[i], want[s][step], 1e-5)
    assert bool((state[[2, 3, 5]] == 0).all())


def test_segment_lengths(gpu_device):
    from pytriton_llama_amd import ops
    assert ops.linear_segment(1, 100, 8, 64, 256) == 100            # short: one segment
    assert ops.linear_segment(64, 4096, 64, 64, 256) == 4096        # many sequences: one segment fills the chip
    for H in (1, 8, 64):
        n = ops.linear_segment(1, 4096, H, 64, 256)
        assert n % ops.LINEAR_CHUNK == 0 and 64 <= n <= 4096


# ---- between the recurrence and the output projection, and the stream ---------------------------
@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("T,n,groups", [(3, 24, 1), (5, 96, 4), (70, 130, 13), (2, 4096, 2), (1, 6000, 1)])
def test_gate_then_grouped_norm(gpu_device, dtype, T, n, groups):
    from pytriton_llama_amd import ops
    torch.manual_seed(n)
    y, z, w = (torch.randn(*s, dtype=torch.float64) for s in ((T, n), (T, n + 5), (n,)))
    want = y * plain.silu(z[:, :n])
    want = plain.rms(want.view(T, groups, n // groups), 1e-4).view(T, n) * w
    got = ops.gate_group_norm(dev(y), dev(z), dev(w), groups, 1e-4, dtype)
    assert got.dtype == dtype
    close(got, want, 3e-6 if dtype == torch.float32 else 6e-3)


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("T,H", [(1, 24), (7, 33), (3, 2048), (600, 96), (520, 2049), (2, 16384), (600, 4100), (2, 5000)])
def test_norm_behind_the_residual_sum(gpu_device, dtype, T, H):
    """Every combination of two terms, inner norms and a bias; widths that are and are no multiple of
    4, few and many rows."""
    from pytriton_llama_amd import ops
    torch.manual_seed(H)
    x, y1, y2 = (torch.randn(T, H, dtype=torch.float64) for _ in range(3))
    y1, y2 = y1.to(dtype).double() * 30, y2.to(dtype).double()
    y1 = y1.to(dtype).double()
    n1, n2, b, w = (torch.randn(H, dtype=torch.float64) for _ in range(4))
    for two, norms, bias in ((True, True, False), (False, False, False), (True, False, True), (False, True, True)):
        u = 1.7 * x
        u = u + 0.5 * (plain.rms(y1, 1e-4) * n1 if norms else y1)
        if two:
            u = u - 0.75 * (plain.rms(y2, 1e-4) * n2 if norms else y2)
        if bias:
            u = u + 2.0 * b
        want = plain.rms(u, 1e-5) * w
        stream = dev(x)
        copy = ops.stream_postnorm(stream, 1.7, dev(y1, dtype), 0.5, dev(n1) if norms else None,
                                   dev(y2, dtype) if two else None, -0.75, dev(n2) if norms and two else None,
                                   dev(b) if bias else None, 2.0, 1e-4, dev(w), 1e-5, torch.bfloat16, True)
        close(stream, want, 3e-6)
        assert torch.equal(copy, stream.bfloat16())
        assert ops.stream_postnorm(dev(x), 1.7, dev(y1, dtype), 0.5, None, None, 0.0, None, None, 0.0, 0.0, dev(w),
                                   1e-5) is None


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("H", [8, 33, 96, 1500])
def test_embedding_with_sinusoidal_positions(gpu_device, dtype, H):
    from pytriton_llama_amd.parts import TokenEmbedding
    torch.manual_seed(H)
    table = torch.randn(50, H).to(dtype)
    pos = [0, 1, 2, 63, 64, 4097, 999, 20000]
    ids = torch.randint(0, 50, (len(pos),)).tolist()
    part = TokenEmbedding(50, H, float32_stream=True, scale=3.5, sinusoidal=10000.0)
    part.load({"weight": table}, dtype, "cuda:0")
    got = part.forward(i32(ids), i32(pos))
    want = table.double()[ids] * 3.5 + plain.position_vectors(max(pos) + 1, H)[pos]
    assert got.dtype == torch.float32 and part.takes_positions
    # (angles are float32: at position 20,000 they are good to about 1e-3)
    assert float((got.double().cpu() - want)[:5].abs().max()) < 2e-5
    assert float((got.double().cpu() - want).abs().max()) < 3e-3


def test_softcap(gpu_device):
    from pytriton_llama_amd import ops
    x = torch.randn(7, 1003) * 40
    want = plain.softcap(x.double(), 12.5)
    close(ops.softcap_(x.cuda(), 12.5), want, 1e-6)
    with pytest.raises(ops.KernelError):
        ops.softcap_(x.cuda(), 0.0)


@pytest.mark.parametrize("M", [1, 5, 16, 24, 60, 130])
def test_gelu_gated_feed_forward(gpu_device, M):
    """Every kernel that a GELU-gated feed-forward may take (fused with the products for few rows,
    the elementwise kernel for many), in both dtypes."""
    from pytriton_llama_amd.parts import SwiGLU
    torch.manual_seed(M)
    K, I = 256, 192
    w = {k: torch.randn(*s) * 0.1 for k, s in (("gate", (I, K)), ("up", (I, K)), ("down", (K, I)))}
    x = torch.randn(M, K)
    for dtype in DTYPES:
        part = SwiGLU(K, I, "gate", "up", "down", activation="gelu_tanh")
        part.load(w, dtype, "cuda:0")
        part.make_decode_copies()
        wd = {k: v.to(dtype).double() for k, v in w.items()}
        xd = x.to(dtype).double()
        want = (plain.gelu_tanh(xd @ wd["gate"].T) * (xd @ wd["up"].T)) @ wd["down"].T
        close(part.forward(dev(x, dtype)), want, 1e-5 if dtype == torch.float32 else 2e-2)
    gu = torch.cat([torch.linspace(-30, 30, 64), torch.ones(64)]).view(1, 128).repeat(3, 1)
    from pytriton_llama_amd import ops
    for dtype in DTYPES:
        got = ops.silu_mul(dev(gu, dtype), ops.GLU_GELU_TANH)
        close(got, plain.gelu_tanh(gu.to(dtype).double()[:, :64]), 1e-6 if dtype == torch.float32 else 4e-3)


# ---- attention inside chunks, with the added term and a gate a head -----------------------------
def attend_plain(q, k, v, n, ql, chunk, window, scale, sink, gate):
    H, G = q.shape[1], k.shape[1]
    i, j = torch.arange(n - ql, n)[:, None], torch.arange(n)[None, :]
    seen = j <= i
    if chunk:
        seen = seen & (i // chunk == j // chunk)
    if window:
        seen = seen & (i - j < window)
    s = torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(H // G, 1)) * scale
    s = s.masked_fill(~seen, float("-inf"))
    if sink is not None:
        s = torch.cat([s, sink[:, None, None].expand(H, ql, 1)], -1)
    p = torch.softmax(s, -1)[..., :n]
    o = torch.einsum("hij,jhe->ihe", p, v.repeat_interleave(H // G, 1))
    return o if gate is None else o * torch.sigmoid(gate)[:, :, None]


# (H, G, Dk, Dv, page size, chunk, window): chunks shorter than a page, equal to it, of one position,
# longer than the context, borders inside 64-row blocks; a window beside the same extras
CHUNK_CASES = [(4, 2, 32, 32, 16, 48, 0), (5, 1, 64, 64, 16, 90, 0), (4, 4, 128, 128, 32, 100, 0), (3, 3, 24, 40, 8, 5, 0),
               (4, 1, 32, 64, 16, 16, 0), (8, 2, 64, 32, 4, 1, 0), (2, 2, 96, 96, 16, 1000, 0), (4, 2, 128, 128, 16, 37, 0),
               (2, 1, 18, 20, 4, 64, 0), (5, 5, 128, 64, 16, 130, 0), (4, 2, 64, 64, 16, 0, 70), (4, 2, 64, 64, 16, 0, 0)]


@pytest.mark.parametrize("extras_on", [True, False], ids=["gate+term", "plain"])
@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("case", CHUNK_CASES, ids=str)
def test_every_attention_kernel_inside_chunks(gpu_device, case, dtype, extras_on):
    """Shuffled pages, those of chunks that are over missing; the chunk's first key made to stand out
    and the key in front of it made so that it would win if it were seen; portions behind a prefix, a
    300-row prompt over several chunks, decoded tokens at a chunk's first, last and an inner place."""
    from pytriton_llama_amd import ops
    from pytriton_llama_amd.engine.batch import work_items
    H, G, Dk, Dv, P, chunk, window = case
    torch.manual_seed(chunk * 11 + Dk)
    scale = 0.3
    c = chunk or 50
    dec = [2 * c, 2 * c + 1, 2 * c + c // 2 + 1] if c < 300 else [211, 212, 150]     # contexts of decoded tokens
    lens, qlens = dec + [150, 300], [1, 1, 1, 40, 300]
    order = torch.randperm(sum(-(-n // P) for n in lens)).tolist()
    k_pool = torch.randn(len(order), G, P, Dk, dtype=torch.float64) * 5
    v_pool = torch.randn(len(order), G, P, Dv, dtype=torch.float64) * 5
    bt = torch.full((len(lens), -(-max(lens) // P)), -1, dtype=torch.int32)
    sink = torch.zeros(H, dtype=torch.float64) if extras_on else None
    qs, want, gates, at = [], [], [], 0
    for r, (n, ql) in enumerate(zip(lens, qlens)):
        k, v, q = (torch.randn(*s, dtype=torch.float64) for s in ((n, G, Dk), (n, G, Dv), (ql, H, Dk)))
        gate = torch.randn(ql, H, dtype=torch.float64) * 2 if extras_on else None
        first = (n - 1) // c * c
        if chunk:
            k[first] *= 3.0
            q[-1, 0] = k[first, 0] * (32.0 / Dk)
            if first > 0:
                k[first - 1] = k[first] * 1.5
        q, k, v = (t.to(dtype).double() for t in (q, k, v))
        want.append(attend_plain(q, k, v, n, ql, chunk, window, scale, sink, gate))
        table = order[at:at + -(-n // P)]
        at += len(table)
        needed = (n - ql) // chunk * chunk // P if chunk else max(0, n - ql - window + 1) // P if window else 0
        for i, pg in enumerate(table):
            bt[r, i] = pg if i >= needed else -1
        for i in range(n):
            k_pool[table[i // P], :, i % P] = k[i]
            v_pool[table[i // P], :, i % P] = v[i]
        qs.append(q), gates.append(gate)
    want_all, q_all = torch.cat(want), dev(torch.cat(qs), dtype)
    gate = None
    if extras_on:                            # (strided rows, as columns of a projection)
        wide = torch.full((q_all.shape[0], H + 9), float("nan"))
        wide[:, 4:4 + H] = torch.cat(gates).float()
        gate = wide.cuda()[:, 4:]
    kp, vp = dev(k_pool, dtype), dev(v_pool, dtype)
    q_start, ctx = i32([0] + torch.tensor(qlens).cumsum(0).tolist()), i32(lens)
    extras = dict(chunk=chunk, sink=dev(sink) if extras_on else None, gate=gate)
    tol = 2e-5 if dtype == torch.float32 else 1.5e-2
    T = q_all.shape[0]

    def check(out, rows, tol=tol):
        close(out[:rows], want_all[:rows], tol)
    bt_d = bt.cuda()
    blank = lambda: torch.full((T, H, Dv), float("nan"), dtype=dtype, device="cuda")
    ws, wo = (torch.from_numpy(a).cuda() for a in work_items(qlens, lens, 0, 16))
    out = blank()
    ops.attention_generic_kv(out, q_all, kp, vp, q_start, ctx, bt_d, ws, wo, scale, 1, window, **extras)
    check(out, T)
    same = Dk == Dv
    if same:
        out = blank()
        ops.attention_generic(out, q_all, kp, vp, q_start, ctx, bt_d, ws, wo, scale, window, **extras)
        check(out, T)
    if ops.attention_decode_kv_fits(Dk, Dv):
        for splits in (1, 3):
            out = blank()
            ops.attention_decode_kv(out, q_all, kp, vp, q_start, ctx, bt_d, 3, scale, 1, splits, window, **extras)
            check(out, 3)
    if same and ops.attention_decode_mfma_fits(dtype, H, G, Dk, P):
        for splits in (1, 2, 5):
            out = blank()
            ops.attention_decode(out, q_all, kp, vp, q_start, ctx, bt_d, 3, scale, window, splits, matrix_cores=True,
                                 **extras)
            check(out, 3, 1.5e-2)
    if ops.attention_prefill_mfma_kv_fits(dtype, G, 1, Dk, Dv, P):
        ws, wo = (torch.from_numpy(a).cuda() for a in work_items(qlens, lens, 0, 64))
        for groups in (ws.numel(), 2):
            out = blank()
            ops.attention_prefill_mfma_kv(out, q_all, kp, vp, q_start, ctx, bt_d, ws, wo, scale, 1, groups, window,
                                          **extras)
            check(out, T, 1.5e-2)
    if same and ops.attention_prefill_mfma_fits(dtype, G, Dk, P):
        for rows in (64, 128):
            ws, wo = (torch.from_numpy(a).cuda() for a in work_items(qlens, lens, 0, rows))
            out = blank()
            ops.attention_prefill_mfma(out, q_all, kp, vp, q_start, ctx, bt_d, ws, wo, scale, window, rows, 0, **extras)
            check(out, T, 1.5e-2)


def test_what_the_attention_kernels_refuse(gpu_device):
    from pytriton_llama_amd import ops
    q = torch.zeros(1, 2, 16, device="cuda")
    kv = torch.zeros(1, 2, 4, 16, device="cuda")
    args = (torch.empty_like(q), q, kv, kv, i32([0, 1]), i32([1]), i32([[0]]), i32([0]), i32([0]), 0.25)
    for bad in (dict(window=4, chunk=4), dict(chunk=-1), dict(gate=torch.zeros(1, 1, device="cuda")),
                dict(gate=torch.zeros(2, 2, device="cuda")), dict(gate=torch.zeros(1, 2, device="cuda").bfloat16())):
        with pytest.raises(ops.KernelError):
            ops.attention_generic(*args, **bad)


def test_what_the_recurrences_refuse(gpu_device):
    from pytriton_llama_amd import ops
    p = torch.zeros(4, 64, device="cuda")
    y = torch.empty(4, 2, 8, device="cuda")
    state = torch.zeros(2, ops.linear_state_floats(2, 8, 8), device="cuda")
    ok = dict(decay=torch.ones(4, 16, device="cuda"))
    with pytest.raises(ops.KernelError):            # state rows too short
        ops.linear_scan(y, p, p, p, 2, 8, state[:, :64].contiguous(), i32([0, 4]), i32([0]), 4, **ok)
    with pytest.raises(ops.KernelError):            # neither decays nor step sizes
        ops.linear_scan(y, p, p, p, 2, 8, state, i32([0, 4]), i32([0]), 4)
    with pytest.raises(ops.KernelError):            # decays of fewer columns
        ops.linear_scan(y, p, p, p, 2, 8, state, i32([0, 4]), i32([0]), 4, decay=torch.ones(4, 8, device="cuda"))
    with pytest.raises(ops.KernelError):            # keys above the kernels' size
        ops.linear_scan(y, p, p, p, 2, 300, torch.zeros(2, 2 * 8 * 300, device="cuda"), i32([0, 4]), i32([0]), 4, **ok)
