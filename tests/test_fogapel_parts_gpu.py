"""Each kernel that Fogapel added or widened, alone, against tests/plain_fogapel.py or a few lines of
float64."""
import pytest
import torch

import plain_fogapel as plain

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


def rounds(lens, cuts):
    """Sequences of ``lens`` rows advanced together: round i brings cuts[i][s] rows of sequence s (no
    more than are left). Yields [(sequence, first row, rows)], single rows first."""
    done = [0] * len(lens)
    for cut in cuts:
        live = [(s, done[s], min(n, lens[s] - done[s])) for s, n in enumerate(cut) if min(n, lens[s] - done[s]) > 0]
        if live:
            yield sorted(live, key=lambda x: x[2] != 1)
        for s, _, n in live:
            done[s] += n
    assert done == list(lens)


CUTS = {
    "whole": [[10 ** 6] * 4],
    "portions": [[2, 31, 64, 5], [33, 3, 2, 1], [1, 1, 100, 32], [17, 40, 2, 2], [200, 200, 200, 200]],
    "ones": [[5, 1, 30, 16]] + [[1, 1, 1, 1]] * 40 + [[300] * 4],
}


# ---- the recurrence with a bonus ---------------------------------------------------------------
# (heads, D, Dv)
SIZES = [(2, 16, 16), (3, 20, 28), (1, 13, 9), (2, 64, 64), (2, 128, 130), (1, 200, 40), (1, 256, 16)]


def bonus_case(H, D, Dv, T, seed, pad=0, strong=False, u=None):
    g = torch.Generator().manual_seed(seed)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    m = rn(T, pad + 2 * H * D + H * Dv).float().double()
    z = rn(T, H * D) * (3.0 if strong else 1.0) + (1.0 if strong else -2.0)
    decay = torch.exp(-torch.exp(z)).float().double()
    u = rn(H, D).float().double() if u is None else u
    r = m[:, pad:pad + H * D].view(T, H, D)
    k = m[:, pad + H * D:pad + 2 * H * D].view(T, H, D)
    v = m[:, pad + 2 * H * D:].reshape(T, H, Dv)
    log_decay = torch.log(decay.clamp_min(1e-300)).view(T, H, D)
    return m, decay, u, plain.wkv_recurrence(r, k, v, log_decay, u)


def run_bonus(ops, cases, lens, cuts, H, D, Dv, pad, slots, seg_len=0, W=11, x_dtype=torch.float32):
    """All rows through the scan on slots whose rest is marked; the last rows of a matrix x are kept."""
    off = ops.linear_state_floats(H, D, Dv)
    state = torch.full((7, -(-(off + W) // 4) * 4), 7.5, dtype=torch.float32, device="cuda")
    for s in slots:
        state[s] = 0
    u = dev(cases[0][2])
    xs = [torch.randn(n, W).to(x_dtype) for n in lens]
    out = [torch.full((n, H, Dv), float("nan")) for n in lens]
    for live in rounds(lens, cuts):
        p = dev(torch.cat([cases[s][0][a:a + n] for s, a, n in live]))
        decay = dev(torch.cat([cases[s][1][a:a + n] for s, a, n in live]))
        x = torch.cat([xs[s][a:a + n] for s, a, n in live]).cuda()
        q_start = [0]
        for _, _, n in live:
            q_start.append(q_start[-1] + n)
        y = torch.full((q_start[-1], H, Dv), float("nan"), device="cuda")
        ops.linear_scan(y, p[:, pad:], p[:, pad + H * D:], p[:, pad + 2 * H * D:], H, D, state, i32(q_start),
                        i32([slots[s] for s, _, _ in live]), max(n for _, _, n in live), decay=decay, bonus=u,
                        keep=(x, off), seg_len=seg_len)
        for (s, a, n), at in zip(live, q_start):
            out[s][a:a + n] = y[at:at + n].cpu()
            assert torch.equal(state[slots[s], off:off + W].cpu(), xs[s][a + n - 1].float())
    untouched = [s for s in range(7) if s not in slots]
    assert bool((state[untouched] == 7.5).all())
    return out, state


@pytest.mark.parametrize("cut", sorted(CUTS))
@pytest.mark.parametrize("sizes", SIZES, ids=str)
def test_scan_with_a_bonus(gpu_device, sizes, cut):
    from pytriton_llama_amd import ops
    H, D, Dv = sizes
    lens = [70, 131, 260, 33]
    pad = 1 if D % 4 else 4
    first = bonus_case(H, D, Dv, lens[0], 200, pad)
    cases = [first] + [bonus_case(H, D, Dv, n, 201 + i, pad, u=first[2]) for i, n in enumerate(lens[1:])]
    out, _ = run_bonus(ops, cases, lens, CUTS[cut], H, D, Dv, pad, [1, 4, 0, 3])
    for o, c in zip(out, cases):
        close(o, c[3], 3e-6)


@pytest.mark.parametrize("seg_len", [32, 64, 96, 0])
def test_segments_side_by_side_and_the_state_they_leave(gpu_device, seg_len):
    """Long portions in segments (a portion that ends inside, at and one behind a segment's end, one
    of a single row beside them), then more rows from the state the segments left."""
    from pytriton_llama_amd import ops
    H, D, Dv = 3, 48, 80
    lens = [700, 385, 384, 41]
    cuts = [[640, 321, 320, 1], [33, 63, 64, 8], [1, 1, 0, 1], [99, 99, 99, 99]]
    first = bonus_case(H, D, Dv, lens[0], 7)
    cases = [first] + [bonus_case(H, D, Dv, n, 8 + i, u=first[2]) for i, n in enumerate(lens[1:])]
    out, _ = run_bonus(ops, cases, lens, cuts, H, D, Dv, 0, [2, 5, 0, 4], seg_len, W=513, x_dtype=torch.bfloat16)
    for o, c in zip(out, cases):
        close(o, c[3], 5e-6)


def test_decays_that_vanish_and_decays_near_one(gpu_device):
    """Tokens that wipe channels of the state between tokens that keep them: nothing overflows, and what
    follows a wipe keeps its accuracy."""
    from pytriton_llama_amd import ops
    T, H, D, Dv = 230, 3, 40, 36
    case = bonus_case(H, D, Dv, T, 5, strong=True)
    assert float(case[1].min()) == 0.0 and float(case[1].max()) > 0.999
    for cuts in ([[T]], [[3], [50], [2], [100], [T]]):
        out, state = run_bonus(ops, [case], [T], cuts, H, D, Dv, 0, [1], 64)
        assert bool(torch.isfinite(out[0]).all()) and bool(torch.isfinite(state).all())
        err = (out[0].double() - case[3]).abs().amax(-1) / case[3].abs().amax(-1).clamp_min(1e-3 * float(case[3].abs().max()))
        assert float(err.max()) < 2e-5, float(err.max())


@pytest.mark.parametrize("rank", [1, 3, 16, 17, 64, 100])
@pytest.mark.parametrize("sizes", SIZES, ids=str)
def test_one_token_with_low_rank_decays_and_a_bonus(gpu_device, sizes, rank):
    from pytriton_llama_amd import ops
    H, D, Dv = sizes
    g = torch.Generator().manual_seed(rank)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64).float().double()
    lens, slots = [8, 5, 11], [4, 1, 0]
    w2, w0, u = rn(H * D, rank) * rank ** -0.5, rn(H * D) - 2.0, rn(H, D)
    width, W = 2 * H * D + H * Dv + rank, 37
    p_all, x_all = [rn(n, width) for n in lens], [rn(n, W) for n in lens]
    want, decays = [], []
    for p in p_all:
        n = p.shape[0]
        z = torch.tanh(p[:, -rank:]) @ w2.T + w0
        decays.append(torch.exp(-torch.exp(z)))
        want.append(plain.wkv_recurrence(p[:, :H * D].view(n, H, D), p[:, H * D:2 * H * D].view(n, H, D),
                                         p[:, 2 * H * D:2 * H * D + H * Dv].reshape(n, H, Dv), -torch.exp(z).view(n, H, D), u))
    a = ops.lowrank_decay(dev(torch.cat(p_all))[:, width - rank:], dev(w2), dev(w0), form=ops.DECAY_EXP)
    close(a, torch.cat(decays), 2e-6)
    off = ops.linear_state_floats(H, D, Dv)
    state = torch.zeros(6, -(-(off + W) // 4) * 4, device="cuda")
    for step in range(max(lens)):
        live = [s for s in range(3) if step < lens[s]]
        p = dev(torch.stack([p_all[s][step] for s in live]))
        x = dev(torch.stack([x_all[s][step] for s in live]))
        y = torch.full((len(live), H, Dv), float("nan"), device="cuda")
        ops.linear_decode_bonus(y, p, 0, H * D, 2 * H * D, 2 * H * D + H * Dv, dev(w2), dev(w0), dev(u), state,
                                i32(list(range(len(live) + 1))), i32([slots[s] for s in live]), D, keep=(x, off))
        for i, s in enumerate(live):
            close(y[i], want[s][step], 1e-5)
            assert torch.equal(state[slots[s], off:off + W].cpu().double(), x_all[s][step])
    assert bool((state[[2, 3, 5]] == 0).all())
    if Dv > ops.LINEAR_HEAD_FUSED:
        return
    # the heads finished by the same kernel: norm, weight, gate
    weight = rn(H * Dv)
    state.zero_()
    for step in range(max(lens)):
        live = [s for s in range(3) if step < lens[s]]
        gate = rn(len(live), H * Dv)
        p = dev(torch.cat([torch.stack([p_all[s][step] for s in live]), gate], dim=1))
        for dtype in DTYPES:
            keep = state.clone()
            y = torch.full((len(live), H * Dv), float("nan"), dtype=dtype, device="cuda")
            ops.linear_decode_bonus(torch.empty(len(live), H, Dv, device="cuda"), p, 0, H * D, 2 * H * D,
                                    2 * H * D + H * Dv, dev(w2), dev(w0), dev(u), keep,
                                    i32(list(range(len(live) + 1))), i32([slots[s] for s in live]), D,
                                    finish=(y, dev(weight), width, 1e-4))
            for i, s in enumerate(live):
                o = plain.rms(want[s][step], 1e-4).reshape(-1) * weight * plain.silu(gate[i])
                close(y[i], o, 2e-5 if dtype == torch.float32 else 6e-3)
        state = keep


@pytest.mark.parametrize("T,C,R", [(1, 5, 1), (70, 33, 7), (300, 130, 64), (65, 64, 16), (17, 200, 65), (3, 70, 200)])
@pytest.mark.parametrize("form", [0, 1])
def test_low_rank_decays_of_all_rows(gpu_device, T, C, R, form):
    from pytriton_llama_amd import ops
    g = torch.Generator().manual_seed(R)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64).float().double()
    r, w, b = rn(T, R + 3), rn(C, R) * R ** -0.5, rn(C)
    if form == ops.DECAY_EXP:
        want = torch.exp(-torch.exp(torch.tanh(r[:, 2:2 + R]) @ w.T + b))
    else:
        want = torch.sigmoid(r[:, 2:2 + R] @ w.T + b) ** (1 / 5.0)
    close(ops.lowrank_decay(dev(r)[:, 2:], dev(w), dev(b), 5.0, form), want, 2e-6)


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("W", [8, 33, 328, 2056])
def test_time_shift_in_portions(gpu_device, W, dtype):
    """Rows whose row before lies in the same portion, in the slot, or nowhere (a first token)."""
    from pytriton_llama_amd import ops
    g = torch.Generator().manual_seed(W)
    lens, slots = [9, 1, 14, 6], [3, 0, 2, 5]
    xs = [torch.randn(n, W, generator=g).to(dtype) for n in lens]
    mu = torch.rand(5, W, generator=g)
    want = [torch.stack([plain.time_mix(x.double(), mu[j].double()) for j in range(5)]) for x in xs]
    state = torch.full((6, W + 10), 3.25, device="cuda")
    state[slots, 7:7 + W] = 0
    for live in rounds(lens, [[2, 1, 1, 0], [1, 0, 3, 1], [3, 0, 1, 4], [1, 0, 1, 1], [9, 9, 9, 9]]):
        x = torch.cat([xs[s][a:a + n] for s, a, n in live]).cuda()
        q_start = [0]
        for _, _, n in live:
            q_start.append(q_start[-1] + n)
        got = ops.time_shift(x, mu.cuda(), state, 7, i32(q_start), i32([slots[s] for s, _, _ in live]))
        assert got.dtype == dtype
        for (s, a, n), at in zip(live, q_start):
            close(got[:, at:at + n], want[s][:, a:a + n], 1e-6 if dtype == torch.float32 else 6e-3)
            state[slots[s], 7:7 + W] = xs[s][a + n - 1].float().cuda()


# ---- several products side by side -------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("K,cols,last", [(64, 32, 16), (96, 48, 48), (50, 16, 32), (256, 96, 8), (512, 512, 64)])
def test_products_in_groups(gpu_device, K, cols, last, dtype):
    from pytriton_llama_amd import ops
    g = torch.Generator().manual_seed(K)
    S = 5
    w = torch.randn((S - 1) * cols + last, K, generator=g)
    wd = dev(w, dtype)
    blocked = ops.blocked_weight(wd) if dtype == torch.bfloat16 else None
    for M in (1, 7, 16, 17, 40, 64, 65, 300):
        x = torch.randn(S, M, K, generator=g)
        xd = dev(x, dtype)
        want = torch.cat([xd[s].double().cpu() @ wd[s * cols:(s + 1) * cols if s < S - 1 else None].double().cpu().T
                          for s in range(S)], dim=1)
        for b in (None, blocked) if blocked is not None else (None,):
            got = ops.gemm_groups(xd, wd, cols, b)
            assert got.dtype == torch.float32 and got.shape == want.shape
            close(got, want, 2e-6)
    with pytest.raises(ops.KernelError):
        ops.gemm_groups(xd, wd, cols + 8)
    with pytest.raises(ops.KernelError):
        ops.gemm_groups(xd, wd[:4 * cols].contiguous(), cols)


# ---- queries, keys and values behind a convolution -----------------------------------------------
# (Hq, Hk, Dk, Dv, rot_dims, taps)
CONV_CASES = [(4, 2, 24, 16, 16, 4), (3, 3, 18, 22, 6, 1), (2, 1, 12, 20, 0, 7), (4, 4, 40, 8, 2, 4), (2, 1, 128, 64, 128, 4),
              (2, 2, 13, 9, 12, 3), (1, 1, 200, 136, 64, 4), (2, 1, 640, 640, 100, 2), (8, 2, 16, 16, 16, 0)]


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("layout", [0, 1], ids=["pairs", "half"])
@pytest.mark.parametrize("case", CONV_CASES, ids=str)
def test_convolution_rotation_and_norm(gpu_device, case, layout, dtype):
    from pytriton_llama_amd import ops
    Hq, Hk, Dk, Dv, rot, taps = case
    P, base, eps = 4, 500.0, 1e-5
    g = torch.Generator().manual_seed(Dk + taps)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64).float().double()
    lens, slots = [70, 9, 33, 5], [2, 0, 3, 4]
    nq, nk, nv = Hq * Dk, Hk * Dk, Hk * Dv
    C, off = nq + nk + nv, (3, 3 + nq + 5, 3 + nq + 5 + nk)
    bias = rn(C)
    cw = rn(C, taps) if taps else None
    p_all = [rn(n, off[2] + nv + 2) for n in lens]

    def turn(x):
        if layout == ops.ROT_PAIRS:
            return plain.rotate_pairs(x, rot, base)
        order = [i // 2 + (i % 2) * (rot // 2) for i in range(rot)] + list(range(rot, Dk))
        y = plain.rotate_pairs(x[..., order], rot, base)
        back = torch.empty_like(y)
        back[..., order] = y
        return back
    want = []
    for p in p_all:
        u = torch.cat([p[:, o:o + n] for o, n in zip(off, (nq, nk, nv))], dim=1) + bias
        y = plain.short_conv(u, cw) if taps else u
        n = p.shape[0]
        want.append((plain.rms(turn(y[:, :nq].reshape(n, Hq, Dk)), eps), plain.rms(turn(y[:, nq:nq + nk].reshape(n, Hk, Dk)), eps),
                     y[:, nq + nk:].reshape(n, Hk, Dv)))
    pages = [-(-n // P) for n in lens]
    table = torch.randperm(sum(pages), generator=g).tolist()
    first = [sum(pages[:s]) for s in range(4)]
    k_pool = torch.zeros(sum(pages), Hk, P, Dk, dtype=dtype, device="cuda")
    v_pool = torch.zeros(sum(pages), Hk, P, Dv, dtype=dtype, device="cuda")
    tail_off = 6
    state = torch.full((6, tail_off + max(taps - 1, 0) * C + 3), -2.5, device="cuda")
    state[slots, tail_off:tail_off + max(taps - 1, 0) * C] = 0
    freq = (base ** (-torch.arange(0, rot, 2, dtype=torch.float64) / max(rot, 1))).float().cuda() if rot else None
    tol = 3e-5 if dtype == torch.float32 else 8e-3
    cuts = [[2, 1, 16, 1], [31, 1, 1, 1], [1, 3, 1, 2], [1, 1, 1, 1], [99, 99, 99, 99]]
    for live in rounds(lens, cuts):
        single = sum(n == 1 for _, _, n in live)
        p = dev(torch.cat([p_all[s][a:a + n] for s, a, n in live] + [torch.zeros(2, p_all[0].shape[1], dtype=torch.float64)]))
        q_start, pos, rows = [0], [], []
        for s, a, n in live:
            q_start.append(q_start[-1] + n)
            pos += list(range(a, a + n))
            rows += [table[first[s] + i // P] * P + i % P for i in range(a, a + n)]
        T = q_start[-1] + 2                  # two rows that belong to nobody
        q = torch.full((T, Hq, Dk), float("nan"), dtype=dtype, device="cuda")
        qs, sl = i32(q_start), i32([slots[s] for s, _, _ in live])
        ops.conv_qkv_prepare(q, p, *off, dev(bias), None if cw is None else dev(cw), state if taps > 1 else None, tail_off,
                             qs, sl, single, i32(pos + [0, 0]), i32(rows + [-1, -1]), rot, layout, freq, True, eps, k_pool,
                             v_pool, Hq, Hk, Hk, Dk, Dv, P)
        if taps > 1 and single < len(live):
            flat = torch.cat([p[:, o:o + n] for o, n in zip(off, (nq, nk, nv))], dim=1).contiguous()
            ops.conv_tail_update(flat, 0, C, taps, state, tail_off, qs[single:], sl[single:], dev(bias))
        for (s, a, n), at in zip(live, q_start):
            close(q[at:at + n], want[s][0][a:a + n], tol)
    for s, n in enumerate(lens):
        at = torch.tensor([table[first[s] + i // P] for i in range(n)]), torch.arange(n) % P
        close(k_pool.cpu()[at[0], :, at[1]], want[s][1], tol)
        close(v_pool.cpu()[at[0], :, at[1]], want[s][2], tol)
        if taps > 1:
            u = torch.cat([p_all[s][:, o:o + m] for o, m in zip(off, (nq, nk, nv))], dim=1) + bias
            kept = torch.cat([torch.zeros(taps - 1, C, dtype=u.dtype), u])[-(taps - 1):]
            close(state[slots[s], tail_off:tail_off + (taps - 1) * C].view(taps - 1, C), kept, 1e-6)
    assert bool((state[[1, 5]] == -2.5).all()) and bool((state[:, :tail_off] == -2.5).all())


def test_many_rows_take_the_convolution_in_runs(gpu_device):
    """Enough rows that a wave walks several of them: borders of runs inside and between sequences."""
    from pytriton_llama_amd import ops
    Hq, Hk, D, taps, eps = 16, 4, 32, 4, 1e-6
    g = torch.Generator().manual_seed(2)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64).float().double()
    lens = [1, 1, 3000, 2, 1501, 1003]
    C = (Hq + 2 * Hk) * D
    bias, cw, p = rn(C), rn(C, taps), rn(sum(lens), C)
    state = torch.randn(8, (taps - 1) * C, generator=g).cuda()
    q_start = [0] + torch.tensor(lens).cumsum(0).tolist()
    kept = [state[s].view(taps - 1, C).double().cpu() for s in range(len(lens))]
    y = []
    for s, n in enumerate(lens):
        u = torch.cat([kept[s], p[q_start[s]:q_start[s + 1]] + bias])
        y.append(sum(u[j:j + n] * cw[:, j] for j in range(taps)))
    y = torch.cat(y)
    T = len(y)
    q = torch.empty(T, Hq, D, device="cuda")
    kp, vp = torch.zeros(T, Hk, 1, D, device="cuda"), torch.zeros(T, Hk, 1, D, device="cuda")
    ops.conv_qkv_prepare(q, dev(p), 0, Hq * D, (Hq + Hk) * D, dev(bias), dev(cw), state, 0, i32(q_start), i32(range(len(lens))),
                         2, i32([0] * T), i32(range(T)), 0, 0, None, True, eps, kp, vp, Hq, Hk, Hk, D, D, 1)
    close(q, plain.rms(y[:, :Hq * D].view(T, Hq, D), eps), 1e-5)
    close(kp[:, :, 0], plain.rms(y[:, Hq * D:(Hq + Hk) * D].view(T, Hk, D), eps), 1e-5)
    close(vp[:, :, 0], y[:, (Hq + Hk) * D:].view(T, Hk, D), 1e-5)


# ---- the stream --------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("T,H", [(1, 24), (7, 33), (3, 2048), (600, 96), (520, 2049), (2, 16384), (600, 4100), (2, 5000)])
def test_scaled_sum_and_the_norm_that_follows(gpu_device, dtype, T, H):
    from pytriton_llama_amd import ops
    torch.manual_seed(H)
    x, y1, y2 = (torch.randn(T, H, dtype=torch.float64).float().double() for _ in range(3))
    y2 = y2.to(dtype).double()
    s1, s2, b, w = (torch.randn(H, dtype=torch.float64).float().double() for _ in range(4))
    for one, two, scaled, bias, norm in ((1, 1, 1, 1, 1), (1, 0, 1, 0, 1), (1, 1, 0, 0, 0), (0, 1, 1, 0, 1), (0, 0, 0, 0, 1),
                                         (1, 0, 0, 1, 1)):
        want = x.clone()
        if one:
            want += (s1 if scaled else 1.0) * (y1 + (b if bias else 0.0))
        if two:
            want += (s2 if scaled else 1.0) * y2
        stream = dev(x)
        out = ops.stream_scaled_sum(stream, dev(y1) if one else None, dev(s1) if scaled else None,
                                    dev(b) if bias else None, dev(y2, dtype) if two else None,
                                    dev(s2) if scaled else None, dev(w) if norm else None, 1e-5, dtype)
        close(stream, want, 1e-6)
        if norm:
            assert out.dtype == dtype
            close(out, plain.rms(want, 1e-5) * w, 3e-6 if dtype == torch.float32 else 6e-3)
        else:
            assert out is None
    with pytest.raises(ops.KernelError):
        ops.stream_scaled_sum(dev(x))
    with pytest.raises(ops.KernelError):
        ops.stream_scaled_sum(dev(x), dev(y1)[:, :-1])


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("T,H", [(1, 24), (7, 33), (9, 2048), (30, 1100)])
def test_mixes_made_behind_the_norm(gpu_device, dtype, T, H):
    """Rows that are sequences of one token: the norm's kernel makes the time mixer's inputs as well,
    the same that time_shift makes from its result."""
    from pytriton_llama_amd import ops
    torch.manual_seed(H)
    stream, y1 = torch.randn(T, H).cuda(), torch.randn(T, H).cuda()
    w, mu = torch.randn(H).cuda(), torch.rand(5, H).cuda()
    state = torch.randn(T + 2, H + 6).to(dtype).float().cuda()
    slots = i32((torch.randperm(T + 2)[:T]).tolist())
    again = stream.clone()
    h, mixed = ops.stream_scaled_sum(stream, y1, norm_weight=w, eps=1e-5, out_dtype=dtype,
                                     mixes=ops.TimeMixes(mu, state, 4, slots))
    assert torch.equal(h, ops.stream_scaled_sum(again, y1, norm_weight=w, eps=1e-5, out_dtype=dtype))
    assert torch.equal(stream, again)
    assert torch.equal(mixed, ops.time_shift(h, mu, state, 4, i32(range(T + 1)), slots))
    with pytest.raises(ops.KernelError):
        ops.stream_scaled_sum(stream, y1, norm_weight=w, out_dtype=dtype, mixes=ops.TimeMixes(mu, state, 7, slots))
    with pytest.raises(ops.KernelError):
        ops.stream_scaled_sum(stream, y1, norm_weight=w, out_dtype=dtype, mixes=ops.TimeMixes(mu, state, 0, slots[:-1]))


# ---- feed-forwards -----------------------------------------------------------------------------
@pytest.mark.parametrize("M", [1, 5, 16, 24, 60, 130])
@pytest.mark.parametrize("activation", ["clamped", "silu"])
def test_gated_feed_forward(gpu_device, M, activation):
    """Every kernel that it may take (fused with the products for few rows, the elementwise kernel
    for many), in both dtypes."""
    from pytriton_llama_amd.parts import GatedMLP
    torch.manual_seed(M)
    K, I, limit = 256, 192, 0.7
    w = {k: torch.randn(*s) * 0.1 for k, s in (("gate", (I, K)), ("up", (I, K)), ("down", (K, I)))}
    x = torch.randn(M, K)
    for dtype in DTYPES:
        part = GatedMLP(K, I, activation, limit)
        part.load(w, dtype, "cuda:0")
        part.make_decode_copies()
        wd = {k: v.to(dtype).double() for k, v in w.items()}
        xd = x.to(dtype).double()
        want = plain.clamped_ff(xd, wd, "", limit) if activation == "clamped" else plain.silu_ff(xd, wd, "")
        close(part.forward(dev(x, dtype)), want, 1e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("T,E,top", [(1, 3, 1), (9, 5, 5), (70, 13, 5), (33, 70, 6), (5, 300, 8)])
def test_routing_by_the_softmax_over_the_chosen(gpu_device, T, E, top):
    from pytriton_llama_amd import ops
    torch.manual_seed(E)
    z, b = torch.randn(T, E), torch.randn(E) * 3
    z[0] *= 200.0                            # (scores of the whole softmax that vanish in float32)
    r = ops.moe_route(dev(z), E, top, 0, True, ops.SCORE_SOFTMAX, logit_bias=dev(b))
    best, which = torch.topk((z + b).double(), top, dim=-1)
    assert torch.equal(r.idx.view(T, top).cpu().long(), which)
    close(r.wgt.view(T, top), torch.softmax(best, -1), 2e-6)


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("shared", [0, 40])
@pytest.mark.parametrize("T", [1, 6, 30, 150])
def test_routed_experts(gpu_device, T, shared, dtype):
    from pytriton_llama_amd.parts import GatedMLP, RoutedExperts
    torch.manual_seed(T + shared)
    W, I, E, top = 64, 48, 7, 3
    part = RoutedExperts(W, I, E, top, activation="silu", weight_on_input=False, renormalize=True, score="softmax",
                         router_bias_name="router.b", shared=GatedMLP(W, shared) if shared else None, shared_gate=False)
    w = {s.name: torch.randn(s.shape) * (0.15 if len(s.shape) > 1 else 1.0) for s in part.param_sources()}
    w["router"] = w["router"] * 8
    part.load(w, dtype, "cuda:0")
    x = torch.randn(T, W).to(dtype)
    wd = {k: (v.to(dtype).double() if v.dim() > 1 else v.double()) for k, v in w.items()}
    mlp = {"router": {"experts": E, "top": top}, "shared": {"ff": shared} if shared else None}
    z = x.double() @ wd["router"].T + wd["router.b"]
    order = z.sort(-1, descending=True).values
    clear = (order[:, top - 1] - order[:, top]) > 1e-3      # (a tie may go either way)
    want = plain.routed(x.double(), mlp, wd, "")
    got = part.forward(x.cuda()).cpu()
    close(got[clear], want[clear], 1e-5 if dtype == torch.float32 else 2e-2)
    # the sum left to the kernel that adds it to the stream
    from pytriton_llama_amd import ops
    assert part.can_defer_sum
    stream, scale, nw = torch.randn(T, W), torch.randn(W), torch.randn(W)
    left = part.forward(x.cuda(), defer_sum=True)
    assert isinstance(left, ops.RoutedSum) and left.shape == (T, W)
    close(left.tensor()[clear.cuda()], want[clear], 1e-5 if dtype == torch.float32 else 2e-2)
    held = stream.cuda()
    out = ops.stream_scaled_sum(held, y2=left, scale2=scale.cuda(), norm_weight=nw.cuda(), eps=1e-5, out_dtype=dtype)
    total = stream.double() + scale.double() * left.tensor().double().cpu()
    close(held, total, 1e-6)
    close(out, plain.rms(total, 1e-5) * nw.double(), 3e-6 if dtype == torch.float32 else 6e-3)


# ---- attention with capped scores ----------------------------------------------------------------
# (H, G, Dk, Dv, page size, chunk, window, cap)
CAP_CASES = [(4, 2, 32, 32, 16, 48, 0, 4.0), (5, 1, 64, 64, 16, 90, 0, 20.0), (4, 4, 128, 128, 32, 100, 0, 9.0),
             (3, 3, 24, 40, 8, 5, 0, 2.0), (4, 1, 32, 64, 16, 16, 0, 15.0), (8, 2, 64, 32, 4, 1, 0, 5.0),
             (2, 2, 96, 96, 16, 1000, 0, 50.0), (6, 2, 96, 64, 16, 170, 0, 17.0), (2, 1, 18, 20, 4, 64, 0, 7.0),
             (5, 5, 128, 64, 16, 130, 0, 12.0), (4, 2, 64, 64, 16, 0, 70, 6.0), (4, 2, 64, 64, 16, 0, 0, 6.0)]


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("case", CAP_CASES, ids=str)
def test_every_attention_kernel_with_capped_scores(gpu_device, case, dtype):
    """Shuffled pages, those of chunks that are over missing; raw scores far beyond the cap (the key in
    front of the chunk's would win by far if it were seen); portions behind a prefix, a 300-row prompt
    over several chunks, decoded tokens at a chunk's last, first and an inner place."""
    from pytriton_llama_amd import ops
    from pytriton_llama_amd.engine.batch import work_items
    H, G, Dk, Dv, P, chunk, window, cap = case
    torch.manual_seed(chunk * 11 + Dk)
    scale = 0.3
    c = chunk or 50
    dec = [2 * c, 2 * c + 1, 2 * c + c // 2 + 1] if c < 300 else [211, 212, 150]     # contexts of decoded tokens
    lens, qlens = dec + [150, 300], [1, 1, 1, 40, 300]
    order = torch.randperm(sum(-(-n // P) for n in lens)).tolist()
    k_pool = torch.randn(len(order), G, P, Dk, dtype=torch.float64) * 5
    v_pool = torch.randn(len(order), G, P, Dv, dtype=torch.float64) * 5
    bt = torch.full((len(lens), -(-max(lens) // P)), -1, dtype=torch.int32)
    sink = torch.zeros(H, dtype=torch.float64)
    qs, want, bare, at = [], [], [], 0
    for r, (n, ql) in enumerate(zip(lens, qlens)):
        k, v, q = (torch.randn(*s, dtype=torch.float64) for s in ((n, G, Dk), (n, G, Dv), (ql, H, Dk)))
        first = (n - 1) // c * c
        if chunk:
            k[first] *= 3.0
            q[-1, 0] = k[first, 0] * (64.0 / Dk)
            if first > 0:
                k[first - 1] = k[first] * 1.5
        q, k, v = (t.to(dtype).double() for t in (q, k, v))
        i, j = torch.arange(n - ql, n)[:, None], torch.arange(n)[None, :]
        seen = j <= i
        if chunk:
            seen = seen & (i // chunk == j // chunk)
        if window:
            seen = seen & (i - j < window)
        s = torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(H // G, 1)) * scale
        for out, scores in ((want, plain.softcap(s, cap)), (bare, s)):
            out.append(torch.einsum("hij,jhe->ihe", plain.softmax_with_one(scores, seen), v.repeat_interleave(H // G, 1)))
        table = order[at:at + -(-n // P)]
        at += len(table)
        needed = (n - ql) // chunk * chunk // P if chunk else max(0, n - ql - window + 1) // P if window else 0
        for i, pg in enumerate(table):
            bt[r, i] = pg if i >= needed else -1
        for i in range(n):
            k_pool[table[i // P], :, i % P] = k[i]
            v_pool[table[i // P], :, i % P] = v[i]
        qs.append(q)
    want_all, q_all = torch.cat(want), dev(torch.cat(qs), dtype)
    tol = 2e-5 if dtype == torch.float32 else 1.5e-2
    if cap <= 9.0 and chunk != 1:            # the cap is felt
        assert float((torch.cat(bare) - want_all).abs().max() / want_all.abs().max()) > 10 * tol
    kp, vp = dev(k_pool, dtype), dev(v_pool, dtype)
    q_start, ctx = i32([0] + torch.tensor(qlens).cumsum(0).tolist()), i32(lens)
    extras = dict(chunk=chunk, sink=dev(sink), softcap=cap)
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


def test_what_the_kernels_refuse(gpu_device):
    from pytriton_llama_amd import ops
    q = torch.zeros(1, 2, 16, device="cuda")
    kv = torch.zeros(1, 2, 4, 16, device="cuda")
    with pytest.raises(ops.KernelError):
        ops.attention_generic(torch.empty_like(q), q, kv, kv, i32([0, 1]), i32([1]), i32([[0]]), i32([0]), i32([0]), 0.25,
                              softcap=-1.0)
    p = torch.zeros(4, 64, device="cuda")
    y = torch.empty(4, 2, 8, device="cuda")
    floats = ops.linear_state_floats(2, 8, 8)
    state = torch.zeros(2, floats + 8, device="cuda")
    args = (y, p, p, p, 2, 8, state, i32([0, 4]), i32([0]), 4)
    decay, u = torch.ones(4, 16, device="cuda"), torch.ones(2, 8, device="cuda")
    for bad in (dict(bonus=u), dict(decay=decay, bonus=u[:1]), dict(decay=decay, bonus=u, keep=(p[:, :8], floats - 4)),
                dict(decay=decay, bonus=u, keep=(p[:, :9], floats)), dict(decay=decay, bonus=u, keep=(p[:2, :8], floats))):
        with pytest.raises(ops.KernelError):
            ops.linear_scan(*args, **bad)
    with pytest.raises(ops.KernelError):                     # kept rows outside the slots
        ops.time_shift(p, torch.zeros(3, 64, device="cuda"), state, floats, i32([0, 4]), i32([0]))
