"""Small Bimopel configurations for the tests, none of them anyone's model. Between them they vary
every size and every branch: both mixers first and last, with and without a feed-forward behind
either, key and value sizes that are equal, that differ either way and that are no multiple of 16
or 4, one to four heads a kv head, one to all heads a group of B and C, norm groups that cut
through heads, convolutions of one to seven taps, chunks of one position up to more than a prompt
has and none at all, states above 128, several blocks of 64 value columns, ranks from 3 to 40, with
and without a cap on the logits."""
import copy
import random


def mamba2(heads, vdim, state, groups, conv, norm_groups):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                      "norm_groups": norm_groups}


def parallel(left, right):
    return "parallel", {"left": left, "right": right}


def chunked(heads, kv_heads, dim, vdim, scale, size):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        m["mask"] = {"size": size}
    return m


def gated(heads, dim, vdim, tau, rank=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}
    if rank is not None:
        m["rank"] = rank
    return m


def layer(kind_mixer, ff):
    kind, m = kind_mixer
    return {"type": kind, "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(vocab, width, eps, scale, alpha, softcap, layers):
    cfg = {"architecture": "Bimopel", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "embedding": {"scale": scale}, "postln_alpha": alpha, "layers": layers}
    if softcap is not None:
        cfg["logit_softcap"] = softcap
    return cfg


def _b1():
    return model(200, 64, 1e-5, 8.0, 1.7, 12.0, [
        layer(mamba2(4, 24, 20, 2, 4, 3), None),
        layer(parallel(chunked(4, 2, 24, 16, 0.3, 24), gated(3, 20, 28, 8.0, 7)), 96),
        layer(mamba2(3, 16, 36, 1, 3, 1), 80),
        layer(parallel(chunked(6, 3, 16, 32, 0.2, 40), gated(2, 16, 16, 2.0, 16)), None),
        layer(mamba2(4, 24, 20, 4, 2, 4), None),
    ])


def _b2():
    """Two mixers side by side first and last; sizes that are no multiple of 4; chunks of one position
    and of fewer than a page has; one head a kv head; a convolution of one tap (no inputs kept)."""
    return model(150, 72, 1e-6, 3.0, 0.6, 25.0, [
        layer(parallel(chunked(3, 3, 18, 22, 0.4, 5), gated(2, 13, 9, 1.0, 5)), None),
        layer(mamba2(6, 10, 7, 3, 1, 2), 56),
        layer(parallel(chunked(2, 1, 12, 20, 0.25, 1), gated(1, 30, 34, 24.0, 3)), 100),
    ])


def _b3():
    """States above 128, several blocks of value columns, a chunk longer than the prompts, seven taps, a
    group a head, no cap; a layer without a mask."""
    return model(120, 96, 1e-4, 1.0, 2.5, None, [
        layer(mamba2(2, 70, 136, 2, 7, 7), 64),
        layer(parallel(chunked(4, 4, 40, 8, 0.2, 300), gated(1, 136, 72, 16.0, 40)), 48),
        layer(parallel(chunked(8, 2, 16, 16, 0.3, None), gated(5, 8, 8, 4.0, 6)), None),
        layer(mamba2(5, 8, 16, 1, 2, 5), None),
    ])


def _b4():
    """Attention beside gated linear attention only: with the right halves' weights at nothing, what a
    key does to the logits is the attention's doing alone."""
    return model(200, 64, 1e-5, 6.0, 1.0, 30.0, [
        layer(parallel(chunked(4, 2, 32, 32, 0.18, 48), gated(2, 16, 16, 8.0, 8)), 64),
        layer(parallel(chunked(4, 1, 32, 32, 0.18, 48), gated(2, 16, 16, 8.0, 8)), None),
    ])


def _b5():
    """Sizes that the matrix-core kernels take, keys and values of one size and of two, head sizes of
    real models in the recurrences."""
    return model(180, 96, 1e-5, 5.0, 1.4, 15.0, [
        layer(parallel(chunked(8, 2, 64, 64, 0.15, 80), gated(2, 128, 128, 16.0, 16)), 80),
        layer(mamba2(4, 64, 128, 2, 4, 2), None),
        layer(parallel(chunked(4, 2, 32, 96, 0.2, 33), gated(4, 64, 32, 4.0, 12)), 96),
        layer(mamba2(8, 32, 64, 1, 4, 1), 64),
    ])


def _b6():
    """Mamba-2 layers only: no pages, state slots alone."""
    return model(130, 48, 1e-5, 2.0, 1.1, 9.0, [
        layer(mamba2(3, 20, 12, 3, 4, 1), None),
        layer(mamba2(4, 12, 24, 2, 5, 6), 40),
    ])


# name -> (config, weight std, page size)
BIMOPEL = {"B1": (_b1(), 0.12, 16), "B2": (_b2(), 0.15, 4), "B3": (_b3(), 0.12, 8), "B4": (_b4(), 0.12, 16),
           "B5": (_b5(), 0.12, 16), "B6": (_b6(), 0.15, 16)}


def bimopel(name):
    cfg, std, page = BIMOPEL[name]
    return copy.deepcopy(cfg), std, page


def drawn(seed):
    """(config, weight std, page size) drawn at random from the design's ranges."""
    r = random.Random(seed)

    def any_mamba2():
        heads = r.choice([1, 2, 3, 4, 6, 8])
        vdim = r.choice([8, 12, 16, 24, 48, 64, 80])
        return mamba2(heads, vdim, r.choice([4, 10, 16, 33, 64, 96, 128]),
                      r.choice([g for g in range(1, heads + 1) if heads % g == 0]), r.choice([1, 2, 3, 4, 6]),
                      r.choice([g for g in (1, 2, 3, 4, 8) if heads * vdim % g == 0]))

    def any_parallel():
        kv = r.choice([1, 2, 3])
        dim = r.choice([16, 24, 32, 64, 96, 128])
        left = chunked(kv * r.choice([1, 2, 4]), kv, dim, r.choice([dim, 16, 40, 64]), r.choice([0.1, 0.2, 0.4]),
                       r.choice([3, 16, 17, 31, 64, 100, 500]))
        return parallel(left, gated(r.choice([1, 2, 3, 4]), r.choice([8, 15, 32, 48, 96]), r.choice([8, 20, 64, 66]),
                                    r.choice([1.0, 4.0, 16.0, 30.0]), r.choice([2, 8, 16, 17])))
    layers = [layer(r.choice([any_mamba2, any_parallel])(), r.choice([None, 32, 72])) for _ in range(r.randint(2, 5))]
    return (model(r.choice([64, 101, 256]), r.choice([32, 50, 56, 80, 100, 128]), r.choice([1e-6, 1e-5, 1e-4]),
                  r.choice([1.0, 4.0, 12.0]), r.choice([0.7, 1.0, 2.2]), r.choice([None, 8.0, 30.0]), layers),
            0.13, r.choice([4, 16, 32]))
