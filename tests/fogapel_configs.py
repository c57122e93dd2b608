"""Small Fogapel configurations for the tests, none of them anyone's model. Between them they vary
every size and every branch: both mixers first and last, dense, routed and no feed-forward behind
either, with and without a shared expert, one to all experts chosen, key and value sizes that are equal,
that differ either way and that are no multiple of 16 or 4, one to four heads a kv head, convolutions
of one to seven taps and none, chunks of one position up to more than a prompt has and none at all,
rotations of all, some and none of a head's entries, with and without a cap on the scores, keys above
128, widths and vocabularies that are no multiple of 8."""
import copy
import random


def attention(heads, kv_heads, dim, vdim, scale, conv=None, size=None, rot=None, softcap=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if conv is not None:
        m["conv"] = conv
    if size is not None:
        m["mask"] = {"size": size}
    if rot is not None:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    if softcap is not None:
        m["softcap"] = softcap
    return "attention", m


def wkv(heads, dim, rank=None):
    m = {"heads": heads, "dim": dim}
    if rank is not None:
        m["rank"] = rank
    return "wkv", m


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def layer(kind_mixer, mlp):
    kind, m = kind_mixer
    return {"type": kind, "mixer": m, "mlp": mlp}


def model(vocab, width, eps, scale, layers):
    return {"architecture": "Fogapel", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": layers}


def _f1():
    return model(200, 64, 1e-5, 8.0, [
        layer(wkv(3, 20, 7), dense(96, 1.2)),
        layer(wkv(2, 16, 16), moe(32, 6, 2)),
        layer(attention(4, 2, 24, 16, 0.4, 4, 24, (10000.0, 16), 8.0), moe(24, 5, 3, 40)),
        layer(attention(6, 3, 16, 32, 0.5, 3, 40, (500.0, 16), 15.0), None),
        layer(wkv(4, 12, 5), None),
    ])


def _f2():
    """Attention first; a width and sizes that are no multiple of 4; chunks of one position and of fewer
    than a page has; one head a kv head; convolutions of one and of seven taps; no rotation and no cap."""
    return model(151, 50, 1e-6, 3.0, [
        layer(attention(3, 3, 18, 22, 0.5, 1, 5, (100.0, 6), 4.0), moe(20, 3, 1, 12)),
        layer(wkv(2, 13, 3), moe(18, 4, 4)),
        layer(attention(2, 1, 12, 20, 0.6, 7, 1, None, None), dense(30, 0.4)),
        layer(wkv(1, 30, 40), None),
    ])


def _f3():
    """Keys above 128, a chunk longer than the prompts, a layer without a mask and without convolutions, one
    with a single pair of entries that turns."""
    return model(120, 96, 1e-4, 1.0, [
        layer(wkv(1, 136, 9), dense(64, 7.0)),
        layer(attention(4, 4, 40, 8, 0.3, 4, 300, (10000.0, 2), 30.0), moe(40, 8, 2, 64)),
        layer(attention(8, 2, 16, 16, 0.5, None, None, (10000.0, 16), 5.0), moe(32, 4, 2)),
        layer(wkv(5, 8, 6), moe(16, 9, 3, 24)),
    ])


def _f4(taps):
    """Attention only: what a token does to the others' logits is the attention's doing alone."""
    return model(200, 64, 1e-5, 6.0, [
        layer(attention(4, 2, 32, 32, 0.3, taps, 48, (10000.0, 32), 9.0), dense(64, 3.0)),
        layer(attention(4, 1, 32, 32, 0.3, taps, 48, (10000.0, 24), 9.0), None),
    ])


def _f5():
    """Sizes that the matrix-core kernels take, keys and values of one size and of two, head sizes of
    real models in the recurrence."""
    return model(184, 96, 1e-5, 5.0, [
        layer(attention(8, 2, 64, 64, 0.25, 4, 80, (10000.0, 64), 12.0), moe(64, 8, 2, 64)),
        layer(wkv(2, 64, 32), moe(64, 8, 3, 32)),
        layer(attention(4, 2, 32, 96, 0.3, 4, 33, (1000.0, 20), 6.0), dense(96, 2.0)),
        layer(wkv(1, 128, 64), dense(64, 1.0)),
        layer(attention(2, 1, 128, 128, 0.1, 2, 64, (10000.0, 128), None), moe(32, 4, 2)),
    ])


def _f6():
    """Time mixers only: no pages, state slots alone."""
    return model(130, 48, 1e-5, 2.0, [
        layer(wkv(3, 20, 4), moe(24, 3, 2, 16)),
        layer(wkv(4, 12, 17), None),
    ])


# name -> (config, weight std, page size)
FOGAPEL = {"F1": (_f1(), 0.12, 16), "F2": (_f2(), 0.15, 4), "F3": (_f3(), 0.12, 8), "F4": (_f4(1), 0.12, 16),
           "F4c": (_f4(4), 0.12, 16), "F5": (_f5(), 0.12, 16), "F6": (_f6(), 0.15, 16)}


def fogapel(name):
    cfg, std, page = FOGAPEL[name]
    return copy.deepcopy(cfg), std, page


def drawn(seed):
    """(config, weight std, page size) drawn at random from the design's ranges."""
    r = random.Random(seed)

    def any_attention():
        kv = r.choice([1, 2, 3])
        dim = r.choice([16, 24, 32, 64, 96, 128])
        return attention(kv * r.choice([1, 2, 4]), kv, dim, r.choice([dim, 16, 40, 64]), r.choice([0.1, 0.3, 0.5]),
                         r.choice([1, 2, 3, 4, 5]), r.choice([3, 16, 17, 31, 64, 100, 500]),
                         (r.choice([100.0, 10000.0, 500000.0]), r.choice([d for d in (4, 8, 16, dim) if d <= dim])),
                         r.choice([3.0, 10.0, 50.0]))

    def any_wkv():
        return wkv(r.choice([1, 2, 3, 4]), r.choice([8, 15, 16, 32, 48, 64, 80]), r.choice([2, 8, 16, 17, 40]))

    def any_mlp():
        experts = r.choice([2, 5, 8, 12])
        return r.choice([None, dense(r.choice([32, 72]), r.choice([0.5, 1.5, 7.0])),
                         moe(r.choice([16, 40]), experts, r.choice([1, 2, experts]), r.choice([None, 24, 64]))])
    layers = [layer(r.choice([any_attention, any_wkv])(), any_mlp()) for _ in range(r.randint(2, 5))]
    return (model(r.choice([64, 101, 256]), r.choice([32, 50, 56, 80, 100, 128]), r.choice([1e-6, 1e-5, 1e-4]),
                  r.choice([0.5, 4.0, 12.0]), layers), 0.13, r.choice([4, 16, 32]))
