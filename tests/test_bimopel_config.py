"""Bimopel's configuration, builder and cache needs on the CPU, and the plain implementation's own
pieces on hand-made inputs."""
import copy
import math

import pytest
import torch

import plain_bimopel as plain
from bimopel_configs import BIMOPEL, bimopel, drawn


def test_config_reads_every_size_and_constant():
    from pytriton_llama_amd.config import BimopelConfig
    cfg, _, _ = bimopel("B1")
    c = BimopelConfig.from_dict(cfg)
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.embedding_scale, c.postln_alpha, c.logit_softcap) == \
        (200, 64, 1e-5, 8.0, 1.7, 12.0)
    assert [l.kind for l in c.layers] == ["mamba2", "parallel", "mamba2", "parallel", "mamba2"]
    assert [l.ff for l in c.layers] == [0, 96, 80, 0, 0]
    m, p = c.layers[0].mixer, c.layers[1].mixer
    assert (m.heads, m.vdim, m.state, m.groups, m.conv, m.norm_groups) == (4, 24, 20, 2, 4, 3)
    assert (p.left.heads, p.left.kv_heads, p.left.dim, p.left.vdim, p.left.scale, p.left.chunk) == (4, 2, 24, 16, 0.3, 24)
    assert (p.right.heads, p.right.dim, p.right.vdim, p.right.tau, p.right.rank) == (3, 20, 28, 8.0, 7)
    assert c.to_dict() == cfg
    b3 = BimopelConfig.from_dict(bimopel("B3")[0])
    assert b3.logit_softcap is None and b3.layers[2].mixer.left.chunk is None


@pytest.mark.parametrize("change,text", [
    (lambda c: c["layers"][0].update(type="mamba1"), "unknown layer type"),
    (lambda c: c["layers"][0]["mixer"].pop("state"), "lacks 'state'"),
    (lambda c: c["layers"][0]["mixer"].update(groups=3), "not a multiple of 3 groups"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=7), "7 norm_groups"),
    (lambda c: c["layers"][0]["mixer"].update(conv=0), "conv must be positive"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "not a multiple"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=-4), "size must be positive"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(mask={"length": 3}), "lacks 'size'"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(tau=0), "tau must be positive"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "lacks 'right'"),
    (lambda c: c["layers"][1]["mlp"].update(kind="moe"), "unknown feed-forward kind"),
    (lambda c: c.pop("postln_alpha"), "lacks 'postln_alpha'"),
    (lambda c: c.pop("embedding"), "lacks 'embedding'"),
    (lambda c: c.update(logit_softcap=-1.0), "logit_softcap must be positive"),
    (lambda c: c.update(layers=[]), "empty"),
])
def test_config_errors_name_the_place(change, text):
    from pytriton_llama_amd.config import BimopelConfig, ConfigError
    cfg, _, _ = bimopel("B1")
    change(cfg)
    with pytest.raises(ConfigError) as e:
        BimopelConfig.from_dict(cfg)
    assert text in str(e.value)


@pytest.mark.parametrize("name", sorted(BIMOPEL) + [5, 6])
def test_builder_wires_caches_and_names(name):
    import pytriton_llama_amd  # noqa: F401
    from pytriton_llama_amd.config import build_model
    from pytriton_llama_amd.parts import PagedSpec, StateSpec
    cfg = bimopel(name)[0] if isinstance(name, str) else drawn(name)[0]
    model = build_model(cfg)
    assert [c.block for c in model.schedule] == list(range(len(cfg["layers"])))
    names = {k: src.shape for k, (_, src) in model.expected_tensors().items()}
    W = cfg["width"]
    want = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    for i, (layer, call) in enumerate(zip(cfg["layers"], model.schedule)):
        m, pre = layer["mixer"], f"l{i}.mix."
        want[f"l{i}.norm1"] = (W,)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            want.update({f"l{i}.norm2": (W,), f"l{i}.mlp.gate": (ff, W), f"l{i}.mlp.up": (ff, W),
                         f"l{i}.mlp.down": (W, ff)})
        if layer["type"] == "mamba2":
            spec = model.cache_layers[call.cache_layer]
            inner, C = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            assert isinstance(spec, StateSpec) and spec.dtype == torch.float32
            assert spec.shape[0] >= inner * m["state"] + (m["conv"] - 1) * C
            want.update({pre + "in": (inner + C + m["heads"], W), pre + "conv": (C, m["conv"]), pre + "conv.b": (C,),
                         pre + "dt_bias": (m["heads"],), pre + "A_log": (m["heads"],), pre + "D": (m["heads"],),
                         pre + "norm": (inner,), pre + "o": (W, inner)})
            continue
        left, right = (model.cache_layers[c] for c in call.cache_layer)
        l, r = m["left"], m["right"]
        assert isinstance(left, PagedSpec) and isinstance(right, StateSpec) and right.dtype == torch.float32
        assert left.chunk == (l["mask"]["size"] if "mask" in l else None) and left.window is None
        assert [t.shape for t in left.tensors] == [(l["kv_heads"], l["dim"]), (l["kv_heads"], l["vdim"])]
        q, k, v = l["heads"] * l["dim"], l["kv_heads"] * l["dim"], l["kv_heads"] * l["vdim"]
        R, HD, HV = r["rank"], r["heads"] * r["dim"], r["heads"] * r["vdim"]
        lp, rp = pre + "left.", pre + "right."
        want.update({lp + "q": (q, W), lp + "q.b": (q,), lp + "k": (k, W), lp + "k.b": (k,), lp + "v": (v, W),
                     lp + "v.b": (v,), lp + "q.norm": (q,), lp + "k.norm": (k,), lp + "g": (l["heads"], W),
                     lp + "o": (W, l["heads"] * l["vdim"]), lp + "out": (W,),
                     rp + "q": (HD, W), rp + "k": (HD, W), rp + "v": (HV, W), rp + "g": (HV, W), rp + "o": (W, HV),
                     rp + "norm": (r["vdim"],), rp + "a1": (R, W), rp + "a2": (HD, R), rp + "a2.b": (HD,),
                     rp + "out": (W,)})
    assert names == want


def test_the_rank_of_the_decays_comes_from_the_checkpoint(tmp_path):
    """A config.json without it: the tensors' shapes say (random weights are drawn with the default)."""
    from safetensors.torch import load_file
    from pytriton_llama_amd.config import build_model, read_config_json
    from pytriton_llama_amd.weights import WeightError, load_weights, write_random_model
    cfg, std, _ = bimopel("B1")
    write_random_model(cfg, str(tmp_path), seed=1, dtype=torch.float32, norm_std=0.1, std=std)
    silent = copy.deepcopy(cfg)
    for l in silent["layers"]:
        l["mixer"].get("right", {}).pop("rank", None)
    model = build_model(silent)
    load_weights(model, str(tmp_path), torch.float32, "cpu")
    ranks = [b.mixer.right.rank for b in model.blocks if hasattr(b.mixer, "right")]
    assert ranks == [7, 16]
    w = load_file(str(tmp_path / "model.safetensors"))
    assert set(w) == set(build_model(read_config_json(str(tmp_path))).expected_tensors())
    w["l1.mix.right.a2"] = w["l1.mix.right.a2"][:, :5].contiguous()
    from safetensors.torch import save_file
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(WeightError) as e:
        load_weights(build_model(silent), str(tmp_path), torch.float32, "cpu")
    assert "l1.mix.right.a2" in str(e.value)


def test_pages_of_a_chunk_that_is_over_are_given_back():
    from pytriton_llama_amd.cache import RELEASED, CacheManager
    from pytriton_llama_amd.parts import PagedSpec, PagedTensor
    kv = (PagedTensor("k", (1, 8), 1), PagedTensor("v", (1, 8), 1))
    m = CacheManager([PagedSpec(kv, chunk=10), PagedSpec(kv, chunk=3), PagedSpec(kv)], 4, 12, 2)
    m.admit("a")
    held = []
    for n in range(1, 34):
        m.append("a", 1)
        m.release_behind_window("a")
        m.check()
        for g, size in ((0, 10), (1, 3)):
            first = n // size * size // 4                 # page of the next query's first key
            table = m.block_table("a", g)
            assert all(p == RELEASED for p in table[:first]) and all(p >= 0 for p in table[first:])
        assert all(p >= 0 for p in m.block_table("a", 2))
        held.append(12 - m.paged[0].pool.num_free)
    assert max(held) == 3                                 # a chunk of 10 touches at most three pages here
    m.free("a")
    assert all(g.pool.num_free == 12 for g in m.paged)
    with pytest.raises(ValueError):
        PagedSpec(kv, window=4, chunk=4)
    with pytest.raises(ValueError):
        PagedSpec(kv, chunk=0)


def test_random_model_folder_round_trip(tmp_path):
    from safetensors.torch import load_file
    from pytriton_llama_amd.config import build_model, read_config_json
    from pytriton_llama_amd.weights import load_weights, write_random_model
    cfg, std, _ = bimopel("B2")
    write_random_model(cfg, str(tmp_path), seed=1, dtype=torch.float32, norm_std=0.1, std=std)
    model = build_model(read_config_json(str(tmp_path)))
    load_weights(model, str(tmp_path), torch.float32, "cpu")
    w = load_file(str(tmp_path / "model.safetensors"))
    logits = plain.forward(cfg, w, [1, 2, 3, 4, 5])
    assert logits.shape == (5, cfg["vocab"]) and bool(torch.isfinite(logits).all())
    assert float(logits.abs().max()) < cfg["logit_softcap"]


def test_plain_pieces_on_hand_made_inputs():
    # positions: the first entries of position 1 of width 4, and position 0
    v = plain.position_vectors(2, 4)
    assert torch.allclose(v[0], torch.tensor([0.0, 1.0, 0.0, 1.0], dtype=torch.float64))
    assert torch.allclose(v[1], torch.tensor([math.sin(1), math.cos(1), math.sin(0.01), math.cos(0.01)],
                                             dtype=torch.float64))
    # chunks of 3: token 3 sees itself alone, token 5 sees 3 to 5
    m = plain.chunk_mask(7, 3)
    assert m[3].tolist() == [False, False, False, True, False, False, False]
    assert m[5].tolist() == [False, False, False, True, True, True, False]
    assert torch.equal(plain.chunk_mask(5, None), torch.ones(5, 5, dtype=torch.bool).tril())
    # one seen key of score 0 beside the added term: half
    p = plain.softmax_with_one(torch.zeros(1, 2), torch.tensor([[True, False]]))
    assert p.tolist() == [[0.5, 0.0]]
    big = plain.softmax_with_one(torch.tensor([[500.0, 500.0]]), torch.tensor([[True, True]]))
    assert torch.allclose(big, torch.tensor([[0.5, 0.5]]))
    small = plain.softmax_with_one(torch.tensor([[-500.0, -500.0]]), torch.tensor([[True, True]]))
    assert float(small.abs().max()) == 0.0
    # the recurrence: a decay of one half a step on the first channel, none on the second
    one = torch.ones(3, 1, 2, dtype=torch.float64)
    la = torch.log(torch.tensor([0.5, 1.0], dtype=torch.float64)).expand(3, 1, 2)
    o = plain.linear_recurrence(one, one, torch.ones(3, 1, 1, dtype=torch.float64), la)
    assert o[:, 0, 0].tolist() == [2.0, 3.5, 4.75]
    # the convolution's last tap is the current token's, zeros stand before the start
    x = torch.tensor([[1.0], [2.0], [3.0]])
    assert plain.short_conv(x, torch.tensor([[10.0, 1.0]]), torch.tensor([0.5])).flatten().tolist() == [1.5, 12.5, 23.5]
    z = torch.tensor([-3.0, -0.5, 0.0, 1.0, 4.0], dtype=torch.float64)
    assert torch.allclose(plain.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert torch.allclose(plain.softcap(torch.tensor([1e-3, 100.0]), 2.0), torch.tensor([1e-3, 2.0]), atol=1e-6)
