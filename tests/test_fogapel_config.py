"""Fogapel's configuration, builder and cache needs on the CPU, and the plain implementation's own
pieces on hand-made inputs."""
import copy
import math

import pytest
import torch

import plain_fogapel as plain
from fogapel_configs import FOGAPEL, drawn, fogapel


def test_config_reads_every_size_and_constant():
    from pytriton_llama_amd.config import FogapelConfig
    cfg, _, _ = fogapel("F1")
    c = FogapelConfig.from_dict(cfg)
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.embedding_scale) == (200, 64, 1e-5, 8.0)
    assert [l.kind for l in c.layers] == ["wkv", "wkv", "attention", "attention", "wkv"]
    w, a = c.layers[0].mixer, c.layers[2].mixer
    assert (w.heads, w.dim, w.rank) == (3, 20, 7)
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.conv, a.chunk, a.rot_dims, a.rot_base, a.softcap) == \
        (4, 2, 24, 16, 0.4, 4, 24, 16, 10000.0, 8.0)
    d, m, s = (c.layers[i].mlp for i in range(3))
    assert (d.kind, d.ff, d.limit) == ("dense", 96, 1.2)
    assert (m.kind, m.ff, m.experts, m.top, m.shared_ff) == ("moe", 32, 6, 2, 0)
    assert (s.ff, s.experts, s.top, s.shared_ff) == (24, 5, 3, 40)
    assert c.layers[3].mlp is None and c.to_dict() == cfg
    f2 = FogapelConfig.from_dict(fogapel("F2")[0]).layers[2].mixer
    assert (f2.rot_dims, f2.softcap, f2.conv) == (0, None, 7)
    f3 = FogapelConfig.from_dict(fogapel("F3")[0]).layers[2].mixer
    assert f3.chunk is None and f3.conv == 0


@pytest.mark.parametrize("change,text", [
    (lambda c: c["layers"][0].update(type="rwkv"), "unknown layer type"),
    (lambda c: c["layers"][0]["mixer"].pop("heads"), "lacks 'heads'"),
    (lambda c: c["layers"][0]["mixer"].update(dim=0), "dim must be positive"),
    (lambda c: c["layers"][2]["mixer"].update(kv_heads=3), "not a multiple"),
    (lambda c: c["layers"][2]["mixer"].update(conv=0), "conv must be positive"),
    (lambda c: c["layers"][2]["mixer"]["mask"].update(size=-4), "size must be positive"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=26), "at most dim"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=3), "must be even"),
    (lambda c: c["layers"][2]["mixer"]["rot"].pop("base"), "lacks 'base'"),
    (lambda c: c["layers"][2]["mixer"].update(softcap=-1.0), "softcap must be positive"),
    (lambda c: c["layers"][2]["mixer"].pop("scale"), "lacks 'scale'"),
    (lambda c: c["layers"][0]["mlp"].update(kind="glu"), "unknown feed-forward kind"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "lacks 'limit'"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=7), "top 7 of 6"),
    (lambda c: c["layers"][1]["mlp"].pop("expert"), "lacks 'expert'"),
    (lambda c: c["layers"][2]["mlp"]["shared"].update(ff=0), "ff must be positive"),
    (lambda c: c.pop("embedding"), "lacks 'embedding'"),
    (lambda c: c.update(layers=[]), "empty"),
])
def test_config_errors_name_the_place(change, text):
    from pytriton_llama_amd.config import ConfigError, FogapelConfig
    cfg, _, _ = fogapel("F1")
    change(cfg)
    with pytest.raises(ConfigError) as e:
        FogapelConfig.from_dict(cfg)
    assert text in str(e.value)


@pytest.mark.parametrize("name", sorted(FOGAPEL) + [5, 6, 7])
def test_builder_wires_caches_and_names(name):
    import pytriton_llama_amd  # noqa: F401
    from pytriton_llama_amd.config import build_model
    from pytriton_llama_amd.parts import PagedSpec, StateSpec
    cfg = fogapel(name)[0] if isinstance(name, str) else drawn(name)[0]
    net = build_model(cfg)
    assert [c.block for c in net.schedule] == list(range(len(cfg["layers"])))
    names = {k: src.shape for k, (_, src) in net.expected_tensors().items()}
    W = cfg["width"]
    want = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}

    def gated(pre, ff):
        want.update({pre + "gate": (ff, W), pre + "up": (ff, W), pre + "down": (W, ff)})
    for i, (entry, call) in enumerate(zip(cfg["layers"], net.schedule)):
        m, mlp, pre = entry["mixer"], entry["mlp"], f"l{i}.mix."
        want.update({f"l{i}.norm1": (W,), f"l{i}.ls1": (W,)})
        if mlp is not None:
            want[f"l{i}.ls2"] = (W,)
            if mlp["kind"] == "dense":
                gated(f"l{i}.mlp.", mlp["ff"])
            else:
                E = mlp["router"]["experts"]
                want.update({f"l{i}.mlp.router": (E, W), f"l{i}.mlp.router.b": (E,)})
                for e in range(E):
                    gated(f"l{i}.mlp.e{e}.", mlp["expert"]["ff"])
                if "shared" in mlp:
                    gated(f"l{i}.mlp.shared.", mlp["shared"]["ff"])
        else:
            assert net.is_ignorable(f"l{i}.ls2")
        if entry["type"] == "wkv":
            spec, C = net.cache_layers[call.cache_layer], m["heads"] * m["dim"]
            assert isinstance(spec, StateSpec) and spec.dtype == torch.float32 and spec.shape[0] >= C * m["dim"] + W
            want.update({pre + "mu." + x: (W,) for x in "rkvgw"})
            want.update({pre + x: (C, W) for x in "rkvg"})
            want.update({pre + "w1": (m["rank"], W), pre + "w2": (C, m["rank"]), pre + "w0": (C,),
                         pre + "u": (m["heads"], m["dim"]), pre + "norm": (C,), pre + "o": (W, C)})
            continue
        sizes = {"q": m["heads"] * m["dim"], "k": m["kv_heads"] * m["dim"], "v": m["kv_heads"] * m["vdim"]}
        taps = m.get("conv", 0)
        if taps > 1:
            pages, state = (net.cache_layers[c] for c in call.cache_layer)
            assert isinstance(state, StateSpec) and state.dtype == torch.float32
            assert state.shape == ((taps - 1) * sum(sizes.values()),)
        else:
            pages = net.cache_layers[call.cache_layer]
        assert isinstance(pages, PagedSpec) and pages.window is None
        assert pages.chunk == (m["mask"]["size"] if "mask" in m else None)
        assert [t.shape for t in pages.tensors] == [(m["kv_heads"], m["dim"]), (m["kv_heads"], m["vdim"])]
        for x, n in sizes.items():
            want.update({pre + x: (n, W), pre + x + ".b": (n,)})
            if taps:
                want[pre + x + ".conv"] = (n, taps)
        want.update({pre + "o": (W, m["heads"] * m["vdim"]), pre + "o.b": (W,)})
    assert names == want


def test_the_rank_of_the_decays_comes_from_the_checkpoint(tmp_path):
    """A config.json without it: the tensors' shapes say (random weights are drawn with the default)."""
    from safetensors.torch import load_file, save_file
    from pytriton_llama_amd.config import build_model, read_config_json
    from pytriton_llama_amd.weights import WeightError, load_weights, write_random_model
    cfg, std, _ = fogapel("F1")
    write_random_model(cfg, str(tmp_path), seed=1, dtype=torch.float32, norm_std=0.1, std=std)
    silent = copy.deepcopy(cfg)
    for l in silent["layers"]:
        l["mixer"].pop("rank", None)
    net = build_model(silent)
    load_weights(net, str(tmp_path), torch.float32, "cpu")
    assert [b.mixer.rank for b in net.blocks if hasattr(b.mixer, "rank")] == [7, 16, 5]
    w = load_file(str(tmp_path / "model.safetensors"))
    assert set(w) == set(build_model(read_config_json(str(tmp_path))).expected_tensors())
    w["l0.mix.w2"] = w["l0.mix.w2"][:, :5].contiguous()
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(WeightError) as e:
        load_weights(build_model(silent), str(tmp_path), torch.float32, "cpu")
    assert "l0.mix.w2" in str(e.value)


def test_random_model_folder_round_trip(tmp_path):
    from safetensors.torch import load_file
    from pytriton_llama_amd.config import build_model, read_config_json
    from pytriton_llama_amd.weights import load_weights, write_random_model
    cfg, std, _ = fogapel("F2")
    write_random_model(cfg, str(tmp_path), seed=1, dtype=torch.float32, norm_std=0.1, std=std)
    load_weights(build_model(read_config_json(str(tmp_path))), str(tmp_path), torch.float32, "cpu")
    w = load_file(str(tmp_path / "model.safetensors"))
    logits = plain.forward(cfg, w, [1, 2, 3, 4, 5])
    assert logits.shape == (5, cfg["vocab"]) and bool(torch.isfinite(logits).all())


def test_what_the_mixers_refuse():
    from pytriton_llama_amd.parts import NormedAttention, TimeMixer
    ok = dict(hidden_size=16, num_heads=2, num_kv_heads=1, dim=8, vdim=8)
    for bad in (dict(taps=3), dict(rot_layout="pairs"), dict(qk_norm="rotated", maps=2),
                dict(qk_norm="rotated", own_kv=False), dict(qk_norm="rotated", rot_layout="thirds"),
                dict(qk_norm="rotated", softcap=-1.0), dict(softcap=5.0, window=9, keep_first=2), dict(qk_norm="rotated", taps=-1), dict(qk_norm="last")):
        with pytest.raises(ValueError):
            NormedAttention(**ok, **bad)
    with pytest.raises(ValueError):
        TimeMixer(16, 1, 300, 1e-5)


def test_plain_pieces_on_hand_made_inputs():
    D = torch.float64
    # pairs of neighbours: at position 1 of base 1 (angle 1 for every pair) the unit vector turns by one radian
    x = torch.tensor([[[1.0, 0.0, 0.0, 1.0, 5.0]]], dtype=D).repeat(2, 1, 1)
    y = plain.rotate_pairs(x, 4, 1.0)
    assert torch.equal(y[0], x[0])
    c, s = math.cos(1), math.sin(1)
    assert torch.allclose(y[1, 0], torch.tensor([c, s, -s, c, 5.0], dtype=D))
    # ... and the second pair of four entries by p base^(-1/2)
    z = plain.rotate_pairs(x, 4, 100.0)[1, 0]
    assert torch.allclose(z[2:4], torch.tensor([-math.sin(0.1), math.cos(0.1)], dtype=D))
    # the convolution's last tap is the current token's, zeros stand before the start
    u = torch.tensor([[1.0], [2.0], [3.0]])
    assert plain.short_conv(u, torch.tensor([[10.0, 1.0]])).flatten().tolist() == [1.0, 12.0, 23.0]
    # time mix: mu 0 the row itself, mu 1 the row before (zeros first)
    h = torch.tensor([[1.0, 1.0], [3.0, 3.0]])
    assert plain.time_mix(h, torch.tensor([0.0, 1.0])).tolist() == [[1.0, 0.0], [3.0, 1.0]]
    # the recurrence: the current token counts u times, the ones before it decay from their own update on
    one = torch.ones(3, 1, 1, dtype=D)
    la = torch.log(torch.tensor(0.5, dtype=D)).expand(3, 1, 1)
    o = plain.wkv_recurrence(one, one, one, la, torch.full((1, 1), 4.0, dtype=D))
    assert o.flatten().tolist() == [4.0, 5.0, 5.5]
    # one seen key of score 0 beside the added term: half; capped scores
    assert plain.softmax_with_one(torch.zeros(1, 2), torch.tensor([[True, False]])).tolist() == [[0.5, 0.0]]
    assert torch.allclose(plain.softcap(torch.tensor([1e-3, 100.0]), 2.0), torch.tensor([1e-3, 2.0]), atol=1e-6)
    assert plain.softcap(torch.tensor([50.0]), None).tolist() == [50.0]
    # chunks of 3: token 3 sees itself alone, token 5 sees 3 to 5
    m = plain.chunk_mask(7, 3)
    assert m[3].tolist() == [False, False, False, True, False, False, False]
    assert m[5].tolist() == [False, False, False, True, True, True, False]
    # routing: the weights are the softmax over the chosen logits alone, the bias counts
    t = {"router": torch.tensor([[1.0], [0.0], [0.5]]), "router.b": torch.tensor([0.0, 3.0, 0.0])}
    for e in range(3):
        t.update({f"e{e}.gate": torch.ones(1, 1), f"e{e}.up": torch.ones(1, 1), f"e{e}.down": torch.full((1, 1), 10.0 ** e)})
    got = plain.routed(torch.ones(1, 1), {"router": {"experts": 3, "top": 2}}, t, "")
    a = torch.softmax(torch.tensor([3.0, 1.0]), 0)
    assert torch.allclose(got, (a[0] * 10 + a[1]).view(1, 1) * plain.silu(torch.ones(1)))
    # the clamped feed-forward: gate from above, up from both sides
    t = {"gate": torch.tensor([[5.0], [-5.0]]), "up": torch.tensor([[-9.0], [9.0]]), "down": torch.tensor([[1.0, 1.0]])}
    sg = lambda v: 1 / (1 + math.exp(-1.702 * v))
    got = plain.clamped_ff(torch.ones(1, 1), t, "", 2.0)
    assert abs(float(got) - (2 * sg(2) * (-2 + 1) - 5 * sg(-5) * (2 + 1))) < 1e-6
