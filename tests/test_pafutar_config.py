"""Pafutar's configuration, plan, cache needs and model folder, and the plain implementation on cases worked by hand:
what runs without a GPU."""
import copy
import math
import os

import pytest
import torch

import plain_pafutar as pp
from pafutar_cases import CONFIGS, write_folder

F64 = torch.float64


def test_configuration_round_trip_and_plan():
    from bitnet_c_amd.config import PafutarConfig, architecture_for
    from bitnet_c_amd.config.pafutar import build_pafutar_plan
    for name, raw in CONFIGS.items():
        assert architecture_for(raw).name == "Pafutar"
        c = PafutarConfig.from_dict(raw)
        assert PafutarConfig.from_dict(c.to_dict()) == c and c.to_dict() == raw
        plan = build_pafutar_plan(c)
        own = [i for i, L in enumerate(raw["layers"]) if "weights_of" not in L]
        assert len(plan.layers) == len(own) and len(plan.schedule) == len(raw["layers"])
        assert plan.max_positions == raw["max_positions"] and plan.embedding_multiplier == raw["embedding"]["scale"]
        D = raw["width"]
        t = plan.expected_tensors()
        assert t["embed"].shape == (raw["vocab"], D) == t["head"].shape and t["final.norm"].shape == (D,)
        assert t["pos"].shape == (raw["max_positions"], D)
        for i, (e, L) in enumerate(zip(plan.schedule, raw["layers"])):
            assert e.layer == own.index(L.get("weights_of", i)) and e.kv_from is None
            p, m = f"l{i}.", L["mixer"]
            if "weights_of" in L:
                assert not [n for n in t if n.startswith(p)]
                continue
            H, G, d = m["heads"], m["kv_heads"], m["dim"]
            want = {"norm1": (D,), "ls1": (D,), "shift": (D,), "mix.q": (H * d, D), "mix.q.b": (H * d,), "mix.k": (G * d, D),
                    "mix.k.b": (G * d,), "mix.temp": (H,), "mix.g": (H * d, D), "mix.o": (D, H * d)}
            if L["mlp"] is not None:
                F = L["mlp"]["ff"]
                want.update({"norm2": (D,), "ls2": (D,), "mlp.up": (F, D), "mlp.down": (D, F)})
            assert {n[len(p):]: s.shape for n, s in t.items() if n.startswith(p)} == want


def _bad(raw, change, match):
    from bitnet_c_amd.config import ConfigError, PafutarConfig
    raw = copy.deepcopy(raw)
    change(raw)
    with pytest.raises(ConfigError, match=match):
        PafutarConfig.from_dict(raw)


def test_configurations_that_cannot_be_are_refused():
    A = CONFIGS["A"]
    _bad(A, lambda r: r["layers"][0].update(type="conv"), "type")
    _bad(A, lambda r: r["layers"][0]["mixer"].update(kv_heads=3), "kv_heads")
    _bad(A, lambda r: r["layers"][0]["mixer"].update(vdim=8), "vdim")
    _bad(A, lambda r: r["layers"][0]["mixer"].pop("scale"), "scale")
    _bad(A, lambda r: r["layers"][0]["mixer"]["mask"].update(size=0), "size")
    _bad(A, lambda r: r["layers"][0]["mixer"]["mask"].update(keep_first=-1), "keep_first")
    _bad(A, lambda r: r["layers"][0]["mixer"].update(mask=[24, 3]), "mask")
    _bad(A, lambda r: r["layers"][0]["mlp"].update(kind="moe"), "kind")
    _bad(A, lambda r: r["layers"][2].update(weights_of=2), "weights_of")
    _bad(A, lambda r: r["layers"][2].update(weights_of=1), "differs")
    _bad(A, lambda r: r["layers"][4].update(weights_of=2), "none of its own")
    _bad(A, lambda r: r["layers"][2]["mixer"].update(mask=dict(size=25, keep_first=3)), "differs")
    _bad(A, lambda r: r.pop("norm"), "norm")
    _bad(A, lambda r: r.pop("postln_alpha"), "postln_alpha")
    _bad(A, lambda r: r.pop("max_positions"), "max_positions")
    _bad(A, lambda r: r.update(layers=[]), "layers")


def test_parts_that_cannot_be_are_refused():
    from bitnet_c_amd.parts import BLOCKS, MIXERS, KVNeed, PartSpec
    att = dict(hidden=32, n_heads=4, n_kv_heads=2, head_dim=8, scale=1.0, position=PartSpec.of("none"))
    for extra in (dict(keep_first=2), dict(qk_norm_weight=False), dict(distance_slopes=(0.5, 0.25)), dict(bias="q"),
                  dict(distance_slopes=(1.0,) * 4, distance_bias=True), dict(bias=True, out_gate=True), dict(bias="qk", conv_taps=2),
                  dict(qk_norm_weight=False, qk_norm_eps=1e-6, qk_norm_span="projection")):
        with pytest.raises(ValueError):
            MIXERS.build(PartSpec.of("attention", **att, **extra))
    with pytest.raises(ValueError):
        KVNeed(2, 8, keep_first=3)
    norm = PartSpec.of("rmsnorm", dim=32, eps=1e-6)
    with pytest.raises(ValueError):
        BLOCKS.build(PartSpec.of("postnorm", hidden=32, mixer=PartSpec.of("attention", **att), ffn=None, mixer_norm=norm, ffn_norm=norm))
    with pytest.raises(ValueError):
        BLOCKS.build(PartSpec.of("postnorm", hidden=32, mixer=PartSpec.of("attention", **att), ffn=None,
                                 mixer_norm=PartSpec.of("none", dim=32)))


def test_cache_needs_and_pages_of_kept_first_tokens():
    """Every layer keeps pages for its window and its first tokens, and one row of the stream; layers that run one layer's
    weights have pages and a row each.  Pages below the window are given back, but never those of the kept tokens."""
    from bitnet_c_amd.cache import PAGE, PagedCache
    from bitnet_c_amd.config import PafutarConfig
    from bitnet_c_amd.config.pafutar import build_pafutar_plan
    from bitnet_c_amd.parts import BLOCKS
    raw = CONFIGS["B"]
    plan = build_pafutar_plan(PafutarConfig.from_dict(raw))
    needs = [BLOCKS.build(plan.layers[e.layer].block).cache_need() for e in plan.schedule]
    for need, L in zip(needs, raw["layers"]):
        m, mask = L["mixer"], L["mixer"].get("mask") or dict(size=0, keep_first=0)
        assert (need.kv.n_kv_heads, need.kv.head_dim, need.kv.v_dim) == (m["kv_heads"], m["dim"], m["dim"])
        assert (need.kv.window, need.kv.keep_first) == (mask["size"], mask["keep_first"])
        assert need.state.shape == (raw["width"],) and need.state.dtype == torch.float32 and need.state.device_addressed
    cache = PagedCache(needs, [e.kv_from for e in plan.schedule], 16 * PAGE)
    assert len(cache.groups) == 3 and cache.group_of(0) == cache.group_of(3)
    s = cache.alloc_slot()
    n = 6 * PAGE + 10
    cache.reserve([s], [n])
    cache.commit([s], [n])
    held = {g: [i for i, p in enumerate(cache.pages_of(g, s)) if p >= 0] for g in range(3)}
    assert held[cache.group_of(0)] == [0, 5, 6]                 # window 33, one kept token: the page of position 0, then the window's
    assert held[cache.group_of(1)] == [0, 1, 6]                 # window 5, 70 kept tokens: two pages of them
    assert held[cache.group_of(2)] == list(range(7))            # no window: everything
    for _ in range(2 * PAGE):
        cache.reserve([s], [1])
        cache.commit([s], [1])
    held = {g: [i for i, p in enumerate(cache.pages_of(g, s)) if p >= 0] for g in range(3)}
    assert held[cache.group_of(1)] == [0, 1, 8] and held[cache.group_of(0)] == [0, 7, 8]
    cache.check()
    cache.free_slot(s)
    cache.check()
    assert all(g.pool.n_free == g.pool.n_pages for g in cache.groups)


def test_a_mixer_state_lies_in_front_of_the_shifted_row():
    from bitnet_c_amd.parts import BLOCKS, PartSpec
    norm = PartSpec.of("rmsnorm", dim=24, eps=1e-6)
    lin = PartSpec.of("lightning", hidden=24, n_heads=2, head_dim=4, v_head_dim=6, decay=(0.9, 0.5), eps=1e-6)
    blk = BLOCKS.build(PartSpec.of("postnorm", hidden=24, mixer=lin, ffn=None, mixer_norm=norm, token_shift=True))
    assert blk.cache_need().state.shape == (2 * 4 * 6 + 24,) and blk.mixer_state == 48
    blk = BLOCKS.build(PartSpec.of("postnorm", hidden=24, mixer=lin, ffn=None, mixer_norm=norm))
    assert blk.cache_need().state.shape == (48,) and "shift.mu" not in blk.tensors() and "mixer_gain" not in blk.tensors()


def test_random_weights_folder_and_plain_reading(tmp_path):
    """The library writes a folder from a configuration alone; the plain implementation reads it and runs."""
    from bitnet_c_amd.config import PafutarConfig, load_config
    from bitnet_c_amd.weights import write_model_folder
    folder = write_model_folder(str(tmp_path / "made"), PafutarConfig.from_dict(CONFIGS["B"]), 5, torch.bfloat16)
    arch, cfg = load_config(folder)
    assert arch.name == "Pafutar" and cfg == PafutarConfig.from_dict(CONFIGS["B"])
    logits = pp.forward(pp.read_config(folder), pp.read_weights(folder), [1, 2, 3, 4])
    assert logits.shape == (4, 77) and bool(torch.isfinite(logits).all())


def test_a_folder_with_a_tensor_missing_or_left_over_is_refused(tmp_path):
    from safetensors.torch import load_file
    from bitnet_c_amd.config import PafutarConfig
    from bitnet_c_amd.config.pafutar import build_pafutar_plan
    from bitnet_c_amd.weights import WeightError, open_tensors, write_file
    folder = write_folder(tmp_path / "m", CONFIGS["A"], 1)
    plan = build_pafutar_plan(PafutarConfig.from_dict(CONFIGS["A"]))
    tensors = load_file(os.path.join(folder, "model.safetensors"))
    tensors["l1.mix.v"] = tensors.pop("l1.mix.g")                   # an attention layer has no value matrix
    tensors["pos"] = tensors["pos"][:-1].contiguous()
    tensors["l2.norm1"] = tensors["l0.norm1"].clone()               # a layer that runs another's weights has no tensors
    write_file(os.path.join(folder, "model.safetensors"), tensors)
    with pytest.raises(WeightError) as err:
        open_tensors(folder, plan.expected_tensors())
    assert err.value.missing == ["l1.mix.g"] and err.value.unexpected == ["l1.mix.v", "l2.norm1"]
    assert [n for n, _, _ in err.value.wrong_shape] == ["pos"]


def test_the_plain_mechanisms_on_cases_worked_by_hand():
    """The oracle itself, where a result can be written down."""
    g = torch.Generator().manual_seed(0)
    # what a position sees
    assert pp.visible(9, dict(size=3, keep_first=2)) == [0, 1, 7, 8, 9]
    assert pp.visible(3, dict(size=3, keep_first=2)) == [0, 1, 2, 3] and pp.visible(4, dict(size=3, keep_first=1)) == [0, 2, 3, 4]
    assert pp.visible(5, dict(size=1, keep_first=0)) == [5] and pp.visible(2, None) == [0, 1, 2]
    assert [pp.head_slope(h, 4) for h in range(4)] == [0.25, 0.0625, 0.015625, 0.00390625]
    assert abs(pp.head_slope(2, 6) - 2.0 ** -4) < 1e-15
    # token shift: the rows mixed in are the inputs; the first token's is zero, or the one handed in
    x = torch.randn(4, 5, generator=g, dtype=F64)
    mu = torch.tensor([0.0, 1.0, 0.5, 0.25, -1.0], dtype=F64)
    y = pp.mix_with_previous(x, mu)
    assert torch.equal(y[:, 0], x[:, 0]) and torch.allclose(y[1:, 1], x[:-1, 1]) and y[0, 1] == 0 and torch.allclose(y[2, 2], (x[1, 2] + x[2, 2]) / 2)
    assert torch.allclose(torch.cat([pp.mix_with_previous(x[:3], mu), pp.mix_with_previous(x[3:], mu, x[2])]), y)
    # the norm behind the sum
    z = pp.add_and_norm(torch.tensor([[3.0, 0.0]], dtype=F64), torch.tensor([[0.0, 2.0]], dtype=F64), 2.0, torch.tensor([1.0, 4.0], dtype=F64),
                        torch.tensor([1.0, 10.0], dtype=F64), 14.0)
    assert torch.allclose(z, torch.tensor([[6.0 / 8.0, 80.0 / 8.0]], dtype=F64))         # mean(36, 64) + 14 = 64
    # attention: equal scores but for the distance give weights 2^-slope...; a key outside the mask carries nothing
    q = torch.zeros(1, 1, 2, dtype=F64)
    k, v = torch.zeros(4, 1, 2, dtype=F64), torch.eye(4, dtype=F64)[:, None, :]
    w = pp.attend(q, k, v, 3, dict(size=2, keep_first=1), 1.0, [1.0], [math.log(2.0)])[0, 0]
    assert torch.allclose(w, torch.tensor([0.125, 0.0, 0.5, 1.0], dtype=F64) / 1.625)
    q[0, 0, 0] = k[0, 0, 0] = 1.0
    w = pp.attend(q, k, v, 3, None, 0.5, [2.0 * math.log(8.0)], [math.log(2.0)])[0, 0]       # the far key's score makes up its distance
    assert torch.allclose(w, torch.tensor([1.0, 0.25, 0.5, 1.0], dtype=F64) / 2.75)
    # a whole mixer: one token sees itself alone, so the result is its key projection (with bias, not normed) gated
    D = 6
    h = torch.randn(5, D, generator=g, dtype=F64)
    W = {"q": torch.randn(4, D, generator=g, dtype=F64), "k": torch.randn(4, D, generator=g, dtype=F64), "g": torch.randn(4, D, generator=g, dtype=F64),
         "o": torch.eye(4, dtype=F64), "q.b": torch.randn(4, generator=g, dtype=F64), "k.b": torch.randn(4, generator=g, dtype=F64),
         "temp": torch.tensor([1.7], dtype=F64)}
    m = dict(heads=1, kv_heads=1, dim=4, vdim=4, scale=0.5, mask=dict(size=3, keep_first=1))
    y, (keys, values) = pp.windowed_attention(h[:1], W, "", m, 1e-6)
    assert torch.allclose(y[0], (h[0] @ W["k"].T + W["k.b"]) * pp.sigmoid(h[0] @ W["g"].T))
    assert torch.allclose(values[0, 0], h[0] @ W["k"].T + W["k.b"]) and abs(float(keys[0, 0].pow(2).mean()) - 1.0) < 1e-4
    whole, _ = pp.windowed_attention(h, W, "", m, 1e-6)
    first, past = pp.windowed_attention(h[:2], W, "", m, 1e-6)
    rest, _ = pp.windowed_attention(h[2:], W, "", m, 1e-6, pos0=2, past=past)
    assert torch.allclose(torch.cat([first, rest]), whole)


def test_plain_layers_carried_over_portions(tmp_path):
    folder = write_folder(tmp_path / "m", CONFIGS["A"], 3)
    c, W = pp.read_config(folder), pp.read_weights(folder)
    toks = torch.randint(0, c["vocab"], (60,), generator=torch.Generator().manual_seed(1)).tolist()
    x = pp.embed(W, toks, 3.0)
    assert torch.allclose(x[7], 3.0 * W["embed"][toks[7]] + W["pos"][7])
    whole, _ = pp.layer_forward(c, W, 0, x)
    parts, carry, at = [], None, 0
    for n in (30, 1, 29):
        y, carry = pp.layer_forward(c, W, 0, x[at:at + n], carry=carry, pos0=at)
        parts.append(y)
        at += n
    assert torch.allclose(torch.cat(parts), whole)
