"""Zenasun's configuration, plan, cache needs and model folder, and the plain implementation on cases worked by hand: what
runs without a GPU."""
import copy
import math
import os

import pytest
import torch

import plain_zenasun as pz
from zenasun_cases import CONFIGS, settled_tokens, write_folder

F64 = torch.float64


def test_configuration_round_trip_and_plan():
    from bitnet_c_amd.config import ZenasunConfig, architecture_for
    from bitnet_c_amd.config.zenasun import build_zenasun_plan
    for raw in CONFIGS.values():
        assert architecture_for(raw).name == "Zenasun"
        c = ZenasunConfig.from_dict(raw)
        assert ZenasunConfig.from_dict(c.to_dict()) == c and c.to_dict()["layers"] == raw["layers"]
        plan = build_zenasun_plan(c)
        own = [i for i, L in enumerate(raw["layers"]) if "weights_of" not in L]
        assert len(plan.layers) == len(own) and len(plan.schedule) == len(raw["layers"])
        assert plan.embedding_multiplier == raw["embedding"]["scale"] and plan.logit_softcap == raw["logit_softcap"]
        D = raw["width"]
        t = plan.expected_tensors()
        assert t["embed"].shape == (raw["vocab"], D) and t["final.norm"].shape == (D,) and "head" not in t
        for i, (e, L) in enumerate(zip(plan.schedule, raw["layers"])):
            assert e.layer == own.index(L.get("weights_of", i)) and e.kv_from is None
            p, m = f"l{i}.", L["mixer"]
            if "weights_of" in L:
                assert not [n for n in t if n.startswith(p)]
                continue
            assert t[p + "norm1"].shape == (D,)
            H = m["heads"]
            if L["type"] == "retention":
                want = {"q": (H * m["dim"], D), "k": (H * m["dim"], D), "v": (H * m["vdim"], D), "g": (H * m["vdim"], D),
                        "o": (D, H * m["vdim"])}
            else:
                R, qr = m["kv_rank"], m["q_rank"]
                want = {"dq": (qr, D), "dq.norm": (qr,), "uq": (H * (m["dim"] + m["rot_dim"]), qr), "dkv": (R + m["rot_dim"], D),
                        "dkv.norm": (R,), "uk": (H * m["dim"], R), "uv": (H * m["vdim"], R), "sink": (H,), "o": (D, H * m["vdim"])}
            assert {n[len(p) + 4:]: s.shape for n, s in t.items() if n.startswith(p + "mix.")} == want
            mlp = L["mlp"]
            assert (p + "norm2" in t) == (mlp is not None)
            if mlp is None:
                assert not [n for n in t if n.startswith(p + "mlp.")]
                continue
            E, I, F = mlp["router"]["experts"], mlp["router"]["identity"], mlp["expert"]["ff"]
            want = {"router": (E + I, D), "correction": (E + I,)}
            for x in range(E):
                want.update({f"e{x}.gate": (F, D), f"e{x}.up": (F, D), f"e{x}.down": (D, F)})
            assert {n[len(p) + 4:]: s.shape for n, s in t.items() if n.startswith(p + "mlp.")} == want


def test_keys_that_may_be_left_out():
    from bitnet_c_amd.config import ZenasunConfig
    raw = copy.deepcopy(CONFIGS["B"])
    raw["layers"][0]["mlp"]["router"].pop("groups")
    raw["layers"][0]["mlp"]["router"].pop("identity")
    assert ZenasunConfig.from_dict(raw) == ZenasunConfig.from_dict(CONFIGS["B"])
    raw["layers"][0]["mlp"]["router"].update(groups=None, identity=None)
    assert ZenasunConfig.from_dict(raw) == ZenasunConfig.from_dict(CONFIGS["B"])


def _bad(raw, change, match):
    from bitnet_c_amd.config import ConfigError, ZenasunConfig
    raw = copy.deepcopy(raw)
    change(raw)
    with pytest.raises(ConfigError, match=match):
        ZenasunConfig.from_dict(raw)


def test_configurations_that_cannot_be_are_refused():
    A = CONFIGS["A"]
    _bad(A, lambda r: r["layers"][0].update(type="conv"), "type")
    _bad(A, lambda r: r["layers"][0]["mixer"].update(decay=[0.5]), "decay")
    _bad(A, lambda r: r["layers"][0]["mixer"].update(decay=[0.5, 0.5, 1.5]), "decay")
    _bad(A, lambda r: r["layers"][0]["mixer"]["rot"].update(dims=18), "rot")
    _bad(A, lambda r: r["layers"][0]["mixer"]["rot"].update(dims=5), "rot")
    _bad(A, lambda r: r["layers"][1]["mixer"].update(rot_dim=7), "rot_dim")
    _bad(A, lambda r: r["layers"][1]["mixer"]["rot"].update(dims=4), "rot")
    _bad(A, lambda r: r["layers"][1]["mixer"].pop("rot"), "rot")
    _bad(A, lambda r: r["layers"][1]["mixer"].pop("scale"), "scale")
    _bad(A, lambda r: r["layers"][1]["mixer"].pop("q_rank"), "q_rank")
    _bad(A, lambda r: r["layers"][0]["mlp"].update(kind="dense"), "kind")
    _bad(A, lambda r: r["layers"][0]["mlp"]["router"].update(top=5), "top")
    _bad(A, lambda r: r["layers"][0]["mlp"]["router"].update(identity=-1), "identity")
    _bad(A, lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(count=4), "groups")
    _bad(A, lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "groups")
    _bad(A, lambda r: r["layers"][2].update(weights_of=2), "weights_of")
    _bad(A, lambda r: r["layers"][2].update(weights_of=1), "differs")
    _bad(A, lambda r: r["layers"][5].update(weights_of=4), "none of its own|differs")
    _bad(A, lambda r: r.pop("norm"), "norm")
    _bad(A, lambda r: r.update(logit_softcap=-1.0), "logit_softcap")
    _bad(A, lambda r: r.update(layers=[]), "layers")


def test_cache_needs_states_pages_and_shared_weights():
    """A retention layer keeps a float32 matrix per head and no pages, a latent layer one row per position; layers that run
    one layer's weights have a state or pages each."""
    from bitnet_c_amd.cache import PAGE, PagedCache
    from bitnet_c_amd.config import ZenasunConfig
    from bitnet_c_amd.config.zenasun import build_zenasun_plan
    from bitnet_c_amd.parts import BLOCKS
    raw = CONFIGS["A"]
    plan = build_zenasun_plan(ZenasunConfig.from_dict(raw))
    needs = [BLOCKS.build(plan.layers[e.layer].block).cache_need() for e in plan.schedule]
    for need, L in zip(needs, raw["layers"]):
        m = L["mixer"]
        if L["type"] == "retention":
            assert need.kv is None and need.state.shape == (m["heads"] * m["dim"] * m["vdim"],)
            assert need.state.dtype == torch.float32 and need.state.device_addressed
        else:
            assert need.state is None and need.kv.n_kv_heads == 1 and need.kv.window == 0
            assert need.kv.head_dim >= m["kv_rank"] + m["rot_dim"] and need.kv.v_dim >= m["kv_rank"]
    cache = PagedCache(needs, [e.kv_from for e in plan.schedule], 16 * PAGE)
    assert cache.group_of(1) == cache.group_of(4) == cache.group_of(5) != cache.group_of(3) and cache.group_of(0) is None
    assert sorted(cache._state_needs) == [0, 2]
    s = cache.alloc_slot()
    cache.reserve([s], [3 * PAGE + 1])
    cache.commit([s], [3 * PAGE + 1])
    assert [len(cache.pages_of(g, s)) for g in range(2)] == [4, 4]
    cache.free_slot(s)
    cache.check()


def test_stored_rows_of_a_latent():
    """Sizes that the matrix-core kernels take stay; sizes a little below one of theirs are filled up, both rows or none;
    the rest are the vector kernel's as they are."""
    from bitnet_c_amd import ops
    assert ops.latent_row_widths(192, 64) == (256, 192) and ops.latent_row_widths(96, 32) == (128, 96)
    assert ops.latent_row_widths(120, 24) == (160, 128) and ops.latent_row_widths(160, 32) == (192, 192)
    assert ops.latent_row_widths(80, 16) == (96, 96) and ops.latent_row_widths(14, 2) == (16, 14)
    assert ops.latent_row_widths(512, 64) == (576, 512) and ops.latent_row_widths(40, 8) == (48, 40)
    for rank in range(2, 513, 2):
        for rot in (0, 2, 16, 32, 64):
            kw, vw = ops.latent_row_widths(rank, rot)
            assert rank + rot <= kw <= (rank + rot) * 1.25 and rank <= vw <= rank * 1.25
            assert (kw, vw) == (rank + rot, rank) or ops.attention_general_supported(torch.bfloat16, kw, vw)


def test_random_weights_folder_and_plain_reading(tmp_path):
    """The library writes a folder from a configuration alone; the plain implementation reads it and runs."""
    from bitnet_c_amd.config import ZenasunConfig, load_config
    from bitnet_c_amd.weights import write_model_folder
    folder = write_model_folder(str(tmp_path / "made"), ZenasunConfig.from_dict(CONFIGS["B"]), 5, torch.bfloat16)
    arch, cfg = load_config(folder)
    assert arch.name == "Zenasun" and cfg == ZenasunConfig.from_dict(CONFIGS["B"])
    W = pz.read_weights(folder)
    assert float(W["l0.norm1"].abs().max()) == 0.0 and float(W["l0.mix.dq.norm"].min()) == 1.0      # both mean a weight of 1
    logits = pz.forward(pz.read_config(folder), W, [1, 2, 3, 4])
    assert logits.shape == (4, 77) and bool(torch.isfinite(logits).all())


def test_a_folder_with_a_tensor_missing_or_left_over_is_refused(tmp_path):
    from safetensors.torch import load_file
    from bitnet_c_amd.config import ZenasunConfig
    from bitnet_c_amd.config.zenasun import build_zenasun_plan
    from bitnet_c_amd.weights import WeightError, open_tensors, write_file
    folder = write_folder(tmp_path / "m", CONFIGS["A"], 1)
    plan = build_zenasun_plan(ZenasunConfig.from_dict(CONFIGS["A"]))
    tensors = load_file(os.path.join(folder, "model.safetensors"))
    tensors["l0.mlp.e5.gate"] = tensors["l0.mlp.e0.gate"].clone()    # an identity expert has no tensors
    tensors["head"] = tensors["embed"].clone()                      # the embedding is the output matrix
    tensors["l2.norm1"] = tensors["l0.norm1"].clone()               # a layer that runs another's weights has no tensors
    tensors["l0.mlp.router"] = tensors["l0.mlp.router"][:-1].contiguous()
    tensors.pop("l1.mix.sink")
    write_file(os.path.join(folder, "model.safetensors"), tensors)
    with pytest.raises(WeightError) as err:
        open_tensors(folder, plan.expected_tensors())
    assert err.value.missing == ["l1.mix.sink"] and sorted(err.value.unexpected) == ["head", "l0.mlp.e5.gate", "l2.norm1"]
    assert [n for n, _, _ in err.value.wrong_shape] == ["l0.mlp.router"]


def test_the_plain_mechanisms_on_cases_worked_by_hand():
    """The oracle itself, where a result can be written down."""
    g = torch.Generator().manual_seed(0)
    T, D = 6, 8
    h = torch.randn(T, D, generator=g, dtype=F64)
    # rotations: position 0 changes nothing, dimensions beyond rot.dims pass, the pairs are the layout's
    x = torch.randn(3, 2, 6, generator=g, dtype=F64)
    for turn, (a, b) in ((pz.rotate_halves, (0, 2)), (pz.rotate_neighbours, (0, 1))):
        r = turn(x, [0, 3, 11], dict(base=100.0, dims=4))
        assert torch.equal(r[0], x[0]) and torch.equal(r[..., 4:], x[..., 4:])
        assert torch.allclose(r[1, 0, a], x[1, 0, a] * math.cos(3.0) - x[1, 0, b] * math.sin(3.0))
        assert torch.allclose(r[1, 0, b], x[1, 0, b] * math.cos(3.0) + x[1, 0, a] * math.sin(3.0))
        assert torch.allclose(r[1, 0, 3], x[1, 0, 3] * math.cos(0.3) + x[1, 0, 1 if a + b == 2 else 2] * math.sin(0.3))
    # the norm around zero: a stored weight of 0 is the plain unit norm
    assert torch.equal(pz.shifted_norm(h, torch.zeros(D, dtype=F64), 1e-3), pz.unit_rms(h, 1e-3))
    # the sink: one token sees itself with weight e^s / (e^s + e^sink)
    w = pz.sink_weights(torch.tensor([[0.3, 9.0], [0.1, 0.2]], dtype=F64), torch.tensor(0.5, dtype=F64))
    assert abs(float(w[0, 0]) - math.exp(0.3) / (math.exp(0.3) + math.exp(0.5))) < 1e-12 and float(w[0, 1]) == 0.0
    assert abs(float(w[1].sum()) - (math.exp(0.1) + math.exp(0.2)) / (math.exp(0.1) + math.exp(0.2) + math.exp(0.5))) < 1e-12
    # latent attention without a rotated part and with a sink far below: the value of the first token is its own
    m = dict(heads=1, dim=3, rot_dim=0, vdim=4, kv_rank=5, q_rank=2, scale=0.7)
    W = {n: torch.randn(s, generator=g, dtype=F64) for n, s in (("dq", (2, D)), ("uq", (3, 2)), ("dkv", (5, D)), ("uk", (3, 5)), ("uv", (4, 5)))}
    W.update({"dq.norm": torch.ones(2, dtype=F64), "dkv.norm": torch.ones(5, dtype=F64), "sink": torch.tensor([-1e3], dtype=F64),
              "o": torch.eye(4, dtype=F64)})
    y = pz.latent_attention(h, W, "", m, 1e-6)
    assert torch.allclose(y[0], W["uv"] @ pz.unit_rms(W["dkv"] @ h[0], 1e-6))
    # decayed sums: decay 0 keeps the current token alone, decay 1 sums everything
    q, k, v = (torch.randn(T, 2, 3, generator=g, dtype=F64), torch.randn(T, 2, 3, generator=g, dtype=F64),
               torch.randn(T, 2, 5, generator=g, dtype=F64))
    o, S = pz.decayed_sums(q, k, v, torch.tensor([0.0, 1.0], dtype=F64))
    assert torch.allclose(o[:, 0], (q[:, 0] * k[:, 0]).sum(-1, keepdim=True) * v[:, 0])
    assert torch.allclose(o[:, 1], torch.tril(q[:, 1] @ k[:, 1].T) @ v[:, 1]) and torch.allclose(S[1], k[:, 1].T @ v[:, 1])
    # groups: the best member ranks a group; choice scores below 0 inside a kept group come before any of a group left out
    c = torch.tensor([-0.9, -0.1, -0.2, -0.3, -0.15, -0.8], dtype=F64)
    pick, kept, best, _ = pz.group_limited_choice(c, dict(count=3, keep=2), 3)
    assert sorted(kept) == [0, 2] and pick.tolist() == [1, 4, 5] and best.tolist() == [-0.1, -0.2, -0.15]
    pick, kept, _, _ = pz.group_limited_choice(c, dict(count=2, keep=1), 2)
    assert kept == [0] and pick.tolist() == [1, 2]
    # the weights: plain scores over their sum; an identity expert hands its input on
    Wr = {"router": torch.tensor([[1.0], [0.9], [-1.0]], dtype=F64), "correction": torch.tensor([0.0, 0.0, 5.0], dtype=F64),
          "e0.gate": torch.tensor([[2.0]], dtype=F64), "e0.up": torch.tensor([[3.0]], dtype=F64), "e0.down": torch.tensor([[0.5]], dtype=F64)}
    mlp = dict(router=dict(experts=2, identity=1, top=2, groups=dict(count=1, keep=1)))
    chosen, w = pz.route(torch.ones(1, 1, dtype=F64), Wr, "", mlp)
    sc = torch.softmax(torch.tensor([1.0, 0.9, -1.0], dtype=F64), 0)
    assert chosen[0].tolist() == [2, 0] and torch.allclose(w[0], sc[[2, 0]] / (sc[0] + sc[2]))
    y = pz.moe_ff(torch.ones(1, 1, dtype=F64), Wr, "", mlp)
    unit = 2.0 / (1.0 + math.exp(-2.0)) * 3.0 * 0.5
    assert abs(float(y) - float(w[0, 0] * 1.0 + w[0, 1] * unit)) < 1e-12


def test_settled_sequences_have_no_close_expert_choice(tmp_path):
    folder = write_folder(tmp_path / "m", CONFIGS["A"], 2)
    toks = settled_tokens(folder, 40, 4)
    assert settled_tokens(folder, 30, 4) == toks[:30]
    margins = []
    pz.forward(pz.read_config(folder), pz.read_weights(folder), toks, margins=margins)
    assert len(margins) == 40 and min(margins) >= 0.05
