"""Configurations and model folders of the Zenasun tests: sizes of this file's own choosing and weights of its own making."""
import json
import math
import os

import torch


def _decays(heads, slowest=0.999):
    """One decay per head, from a fast one to a slow one."""
    return [round(math.exp(-0.5 / (3.0 ** i)), 12) if i < heads - 1 else slowest for i in range(heads)]


def _ret(heads, dim, vdim, rot, mlp, decay=None, weights_of=None):
    m = dict(heads=heads, dim=dim, vdim=vdim, decay=decay or _decays(heads))
    if rot:
        m["rot"] = dict(base=rot[0], dims=rot[1])
    L = dict(type="retention", mixer=m, mlp=mlp)
    if weights_of is not None:
        L["weights_of"] = weights_of
    return L


def _lat(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, base, mlp, weights_of=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale)
    if rot_dim:
        m["rot"] = dict(base=base, dims=rot_dim)
    L = dict(type="latent_attention", mixer=m, mlp=mlp)
    if weights_of is not None:
        L["weights_of"] = weights_of
    return L


def _moe(experts, identity, top, ff, count=1, keep=1):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, identity=identity, top=top, groups=dict(count=count, keep=keep)))


def _model(vocab, width, eps, scale, cap, layers):
    return dict(architecture="Zenasun", vocab=vocab, width=width, norm=dict(eps=eps), embedding=dict(scale=scale), logit_softcap=cap,
                layers=layers)


# Sizes that differ from layer to layer and between the configurations: key and value widths that differ, value widths of
# more than one column block of the recurrence's kernel, rotations over part of a head, over the whole head and none, no
# rotated part beside a latent, layers that run another layer's weights (both kinds of mixers, once and twice, also a
# later layer's), either kind of mixer first and last, layers without a feed-forward; groups of one expert and one group of
# all, every group kept and a single one, no identity expert, one, and more than there are experts, all experts per token.
CONFIGS = {
    "A": _model(97, 64, 1e-5, 3.0, 12.0, [
        _ret(3, 16, 24, (500.0, 8), _moe(5, 1, 2, 32, 3, 2)),
        _lat(4, 12, 8, 20, 40, 24, 0.25, 10000.0, _moe(7, 2, 3, 24, 3, 2)),
        _ret(3, 16, 24, (500.0, 8), _moe(5, 1, 2, 32, 3, 2), weights_of=0),
        _lat(2, 16, 4, 16, 24, 32, 0.3, 100.0, None),
        _lat(4, 12, 8, 20, 40, 24, 0.25, 10000.0, _moe(7, 2, 3, 24, 3, 2), weights_of=1),
        _lat(4, 12, 8, 20, 40, 24, 0.25, 10000.0, _moe(7, 2, 3, 24, 3, 2), weights_of=1)]),
    # sizes that fit no kernel's favourite shape: a width that is no multiple of 8, value heads of 70 (two column blocks),
    # heads of 10 and 40, latents of 14 and 9, experts of 12
    "B": _model(77, 50, 1e-6, 1.5, 40.0, [
        _lat(3, 6, 2, 10, 14, 9, 0.5, 50.0, _moe(3, 0, 3, 12)),
        _ret(2, 10, 70, (100.0, 10), None),
        _ret(1, 40, 12, None, _moe(2, 4, 4, 20, 3, 2)),
        _lat(2, 9, 0, 7, 10, 5, 0.3, None, _moe(4, 1, 1, 16, 5, 2))]),
    # the head sizes of real models: the matrix-core kernels take every layer (key rows of 128, and of 144 stored as 160)
    "C": _model(211, 128, 1e-6, 6.0, 25.0, [
        _ret(2, 64, 64, (10000.0, 64), _moe(12, 4, 3, 64, 4, 2)),
        _lat(4, 32, 32, 32, 96, 48, 0.12, 100000.0, _moe(6, 2, 2, 64, 2, 1)),
        _ret(1, 128, 128, (10000.0, 96), None),
        _lat(3, 64, 24, 64, 120, 64, 0.11, 200000.0, _moe(28, 4, 4, 32, 8, 3)),
        _ret(2, 64, 64, (10000.0, 64), _moe(12, 4, 3, 64, 4, 2), weights_of=0)]),
    # ones everywhere: one head, one expert beside one identity expert, a decay of exactly 1 (nothing fades) and 0
    # (nothing is kept), the first layer runs the last one's weights
    "D": _model(40, 32, 1e-5, 1.0, 3.0, [
        _ret(2, 6, 10, (30.0, 2), _moe(1, 0, 1, 20), decay=[0.0, 0.5], weights_of=3),
        _lat(1, 8, 2, 8, 8, 4, 0.35, 10.0, _moe(1, 1, 1, 8, 2, 1)),
        _ret(1, 8, 8, (100.0, 8), _moe(2, 1, 2, 4, 3, 3), decay=[1.0]),
        _ret(2, 6, 10, (30.0, 2), _moe(1, 0, 1, 20), decay=[0.0, 0.5])]),
    # no latent layer at all (a cache without pages), a head as wide as the kernel takes, more heads than experts
    "E": _model(50, 40, 1e-5, 2.0, 8.0, [
        _ret(1, 256, 6, (10.0, 200), _moe(3, 1, 2, 16, 2, 2)),
        _ret(9, 4, 4, (1000.0, 4), _moe(3, 3, 1, 8, 2, 1))]),
}


def write_folder(path, cfg, seed, dtype=torch.bfloat16, overrides=None):
    """A model folder with weights of this file's own making: matrices N(0, 1/in) (those of the experts larger), the block
    norms' stored weights near 0 and the latents' near 1, sinks of either sign, router rows three times larger, corrections
    that change some choices and push many choice scores below 0, the embedding N(0, 1) / 4.  overrides: name -> tensor."""
    from bitnet_c_amd.config import ZenasunConfig
    from bitnet_c_amd.config.zenasun import build_zenasun_plan
    from bitnet_c_amd.weights import write_file
    plan = build_zenasun_plan(ZenasunConfig.from_dict(cfg))
    g = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, spec in plan.expected_tensors().items():
        shape = tuple(spec.shape)
        r = torch.randn(shape, generator=g)
        if name.endswith(".correction"):
            t = 0.15 * r - 0.15
        elif name.endswith(".sink"):
            t = r
        elif name.endswith(("dq.norm", "dkv.norm")):
            t = 1.0 + 0.2 * r
        elif len(shape) == 1:
            t = 0.2 * r
        elif name == "embed":
            t = 0.25 * r
        elif name.endswith(".router"):
            t = 3.0 * r / math.sqrt(shape[-1])
        elif ".mlp.e" in name:
            t = 1.5 * r / math.sqrt(shape[-1])
        else:
            t = r / math.sqrt(shape[-1])
        tensors[name] = t.to(dtype)
    for name, t in (overrides or {}).items():
        assert tuple(t.shape) == tuple(tensors[name].shape), name
        tensors[name] = t.to(dtype)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_file(os.path.join(path, "model.safetensors"), tensors)
    return str(path)


_settled = {}


def settled_tokens(folder, n, seed, margin=0.05):
    """n token ids for which no expert choice and no choice of groups of the model in `folder` is a close call: built from
    left to right, a few tokens at a time; whatever follows the first token whose smallest routing margin (plain
    implementation, float64) is below `margin` is drawn again.  Routing is causal, so a sequence's beginning stays settled
    however it goes on, and one sequence per (folder, seed) serves every length."""
    import plain_zenasun as pz
    key = (folder, seed)
    if key not in _settled:
        _settled[key] = ([], torch.Generator().manual_seed(seed))
    toks, g = _settled[key]
    if len(toks) < n:
        cfg, W = pz.read_config(folder), pz.read_weights(folder)
        tries = 0
        while len(toks) < n:
            tries += 1
            assert tries < 100 * n, "no sequence without a close expert choice was found"
            more = torch.randint(0, cfg["vocab"], (min(16, n - len(toks)),), generator=g).tolist()
            margins = []
            pz.forward(cfg, W, toks + more, margins=margins)
            good = 0
            while good < len(more) and margins[len(toks) + good] >= margin:
                good += 1
            toks += more[:good]
    return list(toks[:n])
