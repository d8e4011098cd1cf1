"""Configurations and model folders of the Pafutar tests: sizes of this file's own choosing and weights of its own making."""
import json
import math
import os

import torch


def _att(heads, kv, dim, scale, mask, ff, weights_of=None):
    m = dict(heads=heads, kv_heads=kv, dim=dim, vdim=dim, scale=scale)
    if mask:
        m["mask"] = dict(size=mask[0], keep_first=mask[1])
    L = dict(type="attention", mixer=m, mlp=None if ff is None else dict(kind="dense", ff=ff))
    if weights_of is not None:
        L["weights_of"] = weights_of
    return L


# Sizes that differ from layer to layer and between the configurations: windows below, at and above a page, kept first
# tokens fewer and more than the window and than a page, none, no window at all; several kv heads and one, as many kv
# heads as heads; layers without a feed-forward; layers that run another layer's weights, also two of one and a later
# layer's; alpha below, at and above 1.
CONFIGS = {
    "A": dict(architecture="Pafutar", vocab=97, width=64, max_positions=400, norm=dict(eps=1e-5), embedding=dict(scale=3.0),
              postln_alpha=1.3, layers=[
                  _att(4, 2, 16, 0.4, (24, 3), 72),
                  _att(8, 8, 8, 0.6, (70, 5), None),
                  _att(4, 2, 16, 0.4, (24, 3), 72, weights_of=0),
                  _att(6, 2, 12, 0.3, (64, 0), 40),
                  _att(4, 2, 16, 0.4, (24, 3), 72, weights_of=0)]),
    # sizes that fit no kernel's favourite shape: a width that is no multiple of 4, head sizes of 10 and 30, six heads on one
    # kv head, more kept tokens than a page holds, no mask
    "B": dict(architecture="Pafutar", vocab=77, width=50, max_positions=300, norm=dict(eps=1e-6), embedding=dict(scale=1.0),
              postln_alpha=0.8, layers=[
                  _att(2, 2, 30, 0.2, (33, 1), 44, weights_of=3),
                  _att(6, 1, 10, 0.5, (5, 70), 28),
                  _att(3, 3, 14, 0.35, None, 36),
                  _att(2, 2, 30, 0.2, (33, 1), 44)]),
    # the head sizes of real models: the matrix-core attention kernels take every layer
    "C": dict(architecture="Pafutar", vocab=211, width=128, max_positions=1024, norm=dict(eps=1e-6), embedding=dict(scale=0.5),
              postln_alpha=2.5, layers=[
                  _att(4, 2, 64, 0.2, (96, 4), 256),
                  _att(2, 1, 128, 0.15, (31, 33), None),
                  _att(8, 2, 32, 0.3, (64, 130), 136),
                  _att(4, 2, 64, 0.2, (96, 4), 256, weights_of=0),
                  _att(4, 4, 32, 0.25, None, 64)]),
    # ones everywhere: one head, a window of one token with and without a kept one, alpha 1
    "D": dict(architecture="Pafutar", vocab=40, width=32, max_positions=256, norm=dict(eps=1e-5), embedding=dict(scale=1.0),
              postln_alpha=1.0, layers=[
                  _att(1, 1, 8, 1.0, (1, 1), 20),
                  _att(1, 1, 32, 0.35, (1, 0), None),
                  _att(2, 1, 6, 0.5, (2, 1), 1)]),
}


def write_folder(path, cfg, seed, dtype=torch.bfloat16, overrides=None):
    """A model folder with weights of this file's own making: matrices N(0, 1/in), norms and layer scales near 1, biases,
    head temperatures and shifts that matter, position vectors as large as the embedding.  overrides: name -> tensor, put in
    place of what is drawn."""
    from bitnet_c_amd.config import PafutarConfig
    from bitnet_c_amd.config.pafutar import build_pafutar_plan
    from bitnet_c_amd.weights import write_file
    plan = build_pafutar_plan(PafutarConfig.from_dict(cfg))
    g = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, spec in plan.expected_tensors().items():
        shape = tuple(spec.shape)
        if name.endswith(".b"):
            t = 0.5 * torch.randn(shape, generator=g)
        elif name.endswith(".temp"):
            t = 1.0 + 0.5 * torch.rand(shape, generator=g)
        elif name.endswith(".shift"):
            t = torch.rand(shape, generator=g)
        elif len(shape) == 1:
            t = 1.0 + 0.2 * torch.randn(shape, generator=g)
        elif name in ("embed", "pos"):
            t = torch.randn(shape, generator=g)
        else:
            t = torch.randn(shape, generator=g) / math.sqrt(shape[-1])
        tensors[name] = t.to(dtype)
    for name, t in (overrides or {}).items():
        assert tuple(t.shape) == tuple(tensors[name].shape), name
        tensors[name] = t.to(dtype)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_file(os.path.join(path, "model.safetensors"), tensors)
    return str(path)


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(1000 + seed)).tolist()
