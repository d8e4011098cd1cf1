"""Plain, slow implementation of the Zenasun decoder, for tests only.

Whole sequences, no cache, nothing carried between calls, one function per mechanism, CPU tensors in float64.  It shares
no code with the package under test: its own reading of config.json, its own safetensors reading (through the
`safetensors` library), its own greedy loop.  Notation: h is a sublayer's input [T, D]; positions count from 0; linear
weights are [out, in]; the recurrence is written token by token, the way its definition reads.
"""
from __future__ import annotations

import json
import os

import torch

F64 = torch.float64
WEIGHT_FLOOR = 1e-20        # joins the sum of the chosen scores that the experts' weights are divided by


def read_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def read_weights(folder: str) -> dict:
    from safetensors.torch import load_file
    return {k: v.to(F64) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}


# ---- small pieces ----------------------------------------------------------------------------------------------

def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis; eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def shifted_norm(x, w, eps):
    """The norm whose stored weight w means 1 + w."""
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def angles(positions, rot: dict, angle_dtype=F64):
    """[T, dims / 2]: position * base^(-2i/dims).  angle_dtype float32: frequency and angle rounded as an engine that keeps
    them in 32 bits forms them."""
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)], dtype=F64)
    pos = torch.as_tensor(list(positions), dtype=F64)
    return (pos.to(angle_dtype)[:, None] * f.to(angle_dtype)[None, :]).to(F64)


def rotate_halves(x, positions, rot: dict, angle_dtype=F64):
    """x [T, heads, d]: dimension i turns with dimension i + dims / 2; dimensions from dims on pass unchanged."""
    half = rot["dims"] // 2
    a = angles(positions, rot, angle_dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., :half], x[..., half:2 * half]
    out[..., :half] = u * torch.cos(a) - v * torch.sin(a)
    out[..., half:2 * half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def rotate_neighbours(x, positions, rot: dict, angle_dtype=F64):
    """x [T, heads, d]: dimension 2i turns with dimension 2i + 1; dimensions from dims on pass unchanged."""
    dims = rot["dims"]
    a = angles(positions, rot, angle_dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * torch.cos(a) - v * torch.sin(a)
    out[..., 1:dims:2] = v * torch.cos(a) + u * torch.sin(a)
    return out


# ---- mixers ----------------------------------------------------------------------------------------------------

def sink_weights(s, sink):
    """Causal softmax weights of scores s [T, T] (query, key) whose denominators also hold exp(sink)."""
    T = s.shape[0]
    s = s.masked_fill(torch.arange(T)[None, :] > torch.arange(T)[:, None], -float("inf"))
    top = torch.maximum(s.max(dim=1).values, sink)[:, None]
    e = torch.exp(s - top)
    return e / (e.sum(dim=1, keepdim=True) + torch.exp(sink - top))


def latent_attention(h, W, p, m, eps, angle_dtype=F64):
    """Queries through a normed latent; keys and values from a normed latent c of kv_rank numbers per token, plus one
    rotated key part of rot_dim numbers that all heads share and that is not normed.  Head i's query is [dim plain, rot_dim
    rotated]; its score against position j is (q_plain . W_uk,i c_j + q_rot . k_rot,j) * scale; causal softmax with one
    learned sink per head, which is not scaled; values W_uv,i c_j; W_o."""
    T = h.shape[0]
    H, d, r, vd, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = unit_rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]
    q = (cq @ W[p + "uq"].T).reshape(T, H, d + r)
    dkv = h @ W[p + "dkv"].T
    c = unit_rms(dkv[:, :R], eps) * W[p + "dkv.norm"]
    k_rot, q_rot = dkv[:, R:].reshape(T, 1, r), q[..., d:]
    if r:
        rot = dict(base=m["rot"]["base"], dims=r)
        k_rot = rotate_neighbours(k_rot, range(T), rot, angle_dtype)
        q_rot = rotate_neighbours(q_rot, range(T), rot, angle_dtype)
    k = (c @ W[p + "uk"].T).reshape(T, H, d)
    v = (c @ W[p + "uv"].T).reshape(T, H, vd)
    out = torch.zeros((T, H, vd), dtype=F64)
    for i in range(H):
        s = (q[:, i, :d] @ k[:, i].T + q_rot[:, i] @ k_rot[:, 0].T) * m["scale"]
        out[:, i] = sink_weights(s, W[p + "sink"][i]) @ v[:, i]
    return out.reshape(T, H * vd) @ W[p + "o"].T


def decayed_sums(q, k, v, decay, state=None):
    """q, k [T, H, d], v [T, H, vd], decay [H]: token by token S <- decay S + k v^T, o = S^T q.  Returns (o, the state
    after the last token [H, d, vd])."""
    T, H, d = q.shape
    S = torch.zeros((H, d, v.shape[-1]), dtype=F64) if state is None else state.clone()
    o = torch.zeros((T, H, v.shape[-1]), dtype=F64)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return o, S


def retention(h, W, p, m, eps, angle_dtype=F64):
    """q, k [heads, dim] rotated by position, k then divided by sqrt(dim), v [heads, vdim], all straight from their
    projections; decayed sums from a state of zeros; every head's output divided by its own root mean square (no weight);
    heads side by side times silu(W_g h); W_o."""
    T = h.shape[0]
    H, d, vd = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).reshape(T, H, d)
    k = (h @ W[p + "k"].T).reshape(T, H, d)
    v = (h @ W[p + "v"].T).reshape(T, H, vd)
    if m.get("rot"):
        q, k = rotate_halves(q, range(T), m["rot"], angle_dtype), rotate_halves(k, range(T), m["rot"], angle_dtype)
    o, _ = decayed_sums(q, k * d ** -0.5, v, torch.tensor([float(x) for x in m["decay"]], dtype=F64))
    return (unit_rms(o, eps).reshape(T, H * vd) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


# ---- feed-forward ----------------------------------------------------------------------------------------------

def group_limited_choice(c, groups, top):
    """c [E] choice scores -> (the `top` chosen experts in descending order, the groups left in, all groups' scores).  The
    experts fall into groups.count runs of neighbours; a group scores its largest member; experts outside the groups.keep
    best groups cannot be chosen."""
    E = c.shape[0]
    size = E // groups["count"]
    best = torch.stack([c[g * size:(g + 1) * size].max() for g in range(groups["count"])])
    kept = torch.argsort(best, descending=True, stable=True)[:groups["keep"]].tolist()
    masked = torch.full_like(c, -float("inf"))
    for g in kept:
        masked[g * size:(g + 1) * size] = c[g * size:(g + 1) * size]
    return torch.argsort(masked, descending=True, stable=True)[:top], kept, best, masked


def route(h, W, p, mlp, margins=None):
    """(chosen [T, top], weights [T, top]).  Scores: the softmax of the router's logits over the experts and the identity
    experts behind them; choice by score + correction inside the best groups; weights: the plain scores of the chosen over
    their sum.  margins: a list that receives, per token, how far the decisions are from falling the other way (the last
    group kept against the first left out, the last expert chosen against the first left out), in units of what a small
    relative change of the logits does to a score (score times the logits' root mean square): a small number is a close
    call."""
    r = mlp["router"]
    z = h @ W[p + "router"].T
    e = torch.exp(z - z.max(dim=-1, keepdim=True).values)
    s = e / e.sum(dim=-1, keepdim=True)
    c = s + W[p + "correction"]
    E = z.shape[1]
    groups = r.get("groups") or dict(count=1, keep=1)
    size, chosen, low = E // groups["count"], [], []
    for t in range(h.shape[0]):
        pick, kept, best, masked = group_limited_choice(c[t], groups, r["top"])
        chosen.append(pick)
        if margins is None:
            continue
        rz = float(z[t].pow(2).mean().sqrt())
        gap = float("inf")

        def call(a, b):                                       # experts a (in) and b (out)
            return float(c[t, a] - c[t, b]) / max(float(torch.maximum(s[t, a], s[t, b])) * rz, 1e-300)
        if groups["keep"] < groups["count"]:
            order = torch.argsort(best, descending=True, stable=True).tolist()
            a, b = order[groups["keep"] - 1], order[groups["keep"]]
            gap = min(gap, call(int(c[t, a * size:(a + 1) * size].argmax()) + a * size,
                                int(c[t, b * size:(b + 1) * size].argmax()) + b * size))
        rest = masked.clone()
        rest[pick] = -float("inf")
        if float(rest.max()) > -float("inf"):
            gap = min(gap, call(int(pick[-1]), int(rest.argmax())))
        low.append(gap)
    if margins is not None:
        margins.append(torch.tensor(low, dtype=F64))
    chosen = torch.stack(chosen)
    w = torch.gather(s, 1, chosen)
    return chosen, w / (w.sum(dim=-1, keepdim=True) + WEIGHT_FLOOR)


def expert(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def moe_ff(h, W, p, mlp, margins=None):
    """The weighted sum of the chosen experts; an identity expert hands its input on."""
    chosen, w = route(h, W, p, mlp, margins)
    n = mlp["router"]["experts"]
    out = torch.zeros_like(h)
    for e in range(n + (mlp["router"].get("identity") or 0)):
        rows = torch.nonzero((chosen == e).any(dim=-1))[:, 0]
        if rows.numel():
            share = (w[rows] * (chosen[rows] == e)).sum(dim=-1, keepdim=True)
            out[rows] += share * (expert(h[rows], W, f"{p}e{e}.") if e < n else h[rows])
    return out


# ---- the model -------------------------------------------------------------------------------------------------

def layer_forward(c, W, i, x, angle_dtype=F64, round_to=None, margins=None):
    """x <- x + (mixer(norm1(x)) + ff(norm2(x))), both halves of the same x.  A layer that names another under weights_of
    runs that layer's tensors."""
    L, eps = c["layers"][i], c["norm"]["eps"]
    src = L.get("weights_of")
    p = f"l{i if src is None else src}."
    rd = (lambda t: t.to(round_to).to(F64)) if round_to is not None else (lambda t: t)
    h = rd(shifted_norm(x, W[p + "norm1"], eps))
    if L["type"] == "latent_attention":
        y = latent_attention(h, W, p + "mix.", L["mixer"], eps, angle_dtype)
    elif L["type"] == "retention":
        y = retention(h, W, p + "mix.", L["mixer"], eps, angle_dtype)
    else:
        raise ValueError(f"unknown mixer {L['type']!r}")
    if L.get("mlp") is not None:
        y = y + moe_ff(rd(shifted_norm(x, W[p + "norm2"], eps)), W, p + "mlp.", L["mlp"], margins)
    return x + y


def forward(c: dict, W: dict, tokens, layers_out=None, angle_dtype=F64, round_to=None, margins=None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  round_to: a norm's output is rounded to this type where a sublayer reads
    it; layers_out: a list that receives the stream after every layer; margins: a list that receives, per token, the
    smallest routing margin over all layers (see route)."""
    x = W["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] * c["embedding"]["scale"]
    per_layer = [] if margins is not None else None
    for i in range(len(c["layers"])):
        x = layer_forward(c, W, i, x, angle_dtype, round_to, per_layer)
        if layers_out is not None:
            layers_out.append(x.clone())
    if margins is not None:
        low = torch.stack(per_layer).min(dim=0).values if per_layer else torch.full((len(tokens),), float("inf"), dtype=F64)
        margins.extend(low.tolist())
    logits = shifted_norm(x, W["final.norm"], c["norm"]["eps"]) @ W["embed"].T
    cap = c["logit_softcap"]
    return cap * torch.tanh(logits / cap)


def generate(c: dict, W: dict, prompt, n_new: int):
    """Greedy continuation, the whole sequence run again for every token."""
    seq = list(prompt)
    for _ in range(n_new):
        seq.append(int(forward(c, W, seq)[-1].argmax()))
    return seq[len(prompt):]
