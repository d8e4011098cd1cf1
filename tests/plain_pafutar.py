"""Plain, slow implementation of the Pafutar decoder, for tests only.

Whole sequences, no cache, nothing carried between calls unless a caller asks for it, one function per mechanism, CPU
tensors in float64.  It shares no code with the package under test: its own reading of config.json, its own safetensors
reading (through the `safetensors` library), its own greedy loop.  Notation: x is the residual stream [T, D], h a
sublayer's input; positions count from 0; linear weights are [out, in]; attention is written query by query and head by
head, the way its definition reads.
"""
from __future__ import annotations

import json
import os

import torch

F64 = torch.float64


def read_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def read_weights(folder: str) -> dict:
    from safetensors.torch import load_file
    return {k: v.to(F64) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}


# ---- small pieces ----------------------------------------------------------------------------------------------

def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis; eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def embed(W, tokens, scale: float, pos0: int = 0):
    """The embedding's rows times a constant, plus the learned vector of each position (which is not scaled)."""
    ids = torch.as_tensor(list(tokens), dtype=torch.long)
    return W["embed"][ids] * scale + W["pos"][pos0:pos0 + len(ids)]


def mix_with_previous(h, mu, before=None):
    """h_t + (h_{t-1} - h_t) * mu, element by element; before: the row in front of the first (None: zeros, a sequence's
    beginning).  The rows mixed in are the inputs as they were, not their mixtures."""
    first = torch.zeros_like(h[:1]) if before is None else before.reshape(1, -1)
    prev = torch.cat([first, h[:-1]])
    return h + (prev - h) * mu


def add_and_norm(x, y, alpha: float, gain, weight, eps: float):
    """The sum of the stream times alpha and a sublayer's result times its own weights, under an RMS norm: the norm's
    output is the stream from here on."""
    return unit_rms(alpha * x + gain * y, eps) * weight


# ---- attention -------------------------------------------------------------------------------------------------

def head_slope(head: int, heads: int) -> float:
    return 2.0 ** (-8.0 * (head + 1) / heads)


def visible(i: int, mask) -> list:
    """The key positions that position i sees: the last `size` positions, itself included, and a sequence's first
    `keep_first` positions however far back they are; without a mask every position up to i."""
    if not mask:
        return list(range(i + 1))
    size, kept = mask["size"], mask.get("keep_first", 0)
    return [j for j in range(i + 1) if i - j < size or j < kept]


def attend(q, k, v, pos0: int, mask, scale: float, temp, slopes) -> torch.Tensor:
    """q [T, H, d] of the positions pos0 .. pos0 + T - 1 over k, v [P, G, *] of the positions 0 .. P - 1: the score of query
    i and key j is (q . k) * scale * temp[head] - slope[head] * (i - j), the softmax runs over the keys that the mask
    leaves.  Returns [T, H, width of v]."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros((T, H, v.shape[-1]), dtype=F64)
    for t in range(T):
        i = pos0 + t
        js = torch.tensor(visible(i, mask))
        far = (i - js).to(F64)
        for hd in range(H):
            g = hd // (H // G)
            s = (k[js, g] @ q[t, hd]) * scale * temp[hd] - slopes[hd] * far
            e = torch.exp(s - s.max())
            out[t, hd] = (e / e.sum()) @ v[js, g]
    return out


def windowed_attention(h, W, p, m, eps, pos0: int = 0, past=None, round_to=None):
    """Grouped-query attention whose values are its key projections (bias included, before the key's norm).  Every query
    and key head is divided by its own root mean square, no weight; attend(); the heads' outputs side by side are multiplied
    by sigmoid(W_g h); then W_o.  past: (keys [P, G, d], values [P, G, d]) of earlier positions.  Returns (output [T, D],
    (keys, values) of all positions so far).  round_to: queries, keys, values and the gated outputs are rounded to this type
    where an engine of that type stores them."""
    rd = (lambda t: t.to(round_to).to(F64)) if round_to is not None else (lambda t: t)
    T = h.shape[0]
    H, G, d = m["heads"], m.get("kv_heads", m["heads"]), m["dim"]
    q = (h @ W[p + "q"].T + W[p + "q.b"]).reshape(T, H, d)
    v = rd((h @ W[p + "k"].T + W[p + "k.b"]).reshape(T, G, d))
    k = rd(unit_rms(v, eps))
    q = rd(unit_rms(q, eps))
    if past is not None:
        k, v = torch.cat([past[0], k]), torch.cat([past[1], v])
    out = attend(q, k, v, pos0, m.get("mask"), m["scale"], W[p + "temp"], [head_slope(hd, H) for hd in range(H)])
    y = rd(out.reshape(T, H * d) * sigmoid(h @ W[p + "g"].T))
    return y @ W[p + "o"].T, (k, v)


# ---- feed-forward ----------------------------------------------------------------------------------------------

def dense_ff(h, W, p):
    """W_down relu(W_up h)^2"""
    a = torch.clamp(h @ W[p + "up"].T, min=0.0)
    return (a * a) @ W[p + "down"].T


# ---- the model -------------------------------------------------------------------------------------------------

def weights_prefix(c: dict, i: int) -> str:
    """A layer that names another layer under weights_of runs that layer's tensors, norms and all."""
    return f"l{c['layers'][i].get('weights_of', i)}."


def layer_forward(c, W, i, x, round_to=None, carry=None, pos0: int = 0):
    """h = x mixed with the previous token's x; x <- norm1(alpha x + ls1 mixer(h)); x <- norm2(alpha x + ls2 ff(x)).
    carry: (the last token's x in front of this layer, keys and values) of earlier tokens.  Returns (x, carry after)."""
    L, eps, alpha, p = c["layers"][i], c["norm"]["eps"], c["postln_alpha"], weights_prefix(c, i)
    rd = (lambda t: t.to(round_to).to(F64)) if round_to is not None else (lambda t: t)
    before, past = carry if carry is not None else (None, None)
    h = rd(mix_with_previous(x, W[p + "shift"], before))
    last = x[-1].clone()
    y, past = windowed_attention(h, W, p + "mix.", L["mixer"], eps, pos0, past, round_to)
    x = add_and_norm(x, rd(y), alpha, W[p + "ls1"], W[p + "norm1"], eps)
    if L.get("mlp") is not None:
        y = dense_ff(rd(x), W, p + "mlp.")
        x = add_and_norm(x, rd(y), alpha, W[p + "ls2"], W[p + "norm2"], eps)
    return x, (last, past)


def forward(c: dict, W: dict, tokens, layers_out=None, round_to=None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  round_to: what an engine with activations of that type rounds where a
    sublayer reads and writes; layers_out: a list that receives the stream after every layer."""
    x = embed(W, tokens, c["embedding"]["scale"])
    for i in range(len(c["layers"])):
        x, _ = layer_forward(c, W, i, x, round_to)
        if layers_out is not None:
            layers_out.append(x.clone())
    h = unit_rms(x, c["norm"]["eps"]) * W["final.norm"]
    if round_to is not None:
        h = h.to(round_to).to(F64)
    return h @ W["head"].T


def generate(c: dict, W: dict, prompt, n_new: int):
    """Greedy continuation, the whole sequence run again for every token."""
    seq = list(prompt)
    for _ in range(n_new):
        seq.append(int(forward(c, W, seq)[-1].argmax()))
    return seq[len(prompt):]
