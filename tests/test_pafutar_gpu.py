"""The Pafutar architecture against the plain implementation of tests/plain_pafutar.py: every mechanism alone (the
kernels through their checked wrappers), then whole models built from folders that this file writes (its own small
configurations and weights), stepped through the engine in every way a request can arrive."""
import json
import math
import os

import pytest
import torch

import plain_pafutar as pp
from conftest import rel_err
from pafutar_cases import CONFIGS, _att, tokens, write_folder

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
# Bounds on the distance from the plain implementation (float64 from the same stored weights).  float32: the largest
# difference of any element over the reference's root mean square: summation order and the float32 functions.
# bfloat16: rounding the halves' inputs and outputs to 8 bits leaves rows of the small configurations 1 to 2 % of their
# root mean square off; a wrong key, a window off by one, a lost row of the state
# or a gate left out moves rows by a good part of their own size; float32 is what pins the formulas.
TOL = {torch.float32: 1e-4, torch.bfloat16: 0.05}
BF16_ELEMENT = 0.15
DEV = "cuda:0"


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """One folder a configuration, weights stored in bfloat16: engines of both types and the plain implementation read
    the same numbers."""
    made = {}

    def get(name):
        if name not in made:
            made[name] = write_folder(tmp_path_factory.mktemp(f"pafutar{name}"), CONFIGS[name], 31 + len(made))
        return made[name]
    return get


_plain_cache = {}


def plain(folder, toks):
    """Every prefix of a sequence has the logits of the sequence: the longest one seen serves the shorter ones."""
    for (f, t), v in _plain_cache.items():
        if f == folder and t[:len(toks)] == tuple(toks):
            return v[:len(toks)]
    _plain_cache[(folder, tuple(toks))] = pp.forward(pp.read_config(folder), pp.read_weights(folder), toks)
    return _plain_cache[(folder, tuple(toks))]


def engine(folder, dtype, max_tokens=1024, **kw):
    import bitnet_c_amd as bn
    return bn.Engine.from_folder(folder, dtype=dtype, max_tokens=max_tokens, **kw)


def close(got, want, dtype):
    e = rel_err(got, want)
    if dtype == torch.float32:
        assert e < TOL[dtype], f"relative error {e}"
        return
    g, w = got.detach().double().cpu().reshape(-1, got.shape[-1]), want.detach().double().cpu().reshape(-1, want.shape[-1])
    rms = float(w.pow(2).mean().sqrt())
    rows = float((g - w).pow(2).mean(dim=-1).sqrt().max()) / max(rms, 1e-30)
    assert rows < TOL[dtype] and e < BF16_ELEMENT, f"a row is {rows} rms off, an element {e}"


def stored(got, want, dtype, f32=1e-5):
    """What one kernel forms in float32 and stores in `dtype`: every element within one rounding."""
    assert got.dtype == dtype
    if dtype == torch.float32:
        return rel_err(got, want) < f32
    got, want = got.double().cpu(), want.double().cpu()
    return bool(((got - want).abs() <= 2.0 ** -8 * want.abs() + 1e-4 * want.pow(2).mean().sqrt()).all())


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


# ------------------------------------------------------------------------------------------------------------------
# mechanisms alone
# ------------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [10, 64, 2500])
def test_embedding_with_learned_position_vectors(dtype, D):
    from bitnet_c_amd import ops
    g = torch.Generator().manual_seed(D)
    table, pos = torch.randn(17, D, generator=g).to(dtype), torch.randn(9, D, generator=g).to(dtype)
    toks, at = [3, 16, 0, 3, 5], [0, 8, 4, -1, 7]
    got = ops.embed_gather_learned(table.to(DEV), i32(toks), i32(at), pos.to(DEV), 2.75)
    want = 2.75 * table[toks].double() + torch.stack([pos[p].double() if p >= 0 else torch.zeros(D).double() for p in at])
    assert got.dtype == torch.float32 and rel_err(got, want) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [7, 50, 64, 2048])
def test_token_shift_over_prompts_portions_and_single_tokens(dtype, D):
    """A step of five sequences (two go on from earlier tokens, one of a single token, one starts in a row that a former
    owner left full), padding rows behind them; then one token each; the state rows hold the last inputs, not their
    mixtures, and rows of no sequence of the step stay."""
    from bitnet_c_amd import ops
    g = torch.Generator().manual_seed(D)
    mu = torch.rand(D, generator=g) * 1.5 - 0.25
    lens, first, slots = [5, 2, 1, 70, 1], [0, 3, 9, 0, 0], [4, 1, 7, 2, 5]
    state = torch.randn(9, D + 4, generator=g)
    x = torch.randn(sum(lens), D, generator=g)
    st = state.to(DEV)
    seq = [b for b, n in enumerate(lens) for _ in range(n)]
    pos = [p0 + i for n, p0 in zip(lens, first) for i in range(n)]
    pad = 3
    out = ops.token_shift(torch.cat([x, torch.full((pad, D), 9.0)]).to(DEV), mu.reshape(1, -1).to(DEV), st, i32(pos + [-1] * pad),
                          i32(seq + [0] * pad), i32(slots), out_dtype=dtype, seq_lens=i32([a + b for a, b in zip(lens, first)]))[0]
    r, ends = 0, []
    for b, n in enumerate(lens):
        want = pp.mix_with_previous(x[r:r + n].double(), mu.double(), state[slots[b], :D].double() if first[b] else None)
        assert stored(out[r:r + n], want, dtype, 1e-6), b
        assert torch.equal(st[slots[b], :D].cpu(), x[r + n - 1])
        r += n
        ends.append(r - 1)
    assert torch.equal(st[:, D:].cpu(), state[:, D:]) and torch.equal(st[[0, 3, 6, 8]].cpu(), state[[0, 3, 6, 8]])
    # a step that reads the state only
    kept = st.clone()
    ops.token_shift(x[:1].to(DEV), mu.reshape(1, -1).to(DEV), st, i32([5]), i32([0]), i32([4]), out_dtype=dtype)
    assert torch.equal(st, kept)
    # one token each, in another order, with a padding row between
    y = torch.randn(4, D, generator=g)
    rows = [(3, 70), (None, -1), (0, 5), (2, 10)]
    got = ops.token_shift(y.to(DEV), mu.reshape(1, -1).to(DEV), st, i32([p for _, p in rows]), i32([0, 1, 2, 3]),
                          i32([slots[b] if b is not None else 8 for b, _ in rows]), out_dtype=dtype, seq_lens=i32([p + 1 for _, p in rows]))[0]
    for i, (b, p) in enumerate(rows):
        if b is None:
            continue
        assert stored(got[i], pp.mix_with_previous(y[i:i + 1].double(), mu.double(), x[ends[b]].double())[0], dtype, 1e-6)
        assert torch.equal(st[slots[b], :D].cpu(), y[i])
    assert torch.equal(st[8].cpu(), state[8])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [10, 24, 256, 2048, 2500, 5120, 9000])
@pytest.mark.parametrize("gained", [True, False])
def test_the_norm_behind_the_sum(dtype, D, gained):
    """alpha x + gain y under an RMS norm replaces the stream: y a tensor or float32 slabs; the rows handed on as they are,
    or mixed with the previous token's row (decode), whose state row then holds the new stream."""
    from bitnet_c_amd import ops
    from bitnet_c_amd.parts import NORMS, PartSpec, PostNormedDelta, ResidualStream
    g = torch.Generator().manual_seed(D)
    T, eps, alpha = 5, 0.3, 1.7                      # an eps that is seen
    x0, y = torch.randn(T, D, generator=g), (2.0 * torch.randn(T, D, generator=g)).to(dtype)
    slabs = torch.randn(3, T, D, generator=g)
    w, gain = 1 + 0.3 * torch.randn(D, generator=g), 1 + 0.5 * torch.randn(D, generator=g)
    mu = torch.rand(D, generator=g)
    norm = NORMS.build(PartSpec.of("rmsnorm", dim=D, eps=eps))
    norm.load({"weight": w}, DEV, dtype)
    none = NORMS.build(PartSpec.of("none", dim=D))
    pos, slots = [4, 0, -1, 300, 1], [2, 0, 5, 1, 4]
    state = torch.randn(6, D, generator=g)

    class Ctx:
        is_decode, act_dtype, positions, slot_ids = True, dtype, i32(pos), i32(slots)

    for delta, d in ((y.to(DEV), y.double()), (ops.PartialSums(slabs.to(DEV)), slabs.double().sum(0))):
        want = pp.add_and_norm(x0.double(), d, alpha, gain.double() if gained else torch.ones(D).double(), w.double(), eps)

        def stream():
            s = ResidualStream(x0.to(DEV).clone())
            s.add(PostNormedDelta(delta, norm, alpha, gain.to(DEV) if gained else None))
            return s
        s = stream()
        assert rel_err(s.flush(), want) < 2e-6 and s.pending is None
        s = stream()
        h = s.normed(none, dtype)
        assert h.dtype == dtype and rel_err(s.x, want) < 2e-6 and torch.equal(h.float(), s.x.to(dtype).float())
        s = stream()                                  # a norm of the next part's own, and a choice of rows: the stream first
        h = s.normed(norm, dtype, rows=i32([3, 0]))
        assert rel_err(s.x, want) < 2e-6
        assert stored(h, (pp.unit_rms(want, eps) * w.double())[[3, 0]], dtype)
        s, st = stream(), state.to(DEV)
        h = s.mixed_with_previous(mu.to(DEV), st, Ctx)
        assert rel_err(s.x, want) < 2e-6 and s.pending is None
        for r in (0, 1, 3, 4):
            before = state[slots[r]].double() if pos[r] > 0 else torch.zeros(D).double()
            assert stored(h[r], want[r] + (before - want[r]) * mu.double(), dtype)
            assert torch.equal(st[slots[r]], s.x[r])
        assert torch.equal(st[[3, 5]].cpu(), state[[3, 5]])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,hs", [(4, 2, 16), (6, 1, 10), (2, 2, 64), (3, 1, 130), (1, 1, 256)])
def test_biases_head_norms_without_weights_and_head_temperatures(dtype, H, G, hs):
    """q + bias and k + bias under norms without weights, the query times its head's number, the keys at their places in the
    pages, the values: the keys with their bias, not normed; gate columns behind the heads and padding rows are left alone."""
    from bitnet_c_amd import ops
    from bitnet_c_amd.cache import PAGE
    g = torch.Generator().manual_seed(H * 100 + hs)
    eps = 1e-2
    pos = [0, 1, 63, 64, 300, -1, 2047]
    T = len(pos)
    x0 = torch.randn(T, (H + G) * hs + H * hs, generator=g).to(dtype)
    bias, temp = torch.randn((H + G) * hs, generator=g), 1.0 + torch.rand(H, generator=g)
    live = [t for t, p in enumerate(pos) if p >= 0]
    qk = x0[:, :(H + G) * hs].double() + bias.double()
    q = (pp.unit_rms(qk[:, :H * hs].view(T, H, hs), eps) * temp.double()[:, None])[live]
    v = qk[:, H * hs:].view(T, G, hs)[live]
    k = pp.unit_rms(v, eps)
    kp = torch.zeros(40, G, PAGE, hs, dtype=dtype, device=DEV)
    vp = torch.zeros(40, G, hs, PAGE, dtype=dtype, device=DEV)
    table = i32([[(7 * j + 3) % 40 for j in range(33)]])
    x, ones = x0.to(DEV).clone(), torch.ones(hs, device=DEV)
    ops.qk_norm_store(x, i32(pos), H, G, hs, q_weight=ones, k_weight=ones, eps=eps, seq_index=i32([0] * T), block_table=table,
                      k_pages=kp, v_pages=vp, v_transposed=True, v_from_k=True, bias=bias.to(DEV), head_temp=temp.to(DEV))
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert rel_err(x[live, :H * hs], q.reshape(len(live), -1)) < tol
    assert torch.equal(x[:, H * hs:].cpu(), x0[:, H * hs:]) and torch.equal(x[5].cpu(), x0[5])
    for n, t in enumerate(live):
        page, at = int(table[0, pos[t] // PAGE]), pos[t] % PAGE
        assert rel_err(kp[page, :, at], k[n]) < tol and rel_err(vp[page, :, :, at], v[n]) < tol


class _Pages:
    """Keys and values of sequences of the given lengths in pages handed out in a shuffled order; every page that belongs to
    no sequence, and every place behind a sequence's end, holds large numbers that would be seen in a result."""

    def __init__(self, lens, G, hs, dtype, g):
        from bitnet_c_amd.cache import PAGE
        self.lens, per = lens, [-(-n // PAGE) for n in lens]
        order = torch.randperm(sum(per) + 2, generator=g).tolist()
        self.table = torch.zeros(len(lens), max(per), dtype=torch.int32)
        kp = torch.full((sum(per) + 2, G, PAGE, hs), 50.0)
        vp = torch.full((sum(per) + 2, G, hs, PAGE), 70.0)
        self.k = [torch.randn(n, G, hs, generator=g).to(dtype) for n in lens]
        self.v = [torch.randn(n, G, hs, generator=g).to(dtype) for n in lens]
        for b, n in enumerate(lens):
            for j in range(per[b]):
                page = order.pop()
                self.table[b, j] = page
                m = min(PAGE, n - j * PAGE)
                kp[page, :, :m] = self.k[b][j * PAGE:j * PAGE + m].permute(1, 0, 2).float()
                vp[page, :, :, :m] = self.v[b][j * PAGE:j * PAGE + m].permute(1, 2, 0).float()
        self.kp, self.vp, self.table = kp.to(dtype).to(DEV), vp.to(dtype).to(DEV), self.table.to(DEV)


def _tiles(n_new, pos0, qt):
    rows, r = [], 0
    for s, (n, p0) in enumerate(zip(n_new, pos0)):
        for i in range(0, n, qt):
            rows.append([s, r + i, min(qt, n - i), p0 + i])
        r += n
    return i32(rows)


MASKS = [(24, 3), (64, 0), (70, 64), (5, 70), (1, 1), (1, 0), (300, 2), (96, 130), (0, 0)]


@pytest.mark.parametrize("kernel", ["vector f32", "vector bf16", "matrix"])
@pytest.mark.parametrize("H,G,hs", [(4, 2, 32), (3, 1, 64), (2, 2, 10)])
@pytest.mark.parametrize("window,keep", MASKS)
def test_windows_with_kept_first_keys_and_a_linear_distance_bias(kernel, H, G, hs, window, keep):
    """Attention over pages for whole prompts, portions that begin at and around page and window edges, and single tokens
    (keys split and not), against the definition; the matrix-core kernels gate as they store."""
    from bitnet_c_amd import ops
    if kernel == "matrix" and hs == 10:
        return
    dtype = torch.float32 if kernel == "vector f32" else torch.bfloat16
    g = torch.Generator().manual_seed(window * 1000 + keep * 10 + hs)
    lens, pos0 = [200, 65, 130, 401, 1, 71], [0, 64, 127, 330, 0, 2]
    n_new = [n - p for n, p in zip(lens, pos0)]
    n_new[3] = lens[3] - pos0[3]
    pages = _Pages(lens, G, hs, dtype, g)
    slopes, temp = torch.tensor([0.05, 0.001, 0.0, 0.01][:H]), [1.0] * H
    bias, scale = (slopes.to(DEV), None), 2.0 * hs ** -0.5
    mask = dict(size=window, keep_first=keep) if window else None
    T = sum(n_new)
    q = torch.randn(T, H * hs, generator=g).to(dtype)
    wide = torch.randn(T, H * hs + 8, generator=g).to(dtype).to(DEV)
    gate = wide[:, 8:] if kernel == "matrix" else None
    want, r = [], 0
    for b, n in enumerate(n_new):
        o = pp.attend(q[r:r + n].double().view(n, H, hs), pages.k[b].double(), pages.v[b].double(), pos0[b], mask, scale, temp, slopes.tolist())
        want.append(o.reshape(n, H * hs))
        r += n
    want = torch.cat(want)
    gated = want * pp.sigmoid(gate.double().cpu()) if gate is not None else want
    tol = 1e-5 if dtype == torch.float32 else 5e-2           # the matrix-core kernels round the softmax's weights to 8 bits
    out = torch.full((T, H * hs), 7.0, dtype=dtype, device=DEV)
    if kernel == "matrix":
        ops.attention_general_prompt(q.to(DEV), out, pages.kp, pages.vp, pages.table, H, G, hs, hs, scale, _tiles(n_new, pos0, 16),
                                     distance_bias=bias, window=window, keep_first=keep, gate=gate)
    else:
        _, _, qt = ops.attention_row_shape(H, G, False)
        ops.attention(q.to(DEV), out, pages.kp, pages.vp, pages.table, H, G, hs, scale, window=window, keep_first=keep,
                      tiles=_tiles(n_new, pos0, qt), qt=qt, v_transposed=True, blocked=False, distance_bias=bias)
    r = 0
    for b, n in enumerate(n_new):                     # sequence by sequence: a short one is not hidden by a long one
        assert rel_err(out[r:r + n], gated[r:r + n]) < tol, b
        r += n
    # the last token of every sequence as a decode step, a padding row among them
    last = [sum(n_new[:b + 1]) - 1 for b in range(len(lens))]
    qd = torch.cat([q[last], torch.zeros(1, H * hs, dtype=dtype)]).to(DEV)
    table = torch.cat([pages.table, torch.zeros_like(pages.table[:1])])
    seq_lens = i32(lens + [0])
    gd = torch.cat([wide[last], wide[:1]])[:, 8:] if gate is not None else None
    plans = [(1, 0)]
    if kernel == "matrix":
        plans += [(4, 128), (7, 64)]
    elif dtype == torch.bfloat16 and window >= 256:
        plans += [(3, 128)]
    for n_splits, chunk in plans:
        out = torch.full((len(lens) + 1, H * hs), 7.0, dtype=dtype, device=DEV)
        if kernel == "matrix":
            ops.attention_general_decode(qd, out, pages.kp, pages.vp, table, seq_lens, H, G, hs, hs, scale, window=window, keep_first=keep,
                                         n_splits=n_splits, chunk=chunk, distance_bias=bias, gate=gd)
        else:
            ops.attention(qd, out, pages.kp, pages.vp, table, H, G, hs, scale, window=window, keep_first=keep, seq_lens=seq_lens,
                          n_splits=n_splits, chunk=chunk, v_transposed=True, blocked=False, distance_bias=bias)
        for b in range(len(lens)):
            assert rel_err(out[b], gated[last[b]]) < tol, (n_splits, b)


@pytest.mark.parametrize("kernel", ["vector f32", "vector bf16", "matrix"])
@pytest.mark.parametrize("window,keep", [(24, 3), (64, 64), (70, 1), (5, 70), (128, 130), (300, 6)])
def test_a_key_at_an_edge_is_seen_or_not(kernel, window, keep):
    """One key is made to stand out (it and the query are scaled along one direction) and moved over every edge there is: the
    first and last kept key, the first one behind, the last that has left the window, the first inside it, page borders, the
    query's own.  Where it is visible its value is the result, in a prompt and decoded; where it is not it carries nothing."""
    from bitnet_c_amd import ops
    dtype = torch.float32 if kernel == "vector f32" else torch.bfloat16
    H, G, hs = 2, 1, 32
    g = torch.Generator().manual_seed(window + keep)
    n = 330
    i = n - 1
    bias, mask = (torch.zeros(H, device=DEV), None), dict(size=window, keep_first=keep)
    pages = _Pages([n], G, hs, dtype, g)
    q = torch.zeros(1, H * hs)
    q[0, 0::hs] = 8.0
    q = q.to(dtype)
    seen = set(pp.visible(i, mask))
    edges = {0, keep - 1, keep, keep + 1, i - window - 1, i - window, i - window + 1, i, 63, 64, 127, 128, 255, 256}
    for j in sorted(e for e in edges if 0 <= e <= i):
        kp = pages.kp.clone()
        page = int(pages.table[0, j // 64])
        kp[page, 0, j % 64] = 0
        kp[page, 0, j % 64, 0] = 8.0
        for form in ("prompt", "decode"):
            out = torch.empty((1, H * hs), dtype=dtype, device=DEV)
            if kernel == "matrix" and form == "prompt":
                ops.attention_general_prompt(q.to(DEV), out, kp, pages.vp, pages.table, H, G, hs, hs, 0.5, i32([[0, 0, 1, i]]), distance_bias=bias,
                                             window=window, keep_first=keep)
            elif kernel == "matrix":
                ops.attention_general_decode(q.to(DEV), out, kp, pages.vp, pages.table, i32([n]), H, G, hs, hs, 0.5, window=window, keep_first=keep,
                                             n_splits=6, chunk=64, distance_bias=bias)
            elif form == "prompt":
                _, _, qt = ops.attention_row_shape(H, G, False)
                ops.attention(q.to(DEV), out, kp, pages.vp, pages.table, H, G, hs, 0.5, window=window, keep_first=keep,
                              tiles=i32([[0, 0, 1, i]]), qt=qt, v_transposed=True, blocked=False, distance_bias=bias)
            else:
                ops.attention(q.to(DEV), out, kp, pages.vp, pages.table, H, G, hs, 0.5, window=window, keep_first=keep, seq_lens=i32([n]),
                              v_transposed=True, blocked=False, distance_bias=bias)
            v = pages.v[0][j, 0].double().repeat(H)
            err = float((out[0].double().cpu() - v).norm() / v.norm())
            assert (err < 0.02) if j in seen else (err > 0.3), (j, form, err)


@pytest.mark.parametrize("M,N,K", [(1, 40, 64), (7, 136, 72), (16, 256, 2048), (17, 64, 64), (5, 30, 50)])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("activation", ["relu2", "gelu_erf"])
def test_a_product_with_its_activation(dtype, M, N, K, activation):
    from bitnet_c_amd import ops
    g = torch.Generator().manual_seed(M + N)
    x, w = torch.randn(M, K, generator=g).to(dtype), (torch.randn(N, K, generator=g) / math.sqrt(K)).to(dtype)
    z = x.double() @ w.double().T
    want = torch.clamp(z, min=0.0) ** 2 if activation == "relu2" else torch.nn.functional.gelu(z)
    streamed = ops.stream_copy(w.to(DEV)) if dtype == torch.bfloat16 and K % 8 == 0 else None
    for sw in (None, streamed):
        got = ops.linear_unary(x.to(DEV), w.to(DEV), activation, sw)
        assert got.dtype == dtype and rel_err(got, want) < (2e-5 if dtype == torch.float32 else 8e-2)


# ------------------------------------------------------------------------------------------------------------------
# whole models through the engine
# ------------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompts_and_the_stream_after_every_layer(folders, name, dtype):
    import bitnet_c_amd as bn
    folder = folders(name)
    eng = engine(folder, dtype)
    for n in (1, 2, 77, 200):
        toks = tokens(CONFIGS[name], n, n)
        streams, got = [], []
        want = pp.forward(pp.read_config(folder), pp.read_weights(folder), toks, streams)
        eng.tap = lambda point, entry, stream, ctx: got.append(stream.flush().clone()) if point == "layer_out" else None
        s = eng.new_sequence()
        logits = eng.step([bn.StepEntry(s, toks, list(range(n)))])
        eng.release(s)
        eng.tap = None
        assert len(got) == len(streams) == len(CONFIGS[name]["layers"])
        for a, b in zip(got, streams):
            close(a, b, dtype)
        close(logits, want, dtype)
        s = eng.new_sequence()                            # and without anybody looking: the fused steps
        close(eng.step([bn.StepEntry(s, toks, list(range(n)))]), want, dtype)
        eng.release(s)
    eng.cache.check()


@pytest.mark.parametrize("graphs", [True, False])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prefill_against_decoding_token_by_token(folders, name, dtype, graphs):
    """A prompt, then 150 tokens one by one (across page borders and every window), against the plain implementation of the
    whole sequence; and the same sequence from its very first token one by one."""
    import bitnet_c_amd as bn
    folder = folders(name)
    eng = engine(folder, dtype, use_graphs=graphs)
    toks = tokens(CONFIGS[name], 200, 1)
    want = plain(folder, toks)
    for first in (50, 1):
        s = eng.new_sequence()
        parts = [eng.step([bn.StepEntry(s, toks[:first], list(range(first)))])]
        for t in range(first, len(toks) if first == 50 else 80):
            parts.append(eng.step([bn.StepEntry(s, [toks[t]], [0])]))
        eng.release(s)
        got = torch.cat(parts)
        close(got, want[:got.shape[0]], dtype)
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_of_several_sizes(folders, name, dtype):
    """A prompt cut into portions of 2, 3, 1, 64, 5, 2, ... tokens gives what the whole prompt gives."""
    import bitnet_c_amd as bn
    folder = folders(name)
    eng = engine(folder, dtype)
    toks = tokens(CONFIGS[name], 200, 1)
    want = plain(folder, toks)
    for cuts in ([2, 3, 1, 64, 5, 2, 40, 2, 31, 50], [2] * 100, [199, 1], [63, 1, 1, 85, 50], [15, 1, 16, 17, 101, 50]):
        assert sum(cuts) == len(toks)
        s, at, parts = eng.new_sequence(), 0, []
        for n in cuts:
            parts.append(eng.step([bn.StepEntry(s, toks[at:at + n], list(range(n)))]))
            at += n
        eng.release(s)
        close(torch.cat(parts), want, dtype)
    eng.cache.check()


@pytest.mark.parametrize("graphs", [True, False])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_unequal_batches_and_slots_used_again(folders, name, dtype, graphs):
    """Requests of 1, 70, 9 and 130 tokens as one batch, decoded together while the shorter ones end; then other
    requests in the slots, pages and state rows that were given back; every request against itself alone (the plain
    implementation)."""
    import bitnet_c_amd as bn
    folder = folders(name)
    eng = engine(folder, dtype, max_tokens=1024, use_graphs=graphs)
    for round_, lens in enumerate(([1, 70, 9, 130], [64, 3, 128], [5])):
        reqs = [tokens(CONFIGS[name], n + 6 + 3 * i, 10 * round_ + i) for i, n in enumerate(lens)]
        slots = [eng.new_sequence() for _ in reqs]
        got = [[] for _ in reqs]
        out = eng.step([bn.StepEntry(s, r[:n], [n - 1]) for s, r, n in zip(slots, reqs, lens)])
        for i in range(len(reqs)):
            got[i].append(out[i:i + 1])
        at = list(lens)
        live = list(range(len(reqs)))
        while live:
            out = eng.step([bn.StepEntry(slots[i], [reqs[i][at[i]]], [0]) for i in live])
            for j, i in enumerate(live):
                got[i].append(out[j:j + 1])
                at[i] += 1
            for i in [i for i in live if at[i] == len(reqs[i])]:
                eng.release(slots[i])
                live.remove(i)
        for i, r in enumerate(reqs):
            close(torch.cat(got[i]), plain(folder, r)[lens[i] - 1:], dtype)
        eng.cache.check()
    assert eng.cache.live_slots() == []


@pytest.mark.parametrize("dtype", DTYPES)
def test_batches_of_more_rows_than_a_tile_of_the_products(folders, dtype):
    """Forty sequences decoded together (products of many rows, partial sums for the last product of a half)."""
    import bitnet_c_amd as bn
    folder = folders("C")
    eng = engine(folder, dtype, max_tokens=40 * 128)
    reqs = [tokens(CONFIGS["C"], 3 + (7 * i) % 60 + 4, 100 + i) for i in range(40)]
    slots = [eng.new_sequence() for _ in reqs]
    eng.step([bn.StepEntry(s, r[:-4], []) for s, r in zip(slots, reqs)])
    outs = [eng.step([bn.StepEntry(s, [r[t]], [0]) for s, r in zip(slots, reqs)]) for t in (-4, -3, -2, -1)]
    for i, r in enumerate(reqs):
        close(torch.stack([o[i] for o in outs]), plain(folder, r)[-4:], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_steps_replayed_from_graphs(folders, name, dtype):
    """Prompt steps of one size run eagerly the first time, are recorded the second time and replayed afterwards, with
    other sequences in other slots each time: every one of them against the plain implementation, and what a recorded step
    left in the cache and in the states is what the tokens decoded behind it go on from."""
    import bitnet_c_amd as bn
    folder = folders(name)
    eng = engine(folder, dtype)
    assert eng.prompt_graphs and eng.use_graphs
    keep = eng.new_sequence()                      # a live neighbour, so that later sequences get other slots
    eng.step([bn.StepEntry(keep, tokens(CONFIGS[name], 9, 1), [])])
    for i in range(5):
        reqs = [tokens(CONFIGS[name], n, 50 + 2 * i + k) for k, n in enumerate((70 + i, 20 - i))]
        slots = [eng.new_sequence() for _ in reqs]
        out = eng.step([bn.StepEntry(s, r[:-3], [0, len(r) - 4]) for s, r in zip(slots, reqs)])
        tail = [eng.step([bn.StepEntry(s, [r[t]], [0]) for s, r in zip(slots, reqs)]) for t in (-3, -2, -1)]
        for k, r in enumerate(reqs):
            want = plain(folder, r)
            close(out[2 * k:2 * k + 2], want[[0, len(r) - 4]], dtype)
            close(torch.cat([t[k:k + 1] for t in tail]), want[-3:], dtype)
        eng.release(slots[i % 2])
    assert eng.graphs_built >= 2                   # a prompt step and the decode steps were recorded
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_step_that_mixes_single_tokens_and_portions(folders, dtype):
    import bitnet_c_amd as bn
    folder, cfg = folders("A"), CONFIGS["A"]
    eng = engine(folder, dtype)
    a, b, c = tokens(cfg, 30, 2), tokens(cfg, 90, 3), tokens(cfg, 12, 4)
    sa, sb, sc = (eng.new_sequence() for _ in range(3))
    eng.step([bn.StepEntry(sa, a[:29], []), bn.StepEntry(sb, b[:10], [])])
    out = eng.step([bn.StepEntry(sa, a[29:], [0]), bn.StepEntry(sb, b[10:], [0, 79]), bn.StepEntry(sc, c, [11])])
    want = torch.stack([plain(folder, a)[29], plain(folder, b)[10], plain(folder, b)[89], plain(folder, c)[11]])
    close(out, want, dtype)


def _peaked_folder(tmp_path):
    """A model whose attention is peaked (large scales and temperatures: single keys carry a query's result, kept first ones
    a thousand tokens away against their distance's price among them), with windows of several sizes."""
    cfg = dict(architecture="Pafutar", vocab=61, width=32, max_positions=2600, norm=dict(eps=1e-5), embedding=dict(scale=2.0),
               postln_alpha=1.1, layers=[_att(8, 2, 8, 1.5, (100, 6), 48), _att(2, 2, 16, 1.0, (33, 70), None),
                                         _att(4, 1, 32, 0.6, None, 40)])
    over = {"l0.mix.temp": torch.full((8,), 2.0), "l1.mix.temp": torch.full((2,), 1.5)}
    return write_folder(tmp_path / "peaked", cfg, 9, overrides=over), cfg


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_with_far_kept_keys(tmp_path, dtype):
    """A long sequence (past a run of a float32 cache's keys, many pages given back), as a prompt in portions and then
    decoded for 80 tokens."""
    import bitnet_c_amd as bn
    folder, cfg = _peaked_folder(tmp_path)
    toks = tokens(cfg, 2200, 2)
    want = pp.forward(pp.read_config(folder), pp.read_weights(folder), toks)
    eng = engine(folder, dtype, max_tokens=4608)
    s, at, parts = eng.new_sequence(), 0, []
    check = [0, 1, 5, 6, 33, 63, 64, 69, 70, 99, 100, 101, 299, 300, 2047, 2048, 2049, 2119]
    for n in (1000, 1047, 73):
        w = [p - at for p in check if at <= p < at + n]
        parts.append(eng.step([bn.StepEntry(s, toks[at:at + n], w)]))
        at += n
    close(torch.cat(parts), want[check], dtype)
    dec = torch.cat([eng.step([bn.StepEntry(s, [toks[t]], [0])]) for t in range(at, 2200)])
    close(dec, want[at:], dtype)
    s2 = eng.new_sequence()                              # and the same positions from one step over the whole sequence
    whole = eng.step([bn.StepEntry(s2, toks, list(range(at, 2200)))])
    if dtype == torch.float32:
        assert rel_err(dec, whole) < 2e-5
    else:
        close(dec, whole.double(), dtype)
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_logits_do_not_depend_on_the_cut_or_the_batch(folders, dtype):
    """Whole, in portions, one by one and beside other requests: float32 logits agree to the last bits, bfloat16 within
    its rounding (steps of few rows and of many take different kernels for the products)."""
    import bitnet_c_amd as bn
    for name in ("A", "C"):
        folder, cfg = folders(name), CONFIGS[name]
        eng = engine(folder, dtype)
        toks, other = tokens(cfg, 160, 1), tokens(cfg, 37, 3)
        s = eng.new_sequence()
        whole = eng.step([bn.StepEntry(s, toks, list(range(160)))])
        eng.release(s)
        s, o = eng.new_sequence(), eng.new_sequence()
        a = eng.step([bn.StepEntry(o, other, []), bn.StepEntry(s, toks[:37], list(range(37)))])
        b = eng.step([bn.StepEntry(s, toks[37:159], list(range(122)))])
        c = eng.step([bn.StepEntry(s, toks[159:], [0]), bn.StepEntry(o, [5], [])])
        got = torch.cat([a, b, c])
        if dtype == torch.float32:
            assert rel_err(got, whole) < 2e-6
        else:
            close(got, whole.double(), dtype)


def test_positions_end_with_their_table(folders):
    import bitnet_c_amd as bn
    from bitnet_c_amd.engine import StepError
    eng = engine(folders("D"), torch.float32, max_tokens=1024)
    toks = tokens(CONFIGS["D"], 257, 1)
    s = eng.new_sequence()
    with pytest.raises(StepError, match="256"):
        eng.step([bn.StepEntry(s, toks, [])])
    got = eng.step([bn.StepEntry(s, toks[:256], [255])])
    close(got, plain(folders("D"), toks[:256])[255:], torch.float32)
    with pytest.raises(StepError, match="256"):
        eng.step([bn.StepEntry(s, toks[256:], [0])])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_greedy_generation_through_the_entry_point(folders, name, dtype):
    """Greedy generation through load() and generate(), the scheduler batching three prompts two at a time: every token that
    was chosen holds, where it was chosen, the plain implementation's largest logit within rounding."""
    import bitnet_c_amd as bn
    folder = folders(name)
    llm = bn.load(folder, dtype="float32" if dtype == torch.float32 else "bfloat16", max_tokens=1024)
    prompts = [tokens(CONFIGS[name], n, 20 + i) for i, n in enumerate((5, 66, 1))]
    got = llm.generate(prompts, max_new_tokens=12, temperature=0.0, stop_ids=(), batch_size=2)
    cfg, W = pp.read_config(folder), pp.read_weights(folder)
    for p, g in zip(prompts, got):
        assert len(g) == 12
        logits = pp.forward(cfg, W, p + g)[len(p) - 1:-1]
        rms = float(logits.pow(2).mean().sqrt())
        for i, tok in enumerate(g):
            gap = float(logits[i].max() - logits[i, tok])
            assert gap <= (1e-4 if dtype == torch.float32 else 0.1) * rms, (i, gap / rms)
    if dtype == torch.float32:
        assert got[0] == pp.generate(cfg, W, prompts[0], 12)
    llm.engine.cache.check()
    assert llm.engine.cache.live_slots() == []


def test_command_line_and_trace_replay(folders, tmp_path):
    """The command line generates from a Pafutar folder (also one that it writes itself from a configuration file, with
    random weights), and the trace replay program steps one through a batch of prompts and single tokens."""
    import subprocess
    import sys
    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder = folders("D")
    cfg, W = pp.read_config(folder), pp.read_weights(folder)
    prompt = tokens(CONFIGS["D"], 8, 1)
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "bitnet"), folder, "--prompt-token-ids", ",".join(map(str, prompt)),
                        "-n", "6", "--repeat-penalty", "1.0", "--fp32", "--token-ids", "--quiet"], capture_output=True, text=True,
                       timeout=300)
    assert p.returncode == 0, p.stderr[-1500:]
    ids = [int(x) for x in [l for l in p.stderr.splitlines() if l and l[0].isdigit()][0].split(",")]
    logits = pp.forward(cfg, W, prompt + ids)[len(prompt) - 1:-1]
    for i, tok in enumerate(ids):
        assert float(logits[i].max() - logits[i, tok]) <= 1e-4 * float(logits.pow(2).mean().sqrt())
    conf = tmp_path / "conf.json"
    conf.write_text(json.dumps(CONFIGS["B"]))
    made = str(tmp_path / "made")
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "bitnet"), made, "--random", str(conf), "--seed", "4",
                        "--prompt-token-ids", "1,2,3", "-n", "4", "--fp32", "--token-ids", "--quiet", "--repeat-penalty", "1.0"],
                       capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-1500:]
    assert len([l for l in p.stderr.splitlines() if l and l[0].isdigit()][0].split(",")) == 4
    assert pp.read_config(made)["layers"] == CONFIGS["B"]["layers"]
    # trace replay: two requests that start together, then go on token by token; the shorter one ends earlier
    folder = folders("A")
    a, b = tokens(CONFIGS["A"], 40, 2), tokens(CONFIGS["A"], 7, 3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:37], "want": [0, 29, 36]}, {"id": "b", "tokens": b[:5], "want": [4]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[37:38], "want": [0]}, {"id": "b", "tokens": b[5:6], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[38:39], "want": []}, {"id": "b", "tokens": b[6:], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[39:], "want": [0]}], "end": ["a"]}]
    for dtype, name in ((torch.float32, "float32"), (torch.bfloat16, "bfloat16")):
        out = tmp_path / ("out_" + name)
        p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", name,
                            "--out", str(out), "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                           capture_output=True, text=True, timeout=300)
        assert p.returncode == 0, p.stderr[-1500:]
        assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
        assert sorted(os.listdir(out)) == ["0.f32", "1.f32", "2.f32", "3.f32"]
        la, lb = plain(folder, a), plain(folder, b)
        want_rows = {0: torch.stack([la[0], la[29], la[36], lb[4]]), 1: la[37:38], 2: lb[6:7], 3: la[39:40]}
        for i, w in want_rows.items():
            got = torch.from_numpy(np.fromfile(str(out / f"{i}.f32"), dtype="<f4").reshape(-1, CONFIGS["A"]["vocab"]))
            close(got, w, dtype)
