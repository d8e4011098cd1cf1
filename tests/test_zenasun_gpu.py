"""The Zenasun architecture against the plain implementation of tests/plain_zenasun.py: every mechanism alone (the kernels
through their checked wrappers), then whole models built from folders that this file writes (its own small configurations
and weights), stepped through the engine in every way a request can arrive."""
import json
import math
import os

import pytest
import torch

import plain_zenasun as pz
from conftest import rel_err
from zenasun_cases import CONFIGS, _lat, _model, _ret, settled_tokens, write_folder

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
# Bounds on the distance from the plain implementation (float64 from the same stored weights).  float32: the largest
# difference of any element over the reference's root mean square.  bfloat16: rounding the two norms' outputs alone moves
# whole rows of these small models by 1.5 to 8 % of their root mean square (measured on the CPU), so a row's
# root-mean-square difference is bounded by 15 % and any element by 60 %; float32 is what pins the formulas.  A wrong key,
# a lost state, a sink left out or another expert moves rows by their own size.
TOL = {torch.float32: 3e-4, torch.bfloat16: 0.15}
BF16_ELEMENT = 0.6
DEV = "cuda:0"


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = write_folder(tmp_path_factory.mktemp(f"zenasun{name}"), CONFIGS[name], 31)
        return made[name]
    return get


_plain_cache = {}


def plain(folder, tokens):
    key = (folder, tuple(tokens))
    if key not in _plain_cache:
        _plain_cache[key] = pz.forward(pz.read_config(folder), pz.read_weights(folder), tokens)
    return _plain_cache[key]


def engine(folder, dtype, max_tokens=1024, **kw):
    import bitnet_c_amd as bn
    return bn.Engine.from_folder(folder, dtype=dtype, max_tokens=max_tokens, **kw)


def close(got, want, dtype, bf16_rows=None):
    e = rel_err(got, want)
    if dtype == torch.float32:
        assert e < TOL[dtype], f"relative error {e}"
        return
    g, w = got.detach().double().cpu().reshape(-1, got.shape[-1]), want.detach().double().cpu().reshape(-1, want.shape[-1])
    rms = float(w.pow(2).mean().sqrt())
    rows = float((g - w).pow(2).mean(dim=-1).sqrt().max()) / max(rms, 1e-30)
    assert rows < (bf16_rows or TOL[dtype]) and e < BF16_ELEMENT, f"a row is {rows} rms off, an element {e}"


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


def f32(v):
    return v.to(torch.float32).to(DEV).contiguous()


# ------------------------------------------------------------------------------------------------------------------
# mechanisms alone
# ------------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [24, 50, 256, 2500, 9000])
def test_two_norms_of_one_stream_and_outputs_that_join_it_together(dtype, D):
    """The first pair of norms, with nothing held back; then a tensor and float32 slabs that join the stream at once in
    front of the next pair; one output alone under one norm; a choice of rows; the sum alone.  The stored weights mean
    1 + w, and the two norms have an eps each."""
    from bitnet_c_amd import ops
    from bitnet_c_amd.parts import NORMS, PartSpec, ResidualStream
    from bitnet_c_amd.parts.base import JoinedDelta
    g = torch.Generator().manual_seed(D)
    T, eps = 6, (1e-5, 0.7)
    x0 = torch.randn(T, D, generator=g)
    w = [0.3 * torch.randn(D, generator=g) for _ in range(2)]
    norms = []
    for wk, ek in zip(w, eps):
        n = NORMS.build(PartSpec.of("rmsnorm", dim=D, eps=ek, offset=1.0))
        n.load({"weight": wk}, DEV, dtype)
        norms.append(n)
    y = (2.0 * torch.randn(T, D, generator=g)).to(dtype)
    slabs = torch.randn(3, T, D, generator=g)
    tol = 1e-5 if dtype == torch.float32 else 2e-2

    def check(pair, x):
        for h, wk, ek in zip(pair, w, eps):
            assert h.dtype == dtype and rel_err(h, pz.shifted_norm(x, wk.double(), ek)) < tol
    stream = ResidualStream(x0.to(DEV).clone())
    X = x0.double()
    check(stream.normed_twice(*norms, dtype), X)
    assert torch.equal(stream.x.cpu(), x0)
    stream.add(JoinedDelta([y.to(DEV), ops.PartialSums(slabs.to(DEV))]))
    check(stream.normed_twice(*norms, dtype), X + y.double() + slabs.double().sum(0))
    X = X + y.double() + slabs.double().sum(0)
    assert stream.pending is None and rel_err(stream.x, X) < 1e-6
    stream.add(JoinedDelta([y.to(DEV)]))
    h = stream.normed(norms[1], dtype)
    X = X + y.double()
    assert rel_err(h, pz.shifted_norm(X, w[1].double(), eps[1])) < tol and rel_err(stream.x, X) < 1e-6
    stream.add(JoinedDelta([ops.PartialSums(slabs.to(DEV)), y.to(DEV)]))
    rows = stream.normed(norms[0], dtype, rows=i32([5, 0, 5]))               # the model's end: a choice of rows
    X = X + y.double() + slabs.double().sum(0)
    assert rel_err(rows, pz.shifted_norm(X, w[0].double(), eps[0])[[5, 0, 5]]) < tol and rel_err(stream.flush(), X) < 1e-6
    stream.add(JoinedDelta([y.to(DEV), y.to(DEV)]))                          # two tensors: one after the other
    check(stream.normed_twice(*norms, dtype), X + 2.0 * y.double())
    stream.add(y.to(DEV))                                                    # an output held back the plain way
    check(stream.normed_twice(*norms, dtype), X + 3.0 * y.double())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chain", [False, True])
@pytest.mark.parametrize("H,dk,dv,rd", [(3, 16, 24, 8), (2, 10, 70, 10), (1, 64, 64, 64), (2, 128, 130, 96), (1, 200, 8, 66), (5, 1, 1, 0),
                                        (4, 6, 20, 2)])
def test_retention_over_prompts_portions_and_single_tokens(dtype, H, dk, dv, rd, chain):
    """The recurrence over rotated queries and keys in a step of three sequences of unequal lengths (one continues at
    position 300 from a state, one starts in a row that a former sequence left its state in), then one token each beside a
    padding row, against the recurrence written token by token; the projections lie side by side in one tensor with other
    columns around them.  Lengths that end on a chunk's edge and one behind it."""
    from bitnet_c_amd import ops
    from bitnet_c_amd.parts.position import rope_frequencies
    g = torch.Generator().manual_seed(dk * 7 + dv)
    decay = torch.tensor([0.9, 1.0, 0.0, 0.999, 0.5][:H], dtype=torch.float64)
    lens, first, slots = [128, 1, 65], [300, 0, 0], [4, 1, 2]
    qc, kc, vc, W = 3, 3 + H * dk + 2, 3 + 2 * H * dk + 4, 3 + 2 * H * dk + 4 + H * dv + 1
    state = torch.zeros(6, H * dk * dv + 3)
    state[1] = 7.0
    rot = dict(base=300.0, dims=rd)
    inv = rope_frequencies(rd, rot["base"]).to(DEV) if rd else None

    def halves(x, p0):
        x = x.double()
        q, k, v = x[:, qc:qc + H * dk].view(-1, H, dk), x[:, kc:kc + H * dk].view(-1, H, dk), x[:, vc:vc + H * dv].view(-1, H, dv)
        if rd:
            at = range(p0, p0 + x.shape[0])
            q, k = pz.rotate_halves(q, at, rot, torch.float32), pz.rotate_halves(k, at, rot, torch.float32)
        return q, k * dk ** -0.5, v
    xs, want, S_after = [], [], []
    for b, (n, p0) in enumerate(zip(lens, first)):
        S0 = None
        if p0:
            S0 = torch.randn(H, dk, dv, generator=g).double()
            state[slots[b], :H * dk * dv] = S0.reshape(-1).float()
            S0 = state[slots[b], :H * dk * dv].double().view(H, dk, dv)
        x = (0.7 * torch.randn(n + 1, W, generator=g)).to(dtype)
        o, _ = pz.decayed_sums(*halves(x, p0), decay, S0)
        _, S = pz.decayed_sums(*halves(x[:-1], p0), decay, S0)
        xs.append(x)
        want.append(o)
        S_after.append(S)
    st, tiles, pos, r = state.to(DEV), [], [], 0
    for b, n in enumerate(lens):
        tiles.append([b, r, n, first[b]])
        pos += list(range(first[b], first[b] + n))
        r += n
    x = torch.cat([t[:-1] for t in xs]).to(DEV)
    feed = dict(silu=False, inv_freq=inv, k_scale=dk ** -0.5)
    o = ops.lightning_scan(x, qc, kc, vc, f32(decay), st, i32(slots), H, dk, dv, tiles=i32(tiles + [[0, 0, 0, 0]]), chain=chain,
                           positions=i32(pos), **feed)
    assert rel_err(o, torch.cat([w[:-1] for w in want]).reshape(sum(lens), -1)) < 3e-5
    for b in range(3):
        assert rel_err(st[slots[b], :H * dk * dv], S_after[b].reshape(-1)) < 3e-5
    assert torch.equal(st[[0, 3, 5]].cpu(), state[[0, 3, 5]]) and torch.equal(st[:, H * dk * dv:].cpu(), state[:, H * dk * dv:])
    xd = torch.stack([xs[2][-1], xs[0][-1], torch.zeros(W, dtype=dtype), xs[1][-1]]).to(DEV)
    od = ops.lightning_scan(xd, qc, kc, vc, f32(decay), st, i32([slots[2], slots[0], 5, slots[1]]), H, dk, dv,
                            seq_lens=i32([lens[2] + 1, first[0] + lens[0] + 1, 0, 2]),
                            positions=i32([lens[2], first[0] + lens[0], -1, 1]), **feed)
    assert rel_err(od[[0, 1, 3]], torch.stack([want[2][-1], want[0][-1], want[1][-1]]).reshape(3, -1)) < 3e-5
    assert torch.equal(st[[0, 3, 5]].cpu(), state[[0, 3, 5]])


@pytest.mark.parametrize("dtype", DTYPES)
def test_retention_meets_a_key_far_back_at_its_distance(dtype):
    """One key far back and the last query are long and alike: under a slow decay the product of the two, turned by their
    distance, is what comes out of the first head, and a distance that is one token off would show; the second head has
    forgotten it.  As a prompt, in portions and decoded."""
    from bitnet_c_amd import ops
    from bitnet_c_amd.parts.position import rope_frequencies
    g = torch.Generator().manual_seed(5)
    H, dk, dv, T, far = 2, 32, 32, 1000, 100
    rot = dict(base=10000.0, dims=32)
    decay = torch.tensor([0.9999, 0.97], dtype=torch.float64)
    x = 0.2 * torch.randn(T, 2 * H * dk + H * dv, generator=g)
    peak = 8.0 * torch.randn(dk, generator=g)
    for h in range(H):
        x[far, H * dk + h * dk:H * dk + (h + 1) * dk] = peak
        x[T - 1, h * dk:(h + 1) * dk] = peak
    x[far, 2 * H * dk:] = 3.0 * torch.randn(H * dv, generator=g)
    x = x.to(dtype)
    q, k, v = (x.double()[:, :H * dk].view(T, H, dk), x.double()[:, H * dk:2 * H * dk].view(T, H, dk), x.double()[:, 2 * H * dk:].view(T, H, dv))
    # positions of three digits times frequencies of one: an angle in float32 is off by 1e-4, against a long key
    q, k = pz.rotate_halves(q, range(T), rot, torch.float32), pz.rotate_halves(k, range(T), rot, torch.float32) * dk ** -0.5
    want, _ = pz.decayed_sums(q, k, v, decay)
    share = 0.9999 ** 899 * float(q[-1, 0] @ k[far, 0]) * v[far, 0]
    off = 0.9999 ** 899 * float(pz.rotate_halves(x.double()[-1:, :H * dk].view(1, H, dk), [T], rot)[0, 0] @ k[far, 0]) * v[far, 0]
    assert float((want[-1, 0] - share).norm() / want[-1, 0].norm()) < 0.3 and float((off - share).norm() / share.norm()) > 0.05
    assert float(want[-1, 1].norm()) < 0.2 * float(want[-1, 0].norm())
    inv = rope_frequencies(32, rot["base"]).to(DEV)
    for cut in (T, T - 1, 700):
        st = torch.zeros(2, H * dk * dv, dtype=torch.float32, device=DEV)
        feed = dict(silu=False, inv_freq=inv, k_scale=dk ** -0.5)
        parts, at = [], 0
        for n in (cut // 3, cut - cut // 3):
            parts.append(ops.lightning_scan(x[at:at + n].to(DEV), 0, H * dk, 2 * H * dk, f32(decay), st, i32([1]), H, dk, dv,
                                            tiles=i32([[0, 0, n, at]]), positions=i32(list(range(at, at + n))), **feed))
            at += n
        for t in range(cut, T):
            parts.append(ops.lightning_scan(x[t:t + 1].to(DEV), 0, H * dk, 2 * H * dk, f32(decay), st, i32([1]), H, dk, dv,
                                            seq_lens=i32([t + 1]), positions=i32([t]), **feed))
        got = torch.cat(parts)
        assert rel_err(got[-1], want[-1].reshape(-1)) < 1e-3 and rel_err(got[:-1], want[:-1].reshape(T - 1, -1)) < 1e-3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dv", [(3, 24), (1, 70), (16, 128)])
def test_heads_normed_one_by_one_without_a_weight_and_gated(dtype, H, dv):
    from bitnet_c_amd import ops
    g = torch.Generator().manual_seed(H + dv)
    T, eps = 5, 1e-3
    o = torch.randn(T, H * dv, generator=g) * torch.logspace(-2, 1, T)[:, None]
    wide = torch.randn(T, H * dv + 5, generator=g).to(dtype)
    want = pz.unit_rms(o.double().view(T, H, dv), eps).reshape(T, -1) * pz.silu(wide[:, 5:].double())
    got = ops.head_norm_gate(f32(o), wide.to(DEV)[:, 5:], None, H, dv, eps)
    assert got.dtype == dtype and rel_err(got, want) < (1e-5 if dtype == torch.float32 else 5e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("interleaved", [True, False])
@pytest.mark.parametrize("R,rot,qr", [(40, 8, 24), (14, 2, 9), (120, 24, 200), (96, 32, 48), (8, 0, 4), (512, 64, 300)])
def test_the_latents_of_keys_and_queries_in_one_kernel(dtype, interleaved, R, rot, qr):
    """The latent under its norm as a key row and in the transposed value page, the rotated part behind it, zeros behind
    that where stored rows are wider; the queries' latent under a norm of its own from other columns of the same row, also
    of a row that stores nothing; positions at a page's border and far away."""
    from bitnet_c_amd import ops
    from bitnet_c_amd.cache import PAGE
    from bitnet_c_amd.parts.position import rope_frequencies
    g = torch.Generator().manual_seed(R + rot)
    eps, col = 1e-5, 3 + qr
    rd = dict(base=5000.0, dims=rot)
    turn = pz.rotate_neighbours if interleaved else pz.rotate_halves
    pos = [0, 1, 63, 64, 300, -1, 2047]
    T = len(pos)
    x = torch.randn(T, col + R + rot + 2, generator=g).to(dtype)
    w, wq = 1 + 0.2 * torch.randn(R, generator=g), 1 + 0.2 * torch.randn(qr, generator=g)
    kw, vw = ops.latent_row_widths(R, rot)
    assert kw >= R + rot and vw >= R and (R, rot) != (120, 24) or (kw, vw) == (160, 128)
    kp = torch.full((40, 1, PAGE, kw), float("nan"), dtype=dtype, device=DEV)
    vp = torch.full((40, 1, vw, PAGE), float("nan"), dtype=dtype, device=DEV)
    table = i32([[(7 * j + 3) % 40 for j in range(33)]])
    inv = rope_frequencies(rot, rd["base"]).to(DEV) if rot else None
    cq = ops.latent_store(x.to(DEV), col, R, f32(w), eps, i32(pos), i32([0] * T), table, kp, vp, rot_dims=rot, inv_freq=inv,
                          interleaved=interleaved, row_widths=(kw, vw), query=(1, f32(wq)))
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert cq.dtype == dtype and rel_err(cq, pz.unit_rms(x[:, 1:1 + qr].double(), eps) * wq.double()) < tol
    live = [t for t, p in enumerate(pos) if p >= 0]
    c = pz.unit_rms(x[:, col:col + R].double(), eps) * w.double()
    for t in live:
        page, at = int(table[0, pos[t] // PAGE]), pos[t] % PAGE
        assert rel_err(kp[page, 0, at, :R], c[t]) < tol and rel_err(vp[page, 0, :R, at], c[t]) < tol
        assert float(kp[page, 0, at, R + rot:].abs().sum()) == 0.0 and float(vp[page, 0, R:, at].abs().sum()) == 0.0
        if rot:
            kr = turn(x[t:t + 1, col + R:col + R + rot].double().view(1, 1, rot), [pos[t]], rd, torch.float32)[0, 0]
            assert rel_err(kp[page, 0, at, R:R + rot], kr) < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [1, 5, 40])
@pytest.mark.parametrize("H,I,O,off,rot", [(3, 20, 24, 14, 8), (2, 44, 160, 120, 24), (2, 7, 9, 4, 4), (1, 96, 576, 512, 64)])
@pytest.mark.parametrize("interleaved", [True, False])
def test_a_product_per_head_whose_last_columns_turn(dtype, T, H, I, O, off, rot, interleaved):
    from bitnet_c_amd import ops
    from bitnet_c_amd.parts.position import rope_frequencies
    g = torch.Generator().manual_seed(T + O)
    x = torch.randn(T, H * I, generator=g).to(dtype)
    w = (torch.randn(H, I, O, generator=g) / math.sqrt(I)).to(dtype)
    pos = [(37 * t) % 500 for t in range(T)]
    if T > 1:
        pos[1] = -1                                                       # a padding row is left as it is
    rd = dict(base=700.0, dims=rot)
    y = torch.stack([x[:, h * I:(h + 1) * I].double() @ w[h].double() for h in range(H)], dim=1)
    turn = pz.rotate_neighbours if interleaved else pz.rotate_halves
    want = y.clone()
    live = [t for t in range(T) if pos[t] >= 0]
    want[live, :, off:off + rot] = turn(y[live][..., off:off + rot], [pos[t] for t in live], rd, torch.float32)
    got = ops.head_linear(x.to(DEV), w.to(DEV), rotate=(i32(pos), rope_frequencies(rot, rd["base"]).to(DEV), off, 1.0, interleaved))
    assert rel_err(got, want.reshape(T, -1)) < (1e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,kw,vw", [(4, 160, 128), (20, 192, 96), (3, 192, 192), (2, 576, 512), (17, 320, 258), (2, 50, 40)])
def test_one_wide_key_row_for_all_heads_with_sinks(dtype, H, kw, vw):
    """Attention of all query heads over one row per position, of the widths a latent beside a rotated part has, with a
    sink per head: one far below every score, one far above.  A key at every border of a page stands out for one query
    each, so that a key that is left out or counted for a neighbour shows; prompt and decoded, in one run and split."""
    from bitnet_c_amd import ops
    from bitnet_c_amd.cache import PAGE
    from bitnet_c_amd.engine.step import _query_tiles
    g = torch.Generator().manual_seed(H * 10 + kw)
    T, scale = 330, kw ** -0.5
    q = torch.randn(T, H, kw, generator=g)
    k = torch.randn(T, kw, generator=g)
    for i, key in ((329, 0), (328, 63), (300, 64), (200, 127), (150, 128), (64, 63), (65, 64), (40, 40)):
        q[i] = 3.0 * k[key]
    q, k = q.to(dtype), k.to(dtype)
    v = torch.randn(T, vw, generator=g).to(dtype)
    sink = torch.randn(H, generator=g)
    sink[0], sink[-1] = -80.0, 200.0
    want = torch.stack([pz.sink_weights((q[:, h].double() @ k.double().T) * scale, sink[h].double()) @ v.double() for h in range(H)], dim=1)
    assert float((want[329, 0] - v[0].double()).abs().max()) < 0.05 and float(want[:, -1].abs().max()) < 1e-3
    table = [5, 2, 7, 0, 3, 6]
    kp = torch.full((8, 1, PAGE, kw), float("nan"), dtype=dtype, device=DEV)
    vp = torch.full((8, 1, vw, PAGE), float("nan"), dtype=dtype, device=DEV)
    for b in range(6):
        n = min(PAGE, T - b * PAGE)
        kp[table[b], 0, :n] = k[b * PAGE:b * PAGE + n].to(DEV)
        vp[table[b], 0, :, :n] = v[b * PAGE:b * PAGE + n].T.to(DEV)
    bt, qd = i32([table]), q.reshape(T, H * kw).to(DEV)
    tol = 3e-5 if dtype == torch.float32 else 5e-2
    for mfma in [False] + ([True] if ops.attention_general_supported(dtype, kw, vw) else []):
        out = torch.empty(T, H * vw, dtype=dtype, device=DEV)
        if mfma:
            ops.attention_general_prompt(qd, out, kp, vp, bt, H, 1, kw, vw, scale, i32(_query_tiles([T], [0], ops.GENERAL_PROMPT_TILE)).reshape(-1, 4),
                                         sink=f32(sink))
        else:
            _, _, qt = ops.attention_row_shape(H, 1, False)
            ops.attention(qd, out, kp, vp, bt, H, 1, kw, scale, tiles=i32(_query_tiles([T], [0], qt)).reshape(-1, 4), qt=qt,
                          v_transposed=True, blocked=False, v_dim=vw, sink=f32(sink))
        assert rel_err(out, want.reshape(T, -1)) < tol, mfma
        for n in (T, T - 1, 65, 64, 1):
            for n_splits, chunk in ((1, 0), (3, 2 * PAGE)) if dtype == torch.bfloat16 else ((1, 0),):
                out = torch.empty(1, H * vw, dtype=dtype, device=DEV)
                if mfma:
                    ops.attention_general_decode(qd[n - 1:n], out, kp, vp, bt, i32([n]), H, 1, kw, vw, scale, n_splits=n_splits,
                                                 chunk=chunk, sink=f32(sink))
                else:
                    ops.attention(qd[n - 1:n], out, kp, vp, bt, H, 1, kw, scale, seq_lens=i32([n]), n_splits=n_splits, chunk=chunk,
                                  v_transposed=True, blocked=False, v_dim=vw, sink=f32(sink))
                assert rel_err(out, want[n - 1:n].reshape(1, -1)) < 2 * tol, (mfma, n, n_splits)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,I,K,D,T,groups", [(5, 1, 2, 64, 40, (3, 2)), (12, 4, 3, 48, 7, (4, 2)), (1, 1, 1, 32, 3, (2, 1)),
                                              (2, 6, 4, 40, 20, (4, 3)), (150, 42, 6, 40, 33, (96, 50)), (7, 0, 3, 72, 19, (7, 4)),
                                              (6, 2, 8, 24, 18, (1, 1)), (4, 4, 2, 50, 21, (2, 1))])
def test_choice_inside_the_best_groups_and_identity_experts(dtype, E, I, K, D, T, groups):
    """Groups rank by their best member's score with the correction, which is below 0 for most, so that a member of a
    group left out must not come in front of one that counts; the weights are the plain scores.  An identity expert hands
    the token's row on.  A pair at a time and (many rows, bfloat16) as grouped products."""
    from bitnet_c_amd import ops
    g = torch.Generator().manual_seed(E * 100 + D)
    F, R = 24, E + I
    h = torch.randn(T, D, generator=g).to(dtype)
    W = {"router": 3.0 * torch.randn(R, D, generator=g) / math.sqrt(D), "correction": 0.3 * torch.randn(R, generator=g) - 0.5}
    mlp = dict(router=dict(experts=E, identity=I, top=K, groups=dict(count=groups[0], keep=groups[1])))
    margins = []
    pick, w = pz.route(h.double(), {n: t.double() for n, t in W.items()}, "", mlp, margins)
    ids, wts = ops.moe_route(h.to(DEV), f32(W["router"]), K, "softmax", True, choice_bias=f32(W["correction"]), weight_floor=1e-20,
                             groups=groups)
    assert T < 7 or float((margins[0] > 1e-3).double().mean()) > 0.7
    for t in range(T):
        if float(margins[0][t]) > 1e-3:
            assert ids[t].tolist() == pick[t].tolist(), t
            assert rel_err(wts[t], w[t]) < 1e-5
    with pytest.raises(ops.KernelError):
        ops.moe_route(h.to(DEV), f32(W["router"]), K, "softmax", True, groups=(R, K - 1) if K > 1 else (R, 0))
    w_gate, w_up = (1.5 * torch.randn(E, F, D, generator=g) / math.sqrt(D)).to(dtype), (torch.randn(E, F, D, generator=g) / math.sqrt(D)).to(dtype)
    w_down = (torch.randn(E, D, F, generator=g) / math.sqrt(F)).to(dtype)
    want = torch.zeros(T, D, dtype=torch.float64)
    We = {f"e{e}.{n}": m[e].double() for e in range(E) for n, m in (("gate", w_gate), ("up", w_up), ("down", w_down))}
    for t in range(T):
        for j in range(K):
            e = int(ids[t, j])
            want[t] += float(wts[t, j]) * (pz.expert(h[t:t + 1].double(), We, f"e{e}.")[0] if e < E else h[t].double())
    assert I == 0 or int((ids >= E).sum()) > 0
    unit = ops.ClampedUnit(float("inf"), 1.0, 0.0)
    stacked = torch.cat([w_gate, w_up], dim=1).contiguous().to(DEV)
    tol = 1e-5 if dtype == torch.float32 else 3e-2
    y = ops.moe_experts(h.to(DEV), stacked, w_down.to(DEV), ids, wts, "silu", False, gated=unit)
    assert rel_err(y.slabs.sum(0), want) < tol
    if ops.moe_grouped_supported(T, D, F, dtype):
        y = ops.moe_experts_grouped(h.to(DEV), stacked, w_down.to(DEV), ids, wts, "silu", False, gated=unit)
        assert rel_err(y.slabs.sum(0), want) < tol
        every = torch.full_like(ids, E)                                   # a step whose tokens all chose identity experts
        y = ops.moe_experts_grouped(h.to(DEV), stacked, w_down.to(DEV), every, wts, "silu", False, gated=unit)
        assert rel_err(y.slabs.sum(0), h.double() * wts.double().cpu().sum(1, keepdim=True)) < tol


# ------------------------------------------------------------------------------------------------------------------
# whole models through the engine
# ------------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompts_and_the_stream_after_every_layer(folders, name, dtype):
    """Every position of a prompt in one step, and the residual stream behind every layer run; the first tokens of the
    sequence and a page's border are among them."""
    import bitnet_c_amd as bn
    folder = folders(name)
    toks = settled_tokens(folder, 75, 1)
    layers = []
    want = pz.forward(pz.read_config(folder), pz.read_weights(folder), toks, layers)
    eng = engine(folder, dtype)
    s = eng.new_sequence()
    close(eng.step([bn.StepEntry(s, toks, list(range(75)))]), want, dtype)
    eng.release(s)
    got = []
    eng.tap = lambda point, entry, stream, ctx: got.append(stream.flush().clone()) if point == "layer_out" else None
    s = eng.new_sequence()
    close(eng.step([bn.StepEntry(s, toks, [74])]), want[74:], dtype)
    assert len(got) == len(layers)
    for a, b in zip(got, layers):
        close(a, b, dtype)


@pytest.mark.parametrize("graphs", [True, False])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prefill_against_decoding_token_by_token(folders, name, dtype, graphs):
    """A shorter prompt, then token by token across a page's border, in a slot that was used before; a sequence decoded
    from its first token on."""
    import bitnet_c_amd as bn
    folder = folders(name)
    toks = settled_tokens(folder, 75, 1)
    want = plain(folder, toks)
    eng = engine(folder, dtype, use_graphs=graphs)
    s = eng.new_sequence()
    whole = eng.step([bn.StepEntry(s, toks, list(range(75)))])
    eng.release(s)
    s = eng.new_sequence()
    got = torch.cat([eng.step([bn.StepEntry(s, toks[:58], list(range(58)))])]
                    + [eng.step([bn.StepEntry(s, [t], [0])]) for t in toks[58:]])
    close(got, want, dtype)
    if dtype == torch.float32:
        assert rel_err(got, whole) < 2e-5
    one = eng.new_sequence()
    close(eng.step([bn.StepEntry(one, toks[:1], [0])]), want[:1], dtype)
    close(torch.cat([eng.step([bn.StepEntry(one, [t], [0])]) for t in toks[1:6]]), want[1:6], dtype)
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,portions", [("A", (2, 3, 5, 2, 17, 1, 40, 2)), ("B", (1, 2, 2, 2, 64, 1)), ("C", (63, 2, 2, 5)),
                                           ("D", (2,) * 12)])
def test_portions_of_several_sizes(folders, name, portions, dtype):
    import bitnet_c_amd as bn
    folder = folders(name)
    n = sum(portions)
    toks = settled_tokens(folder, n, 1)
    want = plain(folder, toks)
    eng = engine(folder, dtype)
    s, at, parts = eng.new_sequence(), 0, []
    for p in portions:
        parts.append(eng.step([bn.StepEntry(s, toks[at:at + p], list(range(p)))]))
        at += p
    close(torch.cat(parts), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_unequal_batches_and_slots_used_again(folders, name, dtype):
    """Requests of unequal lengths start together and are decoded together; the shorter ones end, their slots and pages go
    to new requests while a neighbour lives on; every request against itself alone (the plain implementation)."""
    import bitnet_c_amd as bn
    folder = folders(name)
    eng = engine(folder, dtype, max_tokens=768)
    keep = eng.new_sequence()
    eng.step([bn.StepEntry(keep, settled_tokens(folder, 9, 1), [])])
    for i in range(3):
        reqs = [settled_tokens(folder, n, 1 + (i + k) % 3) for k, n in enumerate((66 + i, 20 - i, 1 + 2 * i))]
        slots = [eng.new_sequence() for _ in reqs]
        heads = [max(1, len(r) - 3) for r in reqs]
        out = eng.step([bn.StepEntry(s, r[:n], [0, n - 1]) for s, r, n in zip(slots, reqs, heads)])
        for k, (r, n) in enumerate(zip(reqs, heads)):
            close(out[2 * k:2 * k + 2], plain(folder, r)[[0, n - 1]], dtype)
        live = list(zip(slots, reqs, heads))
        while any(at < len(r) for _, r, at in live):
            now = [(s, r, at) for s, r, at in live if at < len(r)]
            o = eng.step([bn.StepEntry(s, [r[at]], [0]) for s, r, at in now])
            for k, (s, r, at) in enumerate(now):
                close(o[k:k + 1], plain(folder, r)[at:at + 1], dtype)
            live = [(s, r, at + 1) for s, r, at in live]
        for s in slots[i % 2:]:
            eng.release(s)
    toks = settled_tokens(folder, 10, 1)
    close(eng.step([bn.StepEntry(keep, toks[9:], [0])]), plain(folder, toks)[-1:], dtype)
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_prompt_and_decode_steps_replayed_from_graphs(folders, name, dtype):
    """The same bucket of prompt steps and of decode steps again and again, with other sequences in it and other work
    between the replays: every replay is the plain result."""
    import bitnet_c_amd as bn
    folder = folders(name)
    eng = engine(folder, dtype)
    for i in range(4):
        n = 33 + 7 * (i % 3)
        toks = settled_tokens(folder, n + 3, 1 + i % 3)
        want = plain(folder, toks)
        s = eng.new_sequence()
        close(eng.step([bn.StepEntry(s, toks[:n], [0, n - 1])]), want[[0, n - 1]], dtype)
        torch.cuda.synchronize()
        torch.randn(1000, device=DEV).sum().item()
        for t in range(n, n + 3):
            close(eng.step([bn.StepEntry(s, [toks[t]], [0])]), want[t:t + 1], dtype)
        if i % 2:
            eng.release(s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_step_that_mixes_single_tokens_and_portions(folders, dtype):
    import bitnet_c_amd as bn
    folder = folders("A")
    eng = engine(folder, dtype)
    a, b, c = (settled_tokens(folder, n, 1 + i) for i, n in enumerate((30, 70, 12)))
    sa, sb, sc = (eng.new_sequence() for _ in range(3))
    eng.step([bn.StepEntry(sa, a[:29], []), bn.StepEntry(sb, b[:10], [])])
    out = eng.step([bn.StepEntry(sa, a[29:], [0]), bn.StepEntry(sb, b[10:], [0, 59]), bn.StepEntry(sc, c, [11])])
    close(out, torch.stack([plain(folder, a)[29], plain(folder, b)[10], plain(folder, b)[69], plain(folder, c)[11]]), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,rot", [(12, 4), (112, 16)])
def test_long_decoding_with_far_keys_and_slow_decays(tmp_path, dtype, rank, rot):
    """A model whose attention is peaked (a large scale: single far keys carry a query's result, and where none does the
    sink takes the weight) and whose decays stay next to 1: a prompt of many pages in portions, then 70 decoded tokens."""
    import bitnet_c_amd as bn
    cfg = _model(61, 32, 1e-5, 2.0, 20.0, [
        _lat(2, 8, rot, 8, rank, 6, 1.2, 1000.0, None), _ret(2, 8, 12, (10000.0, 8), None, decay=[0.999, 0.9999]),
        _lat(2, 8, rot, 8, rank, 6, 1.2, 1000.0, None, weights_of=0)])
    folder = write_folder(tmp_path / "peaked", cfg, 9)
    toks = torch.randint(0, 61, (700,), generator=torch.Generator().manual_seed(2)).tolist()     # no experts: no close calls
    want = pz.forward(pz.read_config(folder), pz.read_weights(folder), toks, angle_dtype=torch.float32)
    eng = engine(folder, dtype, max_tokens=2048)
    s, at, parts = eng.new_sequence(), 0, []
    check = [0, 1, 2, 3, 15, 16, 17, 63, 64, 65, 299, 300, 301, 511, 512, 629]
    for n in (300, 257, 73):
        w = [p - at for p in check if at <= p < at + n]
        parts.append(eng.step([bn.StepEntry(s, toks[at:at + n], w)]))
        at += n
    close(torch.cat(parts), want[check], dtype)
    dec = torch.cat([eng.step([bn.StepEntry(s, [toks[t]], [0])]) for t in range(at, 700)])
    close(dec, want[at:], dtype)
    s2 = eng.new_sequence()
    whole = eng.step([bn.StepEntry(s2, toks, list(range(at, 700)))])
    assert rel_err(dec, whole) < (1e-4 if dtype == torch.float32 else BF16_ELEMENT)
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_sink_takes_the_weight_that_no_key_claims(tmp_path, dtype):
    """Sinks from far below every score to far above: with the largest a layer adds nothing through that head, and the sink
    counts once, unscaled, whatever the scale of the scores is."""
    import bitnet_c_amd as bn
    cfg = _model(47, 32, 1e-5, 1.0, 9.0, [_lat(4, 8, 4, 8, 24, 12, 0.05, 100.0, None)])
    folder = write_folder(tmp_path / "sinks", cfg, 3, overrides={"l0.mix.sink": torch.tensor([-30.0, 0.5, 3.0, 40.0])})
    toks = torch.randint(0, 47, (80,), generator=torch.Generator().manual_seed(1)).tolist()
    want = plain(folder, toks)
    other = pz.read_weights(folder)
    other["l0.mix.sink"] = other["l0.mix.sink"] * 0.05                       # a sink that were scaled like the scores
    assert rel_err(pz.forward(pz.read_config(folder), other, toks), want) > 0.05
    eng = engine(folder, dtype)
    s = eng.new_sequence()
    got = eng.step([bn.StepEntry(s, toks[:70], list(range(70)))])
    dec = torch.cat([eng.step([bn.StepEntry(s, [t], [0])]) for t in toks[70:]])
    close(torch.cat([got, dec]), want, dtype, bf16_rows=0.02)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,rot", [(512, 64), (192, 64), (160, 32)])
def test_wide_latents_beside_their_rotated_parts(tmp_path, dtype, rank, rot):
    """Key rows of up to 576 and values of up to 512 numbers.  A prompt across a page's border, then decoded."""
    import bitnet_c_amd as bn
    cfg = _model(59, 64, 1e-5, 2.0, 15.0, [_lat(3, 16, rot, 24, rank, 40, 0.11, 100000.0, None)])
    folder = write_folder(tmp_path / "wide", cfg, 6)
    toks = torch.randint(0, 59, (90,), generator=torch.Generator().manual_seed(4)).tolist()
    want = plain(folder, toks)
    eng = engine(folder, dtype)
    s = eng.new_sequence()
    got = eng.step([bn.StepEntry(s, toks[:70], list(range(70)))])
    dec = torch.cat([eng.step([bn.StepEntry(s, [t], [0])]) for t in toks[70:]])
    close(torch.cat([got, dec]), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_logits_do_not_depend_on_the_cut_or_the_batch(folders, name, dtype):
    """Whole, in portions, one by one and beside other requests: float32 logits agree to the last bits, bfloat16 within its
    rounding (steps of few rows and of many take different kernels for the products and the experts)."""
    import bitnet_c_amd as bn
    folder = folders(name)
    eng = engine(folder, dtype)
    toks, other = settled_tokens(folder, 75, 1), settled_tokens(folder, 37, 3)
    s = eng.new_sequence()
    whole = eng.step([bn.StepEntry(s, toks, list(range(75)))])
    eng.release(s)
    s, o = eng.new_sequence(), eng.new_sequence()
    a = eng.step([bn.StepEntry(o, other, []), bn.StepEntry(s, toks[:37], list(range(37)))])
    b = eng.step([bn.StepEntry(s, toks[37:74], list(range(37)))])
    c = eng.step([bn.StepEntry(s, toks[74:], [0]), bn.StepEntry(o, [5], [])])
    got = torch.cat([a, b, c])
    if dtype == torch.float32:
        assert rel_err(got, whole) < 2e-5
    else:
        close(got, whole.double(), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_greedy_generation_through_the_entry_point(folders, name, dtype):
    """Greedy generation through load() and generate(), the scheduler batching three prompts two at a time.  Every token
    that was chosen holds, where it was chosen, the plain implementation's largest logit within rounding (up to the first
    close expert choice of the sequence that the engine itself wrote)."""
    import bitnet_c_amd as bn
    folder = folders(name)
    llm = bn.load(folder, dtype="float32" if dtype == torch.float32 else "bfloat16", max_tokens=1024)
    prompts = [settled_tokens(folder, n, 1 + i) for i, n in enumerate((5, 66, 1))]
    got = llm.generate(prompts, max_new_tokens=12, temperature=0.0, stop_ids=(), batch_size=2)
    cfg, W = pz.read_config(folder), pz.read_weights(folder)
    for p, g in zip(prompts, got):
        assert len(g) == 12
        margins = []
        logits = pz.forward(cfg, W, p + g, margins=margins)[len(p) - 1:-1]
        settled = 0
        while settled < 12 and margins[len(p) + settled - 1] >= (1e-3 if dtype == torch.float32 else 0.05):
            settled += 1
        rms = float(logits.pow(2).mean().sqrt())
        for i, tok in enumerate(g[:settled]):
            gap = float(logits[i].max() - logits[i, tok])
            # bfloat16: an element of a row may be off by as much as BF16_ELEMENT of the rows' size (see TOL), on either token
            assert gap <= (1e-4 if dtype == torch.float32 else BF16_ELEMENT) * rms, (i, gap / rms)
    llm.engine.cache.check()
    assert llm.engine.cache.live_slots() == []


def test_command_line_and_trace_replay(folders, tmp_path):
    """The command line generates from a Zenasun folder (also one that it writes itself from a configuration file, with
    random weights), and the trace replay program steps one through a batch of prompts and single tokens."""
    import subprocess
    import sys
    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder = folders("D")
    cfg, W = pz.read_config(folder), pz.read_weights(folder)
    prompt = settled_tokens(folder, 8, 1)
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "bitnet"), folder, "--prompt-token-ids", ",".join(map(str, prompt)),
                        "-n", "6", "--repeat-penalty", "1.0", "--fp32", "--token-ids", "--quiet"], capture_output=True, text=True,
                       timeout=300)
    assert p.returncode == 0, p.stderr[-1500:]
    ids = [int(x) for x in [l for l in p.stderr.splitlines() if l and l[0].isdigit()][0].split(",")]
    margins = []
    logits = pz.forward(cfg, W, prompt + ids, margins=margins)[len(prompt) - 1:-1]
    for i, tok in enumerate(ids):
        if min(margins[:len(prompt) + i]) < 1e-3:
            break
        assert float(logits[i].max() - logits[i, tok]) <= 1e-4 * float(logits.pow(2).mean().sqrt())
    conf = tmp_path / "conf.json"
    conf.write_text(json.dumps(CONFIGS["B"]))
    made = str(tmp_path / "made")
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "bitnet"), made, "--random", str(conf), "--seed", "4",
                        "--prompt-token-ids", "1,2,3", "-n", "4", "--fp32", "--token-ids", "--quiet", "--repeat-penalty", "1.0"],
                       capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-1500:]
    assert len([l for l in p.stderr.splitlines() if l and l[0].isdigit()][0].split(",")) == 4
    assert pz.read_config(made)["layers"][2] == CONFIGS["B"]["layers"][2] and pz.read_config(made)["logit_softcap"] == 40.0
    folder = folders("A")
    a, b = settled_tokens(folder, 40, 2), settled_tokens(folder, 7, 3)
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
