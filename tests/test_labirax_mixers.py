"""The mechanisms of the Labirax design one at a time, each op of the
package against the plain functions of tests/labirax_oracle.py or a closed
form: layer norms around a sub-layer on the f32 stream, the gated linear
recurrence with its low-rank decay, windowed latent attention with a value
gate (latent and expanded forms), attention with a distance bias and a query
temperature (row, vector and matrix-core kernels), window edges, bucket
borders and far keys made visible by one dominant score, the router and its
experts, the logits' soft cap. CPU runs check the reference ops; `-m gpu`
runs the HIP kernels in f32 and bf16."""
import math
import os
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import labirax_oracle as L  # noqa: E402

from kaito_amd import ops  # noqa: E402

MODES = [("cpu", torch.float32),
         pytest.param(("cuda", torch.float32), marks=pytest.mark.gpu),
         pytest.param(("cuda", torch.bfloat16), marks=pytest.mark.gpu)]
BS = 16      # page size used here


def i32(x, dev):
    return torch.tensor(x, dtype=torch.int32, device=dev)


def f32(x, dev):
    return torch.tensor(np.asarray(x), dtype=torch.float32, device=dev)


def close(got, want, dtype, scale=None, tight=1e-5, bf16=2e-2):
    want = torch.as_tensor(np.asarray(want), dtype=torch.float64)
    scale = scale if scale is not None else want.abs().max().item() + 1e-9
    err = (got.double().cpu() - want).abs().max().item() / scale
    assert err < (tight if dtype == torch.float32 else bf16), err


def act(a, mode):
    """Values as the activation dtype holds them: (device tensor, float64
    copy of what it holds)."""
    dev, dt = mode
    t = torch.tensor(np.asarray(a), dtype=torch.float32).to(dt).to(dev)
    return t, t.double().cpu().numpy()


# ---- layer norms on the f32 stream --------------------------------------------------

def norm_pair(rng, width, dev):
    w = np.float32(rng.uniform(0.3, 1.8, width))
    b = np.float32(rng.normal(0, 0.7, width))
    return (w.astype(np.float64), b.astype(np.float64)), (f32(w, dev),
                                                          f32(b, dev))


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("width", [20, 75, 256, 1028, 2052, 8196])
def test_sandwich_step(mode, width):
    """x += ln(y + y2), then the next input ln(x): f32 and rounded addends,
    one or two of them, strided views, a stream far from zero mean, with and
    without a next norm."""
    dev, dt = mode
    rng = np.random.default_rng(width)
    T, eps = 5, 1e-3
    (wb, bb), (wbt, bbt) = norm_pair(rng, width, dev)
    (wa, ba), (wat, bat) = norm_pair(rng, width, dev)
    x0 = np.float32(rng.normal(0, 3, (T, width)) + 40.0)
    wide, wide64 = act(rng.normal(0.5, 0.2, (T, width + 4)), mode)
    y, y64 = wide[:, 4:], wide64[:, 4:]
    y2, y264 = act(rng.normal(0, 0.3, (T, width)), mode)
    yf = np.float32(rng.normal(-2, 0.1, (T, width)))
    cases = [(y, y64, None, 0.0), (f32(yf, dev), yf, y2, y264),
             (f32(yf, dev), yf, None, 0.0), (y, y64, y2, y264)]
    for yt, yv, second, sv in cases:
        for follow in (True, False):
            x = f32(x0, dev)
            h = ops.sandwich_norm_residual(
                x, yt, wbt, bbt, wat if follow else None,
                bat if follow else None, eps, dt, y2=second)
            want = x0 + L.layer_norm(yv + sv, wb, bb, eps)
            close(x, want, torch.float32, tight=1e-6)
            if follow:
                assert h.dtype == dt
                # the oracle's norm of the stream as the op stored it
                close(h, L.layer_norm(x.double().cpu().numpy(), wa, ba, eps),
                      dt, tight=2e-5, bf16=1e-2)
            else:
                assert h is None


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("width", [30, 256, 2050, 4096])
def test_embedding_and_output_norm(mode, width):
    dev, dt = mode
    rng = np.random.default_rng(width)
    (w, b), (wt, bt) = norm_pair(rng, width, dev)
    table, t64 = act(rng.normal(0.3, 1, (40, width)), mode)
    ids = torch.tensor([3, 0, 39, 3], device=dev)
    x, h = ops.embed_layer_norm(ids, table, 0.37, wt, bt, 1e-4)
    want = t64[[3, 0, 39, 3]] * 0.37
    close(x, want, torch.float32, tight=1e-6)
    close(h, L.layer_norm(want, w, b, 1e-4), dt, bf16=1e-2)
    out = ops.layer_norm_cast(x, wt, bt, 1e-4, dt)
    assert out.dtype == dt
    close(out, L.layer_norm(want, w, b, 1e-4), dt, bf16=1e-2)


@pytest.mark.parametrize("mode", MODES)
def test_norm_of_a_strided_view(mode):
    """The query latent's norm reads its columns of the fused projection."""
    dev, dt = mode
    rng = np.random.default_rng(0)
    p, p64 = act(rng.normal(0, 1, (6, 50)), mode)
    w = np.float32(rng.uniform(0.5, 1.5, 19))
    got = ops.rms_norm_cast(p[:, 7:26], f32(w, dev), 1e-4, dt)
    close(got, L.rms(p64[:, 7:26], 1e-4) * w, dt, bf16=1e-2)


@pytest.mark.parametrize("mode", MODES[:2])
@pytest.mark.parametrize("shape", [(3, 52), (1, 7), (5, 1001)])
def test_scaled_softcap(mode, shape):
    dev, _ = mode
    a = np.float32(np.random.default_rng(1).normal(0, 30, shape))
    got = ops.scaled_softcap(f32(a, dev), 1.7, 12.0)
    close(got, 12 * np.tanh(a.astype(np.float64) * 1.7 / 12), torch.float32)
    close(ops.scaled_softcap(f32(a, dev), 0.5, 0.0), a * 0.5, torch.float32)


# ---- gated linear attention ----------------------------------------------------------

def gla_inputs(rng, T, H, D, V, R, mode, packed=True):
    q, q64 = act(rng.normal(0, 1, (T, H * D)), mode)
    k, k64 = act(rng.normal(0, 1, (T, H * D)), mode)
    v, v64 = act(rng.normal(0, 1, (T, H * V)), mode)
    g, g64 = act(rng.normal(0, 1, (T, H * V)), mode)
    low = np.float32(rng.normal(0, 1, (T, R)))
    a2 = np.float32(rng.normal(0, 1.5, (R, H * D)))
    ab = np.float32(rng.normal(1, 2, H * D))
    nw = np.float32(rng.uniform(0.5, 1.5, V))
    return torch.cat([q, k, v, g], 1), (q64, k64, v64, g64), low, a2, ab, nw


def gla_want(parts, low, a2, ab, nw, H, D, V, tau, eps):
    q, k, v, g = parts
    T = q.shape[0]
    alpha = L.sigmoid(low.astype(np.float64) @ a2 + ab) ** (1.0 / tau)
    o, S = L.gla_recurrence(q.reshape(T, H, D) * D ** -0.5,
                            k.reshape(T, H, D), v.reshape(T, H, V),
                            alpha.reshape(T, H, D))
    o = L.rms(o, eps) * nw * L.silu(g.reshape(T, H, V))
    return o.reshape(T, H * V), S


def gla_call(rows, low, a2, ab, nw, H, D, V, tau, eps, state, chunks, dev):
    """chunks: (rows, slot, start) in row order."""
    n = [c[0] for c in chunks]
    cu = i32([0] + list(np.cumsum(n)), dev)
    nq, nv = H * D, H * V
    return ops.gla_scan(
        rows[:, :nq].unflatten(-1, (H, D)),
        rows[:, nq:2 * nq].unflatten(-1, (H, D)),
        rows[:, 2 * nq:2 * nq + nv].unflatten(-1, (H, V)),
        rows[:, 2 * nq + nv:].unflatten(-1, (H, V)), low, f32(a2, dev),
        f32(ab, dev), tau, D ** -0.5, f32(nw, dev), state, cu,
        i32([c[1] for c in chunks], dev), i32([c[2] for c in chunks], dev),
        eps)


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("rows_per_lane", ["16", "32"])
@pytest.mark.parametrize("sizes", [(3, 8, 20, 1), (2, 32, 80, 5),
                                   (1, 72, 9, 16), (1, 200, 33, 3),
                                   (2, 128, 16, 8)])
def test_gla_portions_and_batches(mode, sizes, rows_per_lane, monkeypatch):
    """Portions down to one token carry the state in a slot that held
    something else, beside a padding chunk; then two sequences in one step."""
    monkeypatch.setenv("KAITO_DIAG_ROWS_PER_LANE", rows_per_lane)
    dev, dt = mode
    if dev == "cpu" and rows_per_lane == "32":
        pytest.skip("the reference op has no tiling")
    H, D, V, R = sizes
    rng = np.random.default_rng(D + V)
    T, tau, eps = 23, 6.0, 1e-4
    rows, parts, low, a2, ab, nw = gla_inputs(rng, T, H, D, V, R, mode)
    want, S = gla_want(parts, low, a2, ab, nw, H, D, V, tau, eps)
    lowt = f32(low, dev)
    args = (a2, ab, nw, H, D, V, tau, eps)
    state = torch.full((3, H, D, V), -2.0, dtype=torch.float32, device=dev)
    out, at = [], 0
    for n in (1, 6, 2, 1, 13):
        r = torch.cat([rows[at:at + n], rows[:1]], 0)
        lw = torch.cat([lowt[at:at + n], lowt[:1]], 0)
        out.append(gla_call(r, lw, *args, state, [(n, 1, at), (1, -1, 0)],
                            dev)[:n])
        at += n
    close(torch.cat(out), want, dt, tight=5e-5, bf16=2e-2)
    close(state[1], S, torch.float32, tight=1e-4)
    assert state[0].eq(-2.0).all()
    # a second sequence (the same rows from the fifth on) beside the first,
    # slots 0 and 2 starting stale
    w2, _ = gla_want(tuple(p[4:] for p in parts), low[4:], *args[:3], H, D, V,
                     tau, eps)
    r = torch.cat([rows[4:], rows], 0)
    y = gla_call(r, torch.cat([lowt[4:], lowt], 0), *args, state,
                 [(T - 4, 2, 0), (T, 0, 0)], dev)
    close(y, np.concatenate([w2, want]), dt, tight=5e-5, bf16=2e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
def test_gla_many_tokens(dt):
    """A prompt-sized step (several tokens per prep wave, a ragged last one)
    against the reference op."""
    H, D, V, R, T = 32, 16, 32, 7, 517
    rng = np.random.default_rng(2)
    mode = ("cuda", dt)
    rows, _, low, a2, ab, nw = gla_inputs(rng, T, H, D, V, R, mode)
    outs, states = [], []
    for dev in ("cuda", "cpu"):
        state = torch.zeros(2, H, D, V, device=dev)
        outs.append(gla_call(rows.to(dev), f32(low, dev), a2, ab, nw, H, D, V,
                             16.0, 1e-5, state,
                             [(300, 1, 0), (217, 0, 0)], dev).float().cpu())
        states.append(state.cpu())
    close(outs[0], outs[1], dt, bf16=2e-2, tight=2e-4)
    close(states[0], states[1], torch.float32, tight=1e-4)


@pytest.mark.parametrize("mode", MODES)
def test_gla_keeps_a_far_token(mode):
    """Slow decays: the first token's write, read 400 tokens later through
    its own key, dominates; with a fast channel it is gone."""
    dev, dt = mode
    H, D, V, T = 1, 8, 4, 400
    rng = np.random.default_rng(5)
    q, k = np.zeros((T, D)), np.zeros((T, D))
    v = rng.normal(0, 0.02, (T, V))
    k[:, 3] = 0.05
    k[0, 2], v[0], q[:, 2] = 8.0, [1, -1, 2, 0.5], 1.0
    g = np.full((T, V), 3.0)
    for bias, kept in ((12.0, True), (-12.0, False)):
        ab = np.full(D, 12.0, dtype=np.float32)
        ab[2] = bias
        rows, r64 = act(np.concatenate([q, k, v, g], 1), mode)
        low, a2 = np.zeros((T, 1), np.float32), np.zeros((1, D), np.float32)
        nw = np.ones(V, np.float32)
        parts = (r64[:, :D], r64[:, D:2 * D], r64[:, 2 * D:2 * D + V],
                 r64[:, 2 * D + V:])
        want, _ = gla_want(parts, low, a2, ab, nw, H, D, V, 16.0, 1e-9)
        state = torch.zeros(1, H, D, V, device=dev)
        y1 = gla_call(rows[:399], f32(low[:399], dev), a2, ab, nw, H, D, V,
                      16.0, 1e-9, state, [(399, 0, 0)], dev)
        y2 = gla_call(rows[399:], f32(low[399:], dev), a2, ab, nw, H, D, V,
                      16.0, 1e-9, state, [(1, 0, 399)], dev)
        close(torch.cat([y1, y2])[-5:], want[-5:], dt, tight=1e-4)
        if kept:
            first = v[0] / np.sqrt(np.mean(v[0] ** 2)) * L.silu(3.0)
            close(y2[0], first, dt, tight=1e-3, bf16=3e-2)


def gla_module(mx, W, mode, width, eps):
    from kaito_amd.models.hybrid_config import GLASpec
    from kaito_amd.models.mixers import GLAMixer
    dev, dt = mode
    m = GLAMixer(width, GLASpec(**mx), dt, eps).to(dev)
    m.set_decay_rank(W["m.a1"].shape[0])
    with torch.no_grad():
        m.in_proj.copy_(torch.cat([f32(W["m." + n], dev) for n in "qkvg"], 0))
        m.a1.copy_(f32(W["m.a1"], dev))
        m.a2.copy_(f32(W["m.a2"], dev).t())
        m.a_bias.copy_(f32(W["m.a2.b"], dev))
        m.out_norm.copy_(f32(W["m.norm"], dev))
        m.o_proj.copy_(f32(W["m.o"], dev))
    return m


def mixer_weights(layer, width, seed, **kw):
    cfg = L.make_config([layer], width, 8)
    W = L.random_weights(cfg, seed, **kw)
    return {"m." + k[len("l0.mix."):]: v for k, v in W.items()
            if k.startswith("l0.mix.")}


def in_portions(m, ht, mode, sizes, tiled=True):
    """Rows ht through mixer m in portions, pages out of order, a state
    slot that is not the first."""
    dev, _ = mode
    cache = m.alloc_cache(10, BS, 3, dev)
    for t in cache.values():
        t.fill_(3.0)                                  # stale contents
    bt = i32([[6, 1, 4, 2, 9, 0]], dev)
    out, at = [], 0
    for c in sizes:
        pos = torch.arange(at, at + c, device=dev)
        ts, tq = ops.build_query_tiles([c], dev)
        meta = SimpleNamespace(
            cu_seqlens=i32([0, c], dev), state_slots=i32([1], dev),
            seq_starts=i32([at], dev), token_seq=i32([0] * c, dev),
            block_tables=bt, slot_mapping=(
                bt[0].long()[pos // BS] * BS + pos % BS),
            tile_seq=ts if c > 1 and tiled else None, tile_qbase=tq,
            ctx_lens=[at + c], ctx_starts=[at], layer_shared={})
        out.append(m(ht[at:at + c].contiguous(), pos, cache, meta))
        at += c
    return torch.cat(out, 0)


PORTIONS = ([61], [1] * 61, [2, 17, 1, 2, 30, 9], [33, 2, 2, 24])


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("dim,vdim,rank,tau", [(20, 12, 3, 4.0),
                                               (32, 64, 12, 12.0)])
def test_gla_mixer_in_portions(mode, dim, vdim, rank, tau):
    dev, dt = mode
    layer = L.gla_layer(3, dim, vdim, tau)
    W = mixer_weights(layer, 48, dim, decay_rank=rank)
    m = gla_module(layer["mixer"], W, mode, 48, 1e-4)
    ht, h = act(np.random.default_rng(1).normal(0, 1, (61, 48)), mode)
    want = L.gla(h, W, "m.", layer["mixer"], 1e-4)
    for sizes in PORTIONS:
        close(in_portions(m, ht, mode, sizes), want, dt, tight=1e-4,
              bf16=3e-2)


# ---- attention with a distance bias ---------------------------------------------------

def test_bias_table_by_distance():
    """The spread-out table holds the bucket's value at every distance, and
    its last entry every larger one's."""
    from kaito_amd.models.hybrid_config import distance_bias_table
    for buckets, far in ((8, 20), (16, 100), (10, 6), (32, 128), (2, 5),
                         (7, 50), (64, 2000)):
        rel = torch.arange(buckets * 3).view(buckets, 3).to(torch.bfloat16)
        table = distance_bias_table(rel, far)
        assert table.shape == (3, far + 1) and table.dtype == torch.float32
        for n in list(range(far + 1)) + [far + 1, 5 * far]:
            row = L.bucket(n, buckets, far)
            assert torch.equal(table[:, min(n, far)], rel[row].float())
        assert L.bucket(far, buckets, far) == buckets - 1
    with pytest.raises(ValueError):
        distance_bias_table(torch.zeros(16, 2), 8)


def paged(k, v, mode, rng, spare=2):
    """Keys [n, G, D] and values into shuffled pages; the rest of the pool
    holds stale rows of large numbers."""
    dev, dt = mode
    n, G, D = k.shape
    pages = -(-n // BS)
    perm = rng.permutation(pages + spare)[:pages]
    kc = torch.full((pages + spare, G, BS, D), 40.0, dtype=dt)
    vc = torch.full((pages + spare, G, BS, v.shape[2]), 40.0, dtype=dt)
    for j in range(n):
        kc[perm[j // BS], :, j % BS] = torch.as_tensor(k[j]).to(dt)
        vc[perm[j // BS], :, j % BS] = torch.as_tensor(v[j]).to(dt)
    return kc.to(dev), vc.to(dev), i32([perm.tolist()], dev)


def run_attention(q, kc, vc, bt, pos0, mode, scale, table, temp=(0.0, 1),
                  tiled=False, window=0):
    """Rows q at positions pos0.. through the paged kernels; the chunk is
    one portion (tiled: with query tiles, as prompt steps hand them)."""
    dev, dt = mode
    n = q.size(0)
    pos = torch.arange(pos0, pos0 + n, device=dev)
    tiles = None
    if tiled:
        ts, tq = ops.build_query_tiles([n], dev)
        tiles = (ts, tq, i32([0, n], dev), i32([pos0], dev))
    return ops.window_attention(
        q, kc, vc, bt, i32([0] * n, dev), pos, scale, tiles=tiles,
        window=window, dist_bias=f32(table, dev), temp_coef=temp[0],
        temp_every=temp[1])


def biased(q, k, v, scale, table, temp, window=10 ** 9):
    T, H, _ = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        lo = max(0, i - window + 1)
        for n in range(H):
            g = n // (H // k.shape[1])
            s = (k[lo:i + 1, g] @ q[i, n]) * scale \
                * L.temperature(i, temp[0], temp[1])
            d = np.minimum(i - np.arange(lo, i + 1), table.shape[1] - 1)
            out[i, n] = L.softmax(s + table[n, d]) @ v[lo:i + 1, g]
    return out


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("heads,kv,dim,vdim,entries,temp,window", [
    (6, 3, 64, 64, 21, (0.3, 16), 0), (4, 4, 24, 40, 1, (0.0, 1), 0),
    (5, 1, 32, 16, 200, (0.5, 1), 0), (8, 1, 128, 32, 33, (0.2, 50), 0),
    (2, 2, 18, 10, 65, (1.0, 7), 0), (3, 1, 64, 128, 64, (0.3, 1000), 0),
    (16, 1, 64, 32, 47, (0.3, 8), 29)])
def test_attention_with_distance_bias(mode, heads, kv, dim, vdim, entries,
                                      temp, window):
    """Whole sequences, later portions and single rows, with and without
    query tiles: sizes of the matrix-core kernel, of the vector kernel and
    of neither; tables of one entry, shorter and longer than the sequence;
    the bias unlike at every distance."""
    dev, dt = mode
    rng = np.random.default_rng(heads * 100 + entries)
    n, scale = 139, 0.3
    qt, q = act(rng.normal(0, 1, (n, heads, dim)), mode)
    _, k = act(rng.normal(0, 1, (n, kv, dim)), mode)
    _, v = act(rng.normal(0, 1, (n, kv, vdim)), mode)
    table = np.float32(rng.normal(0, 2.0, (heads, entries)))
    want = biased(q, k, v, scale, table, temp, window or 10 ** 9)
    kc, vc, bt = paged(k, v, mode, rng)
    size = np.abs(want).max()
    for tiled in (False, True):
        for at in (0, 41, 130):
            got = run_attention(qt[at:].contiguous(), kc, vc, bt, at, mode,
                                scale, table, temp, tiled=tiled,
                                window=window)
            close(got, want[at:], dt, scale=size)
    for row in (0, 15, 16, 138):
        one = run_attention(qt[row:row + 1].contiguous(), kc, vc, bt, row,
                            mode, scale, table, temp, window=window)
        close(one, want[row:row + 1], dt, scale=size)


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("tiled", [False, True])
def test_one_distance_decides(mode, tiled):
    """Scores are all zero and one distance's bias stands out: every row
    reads exactly the value that far back (the last entry: all from there
    on, evenly). Distances at page and tile borders and beside them."""
    dev, dt = mode
    n, D = 150, 64
    q = torch.zeros(n, 2, D, dtype=dt, device=dev)
    v = np.zeros((n, 1, 64))
    v[np.arange(n), 0, np.arange(n) % 64] = 1.0 + np.arange(n) // 64
    _, v = act(v, mode)
    kc, vc, bt = paged(np.zeros((n, 1, D)), v, mode,
                       np.random.default_rng(2))
    for d in (0, 1, 15, 16, 31, 32, 33, 63, 64, 95, 120):
        table = np.zeros((2, 130), np.float32)
        table[0, d] = 40.0
        table[1, 129] = 40.0
        got = run_attention(q, kc, vc, bt, 0, mode, 1.0, table, tiled=tiled)
        for i in (d, d + 1, 77, n - 1):
            if i >= d:
                close(got[i, 0], v[i - d, 0], dt, scale=1.0, tight=1e-4)
        for i in (129, 140, n - 1):
            close(got[i, 1], v[:i - 128, 0].mean(0), dt, scale=1.0,
                  tight=1e-4)
        for row in (d, n - 1):
            one = run_attention(q[row:row + 1].contiguous(), kc, vc, bt, row,
                                mode, 1.0, table)
            close(one[0, 0], v[row - d, 0], dt, scale=1.0, tight=1e-4)


@pytest.mark.parametrize("mode", MODES)
def test_temperature_steps_at_its_period(mode):
    """Two keys, scores s and 0 with no bias: the weight of the first is a
    logistic of s times the temperature, which changes exactly where
    (position + 1) / every reaches the next integer."""
    dev, dt = mode
    n, D, every, coef = 70, 64, 16, 0.9
    q = torch.zeros(n, 1, D, dtype=dt, device=dev)
    q[:, :, 0] = 1.0
    k, v = np.zeros((n, 1, D)), np.zeros((n, 1, 64))
    k[:, 0, 0] = -200.0
    k[0, 0, 0], k[1, 0, 0], v[0] = 1.0, 0.0, 1.0
    kc, vc, bt = paged(k, v, mode, np.random.default_rng(4))
    table = np.zeros((1, 4), np.float32)
    want = np.array([1 / (1 + math.exp(-(1 + coef * math.log(
        (p + 1) // every + 1)))) for p in range(n)])
    for tiled in (False, True):
        got = run_attention(q, kc, vc, bt, 0, mode, 1.0, table,
                            (coef, every), tiled=tiled)
        close(got[1:, 0, 5], want[1:], dt, scale=1.0, bf16=4e-3)


@pytest.mark.parametrize("mode", MODES)
def test_far_key_among_hundreds_with_bias(mode):
    """One key 700 positions back stands out against hundreds, through the
    bias of all far distances."""
    dev, dt = mode
    n, D, Vd = 801, 32, 16
    rng = np.random.default_rng(1)
    k, v = np.zeros((n, 1, D)), rng.normal(0, 0.1, (n, 1, Vd))
    k[:, 0, 1] = -1.0
    k[99, 0, 1] = 3.0
    v[99] = 2.0
    qn = np.zeros((1, 2, D))
    qn[:, :, 1] = 4.0
    qt, q = act(qn, mode)
    table = np.float32(rng.normal(0, 1, (2, 230)))
    kc, vc, bt = paged(k, v, mode, rng)
    _, vh = act(v, mode)
    got = run_attention(qt, kc, vc, bt, n - 1, mode, 1.0, table)
    d = np.minimum(n - 1 - np.arange(n), 229)
    for h in range(2):
        w = L.softmax(k[:, 0] @ q[0, h] + table[h, d])
        assert w[99] > 0.9
        close(got[0, h], w @ vh[:, 0], dt)


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("heads,kv,dim,vdim,far,buckets", [
    (4, 2, 20, 12, 30, 8), (6, 2, 64, 32, 50, 16), (3, 3, 16, 24, 9, 6)])
def test_biased_attention_mixer_in_portions(mode, heads, kv, dim, vdim, far,
                                            buckets):
    """The whole mixer (biased projections, pages, table, temperature,
    output projection without a bias): portions against the whole."""
    from kaito_amd.models.hybrid_config import (_labirax_layer,
                                                distance_bias_table)
    from kaito_amd.models.mixers import RotaryWindowAttention
    dev, dt = mode
    layer = L.attention_layer(heads, kv, dim, vdim, far, temp=(0.4, 10))
    W = mixer_weights(layer, 48, dim, buckets=buckets)
    m = RotaryWindowAttention(48, _labirax_layer(layer).rattn, dt,
                              1e-4).to(dev)
    assert m.o_bias is None
    with torch.no_grad():
        m.qkv_proj.copy_(torch.cat([f32(W["m." + n], dev) for n in "qkv"]))
        m.qkv_bias.copy_(torch.cat([f32(W[f"m.{n}.b"], dev) for n in "qkv"]))
        m.dist_bias.copy_(distance_bias_table(
            torch.tensor(W["m.rel"]), far).to(dev))
        m.o_proj.copy_(f32(W["m.o"], dev))
    ht, h = act(np.random.default_rng(1).normal(0, 1, (61, 48)), mode)
    want = L.biased_attention(h, W, "m.", layer["mixer"])
    for sizes in PORTIONS:
        close(in_portions(m, ht, mode, sizes), want, dt, tight=1e-4,
              bf16=3e-2)


# ---- windowed latent attention --------------------------------------------------------

def paged_rows(rows, mode, rng, spare=2):
    dev, dt = mode
    n, DT = rows.shape
    pages = -(-n // BS)
    perm = rng.permutation(pages + spare)[:pages]
    cache = torch.full((pages + spare, BS, DT), 30.0, dtype=dt)
    for j in range(n):
        cache[perm[j // BS], j % BS] = torch.as_tensor(rows[j]).to(dt)
    return cache.to(dev), i32([perm.tolist()], dev)


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("shape", [(3, 20, 4), (11, 40, 8), (20, 64, 16),
                                   (2, 200, 32), (4, 33, 2)])
@pytest.mark.parametrize("window", [1, 2, 16, 31, 33, 64, 500, 0])
def test_latent_window(mode, shape, window):
    """Rows at the first tokens, around page and tile borders and far in,
    windows of one key up to longer than the sequence (0: none)."""
    dev, dt = mode
    H, rank, P = shape
    rng = np.random.default_rng(H + window)
    n = 211
    _, rows = act(rng.normal(0, 1, (n, rank + P)), mode)
    cache, bt = paged_rows(rows, mode, rng)
    at = [0, 1, 15, 16, 31, 32, 63, 64, 65, 130, 210]
    qt, q = act(rng.normal(0, 1, (len(at), H, rank + P)), mode)
    got = ops.latent_attention(
        qt, cache, bt, i32([0] * len(at), dev), torch.tensor(at, device=dev),
        0.2, rank, window=window)
    for r, i in enumerate(at):
        lo = max(0, i - window + 1) if window else 0
        for h in range(H):
            w = L.softmax(rows[lo:i + 1] @ q[r, h] * 0.2)
            close(got[r, h], w @ rows[lo:i + 1, :rank], dt, scale=2.0)


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("window", [15, 16, 33, 40])
def test_latent_window_edge_shows(mode, window):
    """Key p matches every query strongly: rows p .. p + window - 1 carry
    its latent, the next row does not move a bit when the key is taken
    away."""
    dev, dt = mode
    n, H, rank, P = 130, 2, 16, 8
    q = torch.zeros(n, H, rank + P, dtype=dt, device=dev)
    q[:, :, 1] = 4.0
    for p in (0, 15, 32, 70):
        outs = []
        for there in (True, False):
            rows = np.random.default_rng(1).normal(0, 0.05, (n, rank + P))
            rows[:, 1] = -4.0
            if there:
                rows[p, 1] = 4.0
            cache, bt = paged_rows(rows, mode, np.random.default_rng(2))
            outs.append(ops.latent_attention(
                q, cache, bt, i32([0] * n, dev),
                torch.arange(n, device=dev), 1.0, rank,
                window=window).cpu())
        end = min(p + window, n)
        assert (outs[0][p:end, :, 1].float() > 3.5).all()
        same = torch.ones(n, dtype=torch.bool)
        same[p:end] = False
        assert torch.equal(outs[0][same], outs[1][same])


def latent_module(layer, W, mode, width, eps):
    from kaito_amd.models.hybrid_config import _labirax_layer
    from kaito_amd.models.mixers import LatentAttention
    dev, dt = mode
    m = LatentAttention(width, _labirax_layer(layer).latent, dt, eps).to(dev)
    with torch.no_grad():
        m.in_proj.zero_()
        m.in_proj[:m.in_rows].copy_(torch.cat(
            [f32(W["m." + n], dev) for n in ("dq", "g", "dkv")], 0))
        for p, n in ((m.q_norm, "dq.norm"), (m.w_uq, "uq"),
                     (m.kv_norm, "dkv.norm"), (m.w_uk, "uk"), (m.w_uv, "uv"),
                     (m.o_proj, "o")):
            p.copy_(f32(W["m." + n], dev))
    return m


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("sizes", [(3, 12, 6, 10, 18, 14, 19),
                                   (4, 48, 16, 32, 64, 40, 16),
                                   (2, 20, 12, 24, 40, 9, 1),
                                   (2, 64, 32, 48, 96, 24, 300)])
def test_latent_mixer_in_portions(mode, sizes):
    """The whole mixer: query latent, rotation, windowed attention, value
    gate. In bf16, portions with query tiles take the expanded form, whose
    scratch holds only the pages the window reaches; without them the
    latent form."""
    dev, dt = mode
    layer = L.latent_layer(*sizes, base=300.0)
    W = mixer_weights(layer, 48, sizes[1])
    m = latent_module(layer, W, mode, 48, 1e-4)
    ht, h = act(np.random.default_rng(1).normal(0, 1, (61, 48)), mode)
    want = L.latent_attention(h, W, "m.", layer["mixer"], 1e-4)
    for sizes_ in PORTIONS:
        for tiled in (True, False):
            close(in_portions(m, ht, mode, sizes_, tiled), want, dt,
                  tight=1e-4, bf16=4e-2)


def test_value_projection_copy_follows_the_weights():
    layer = L.latent_layer(2, 12, 6, 10, 18, 14, 19)
    W = mixer_weights(layer, 48, 3)
    mode = ("cpu", torch.float32)
    m = latent_module(layer, W, mode, 48, 1e-4)
    ht, h = act(np.random.default_rng(1).normal(0, 1, (61, 48)), mode)
    for scale in (1.0, -0.5):
        with torch.no_grad():
            m.w_uv.copy_(f32(W["m.uv"] * scale, "cpu"))
        want = L.latent_attention(h, dict(W, **{"m.uv": W["m.uv"] * scale}),
                                  "m.", layer["mixer"], 1e-4)
        close(in_portions(m, ht, mode, [61]), want, torch.float32,
              tight=1e-4)


def test_gather_skips_pages_behind_the_window():
    cache = torch.arange(12).float().repeat_interleave(BS * 2).view(12, BS, 2)
    bt = torch.tensor([[7, 3, 9, 1], [2, 5, 0, 0]], dtype=torch.int32)
    rows, tables = ops.latent_gather(cache, bt, [50, 20], [33, 0])
    assert rows.view(-1, BS, 2)[:, 0, 0].tolist() == [9, 1, 2, 5]
    assert tables.tolist() == [[0, 0, 0, 1], [2, 3, 0, 0]]


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("n,lead", [(48, 8), (40, 3), (2056, 16)])
def test_value_gate(mode, n, lead):
    """A gate column per value column, read as a slice of a wider row
    (aligned and not)."""
    dev, dt = mode
    rng = np.random.default_rng(n)
    xt, x = act(rng.normal(0, 1, (5, n)), mode)
    gt, g = act(rng.normal(0, 2, (5, n + 24)), mode)
    got = ops.sigmoid_mul(xt, gt[:, lead:lead + n])
    close(got, x * L.sigmoid(g[:, lead:lead + n]), dt, bf16=1e-2)


# ---- routed feed-forward ---------------------------------------------------------------

@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("experts,top,groups", [(5, 2, 1), (7, 7, 1),
                                                (16, 1, 1), (130, 6, 2)])
def test_choice_without_correction(mode, experts, top, groups):
    dev, _ = mode
    z = np.float32(np.random.default_rng(top).normal(0, 2, (9, experts)))
    topi, topw, _ = ops.moe_route(f32(z, dev), None, top, experts, groups,
                                  groups, True, 1.0)
    for t in range(9):
        s = L.softmax(z[t].astype(np.float64))
        picked = np.argsort(-s)[:top]
        got = dict(zip(topi[t].tolist(), topw[t].tolist()))
        assert set(got) == set(picked.tolist())
        for e in picked:
            assert abs(got[e] - s[e] / s[picked].sum()) < 1e-5


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("shape", [(5, 2, 24, 20, 64), (8, 3, 64, 100, 128),
                                   (4, 1, 40, 0, 90), (6, 6, 128, 68, 64)])
def test_routed_experts_with_shared(mode, shape):
    """Fused and per-expert paths, expert and shared widths off the kernels'
    tiles, one expert and all of them, no shared expert; both addends come
    back on their own for the fused norm."""
    from kaito_amd.engine.config import ModelConfig
    from kaito_amd.models.hybrid_config import _labirax_ff, layer_moe_config
    from kaito_amd.models.loader import _load_routed
    from kaito_amd.models.moe import MoEMLP
    from kaito_amd.parallel.state import init_parallel
    init_parallel(1)
    dev, dt = mode
    E, top, ff, shared, width = shape
    mlp = L.moe(E, top, ff, shared)
    if not shared:
        del mlp["shared"]
    cfg = L.make_config([L.gla_layer(1, 4, 4, mlp=mlp)], width, 8)
    W = L.random_weights(cfg, E)

    class Files:
        @staticmethod
        def get(name):
            return torch.tensor(W[name]).to(torch.bfloat16)

        @staticmethod
        def put(p, value):
            assert p.shape == value.shape
            with torch.no_grad():
                p.copy_(value)
    base = ModelConfig(name="x", hidden_size=width, num_layers=1, num_heads=1,
                       num_kv_heads=1, intermediate_size=ff, vocab_size=8,
                       dtype=dt)
    m = MoEMLP(layer_moe_config(base, _labirax_ff(mlp))).to(dev)
    assert m.e_score_correction_bias is None
    _load_routed(Files, m, "l0.mlp.")
    ht, h = act(np.random.default_rng(3).normal(0, 1, (21, width)), mode)
    want = L.routed_experts(h, W, "l0.mlp.", mlp)
    close(m(ht), want, dt, tight=1e-4, bf16=3e-2)
    y, s = m(ht, keep_f32=True, split_shared=True)
    assert y.dtype == torch.float32 and (s is None) == (not shared)
    close(y if s is None else y + s.float(), want, dt, tight=1e-4, bf16=3e-2)
