"""The mechanisms of the Vemenex design one at a time, each op of the
package against the plain functions of tests/vemenex_oracle.py or a closed
form: the two rotations with linearly scaled frequencies and the plain norm
behind them, sigmoid key weights (unnormalised, with a per-head bias) and
the unit sink with a gate per head, the window's edge and far keys made
visible by one dominant score (prompts and single rows, page borders, the
first tokens, stale pages), the matrix-core prompt kernel against the row
kernel, relu gated feed-forward, stream reads and writes, the expert choice
(groups, negative choices, identity outputs, renormalisation) and routed
experts. CPU runs check the reference ops; `-m gpu` runs the HIP kernels in
f32 and bf16."""
import os
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import vemenex_oracle as V  # noqa: E402

from kaito_amd import ops  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
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


# ---- rotation and the norm behind it ----------------------------------------------

@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("interleaved", [True, False])
@pytest.mark.parametrize("dim,dims,factor", [(24, 24, 3.0), (24, 8, 1.0),
                                             (64, 16, 2.5), (130, 130, 1.0),
                                             (48, 32, 1.0), (128, 128, 4.0)])
def test_rotation_then_plain_norm(mode, interleaved, dim, dims, factor):
    from kaito_amd.models.hybrid_config import RotarySpec
    dev, dt = mode
    rng = np.random.default_rng(dim + dims)
    T, H, G, Vd, eps = 5, 3, 2, 24 if dim % 16 == 0 else 20, 1e-3
    pos = np.array([0, 1, 7, 300, 41])
    qt, q = act(rng.normal(0, 0.3, (T, H, dim)), mode)
    kt, k = act(rng.normal(0, 2.0, (T, G, dim)), mode)
    vt, v = act(rng.normal(0, 1, (T, G, Vd)), mode)
    rot = {"dims": dims, "base": 500.0}
    if factor != 1.0:
        rot["scaling"] = {"factor": factor}
    freq, mag = RotarySpec(dims=dims, base=500.0, linear=factor).frequencies()
    assert mag == 1.0
    kc = torch.full((4, G, BS, dim), 9.0, dtype=dt, device=dev)
    vc = torch.full((4, G, BS, Vd), 9.0, dtype=dt, device=dev)
    slots = torch.tensor([3, 16, 47, -1, 63], device=dev)
    qn = ops.qk_norm_cache_write(
        qt, kt, vt, None, None, eps, kc, vc, slots,
        positions=torch.tensor(pos, device=dev), inv_freq=f32(freq, dev),
        unit_norm=True, interleaved=interleaved)
    want_q = V.rms(V.rotate(q, pos, rot, interleaved), eps)
    want_k = V.rms(V.rotate(k, pos, rot, interleaved), eps)
    close(qn, want_q, dt, tight=1e-4)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            close(kc[s // BS, :, s % BS], want_k[t], dt, tight=1e-4)
            close(vc[s // BS, :, s % BS], v[t], dt, bf16=1e-6)
    used = torch.zeros(4 * BS, dtype=torch.bool)
    used[[s for s in slots.tolist() if s >= 0]] = True
    untouched = kc.permute(0, 2, 1, 3).reshape(4 * BS, -1).cpu()[~used]
    assert untouched.eq(9.0).all()          # a padding row writes nothing


# ---- attention over pages ---------------------------------------------------------

def paged(k, v, mode, rng, spare=2):
    """Keys [n, G, D] and values into shuffled pages; the rest of the pool
    holds stale rows of large numbers."""
    dev, dt = mode
    n, G, D = k.shape
    pages = -(-n // BS)
    perm = rng.permutation(pages + spare)[:pages]
    kc = torch.full((pages + spare, G, BS, D), 40.0, dtype=dt, device=dev)
    vc = torch.full((pages + spare, G, BS, v.shape[2]), 40.0, dtype=dt,
                    device=dev)
    for j in range(n):
        kc[perm[j // BS], :, j % BS] = torch.as_tensor(k[j]).to(dt).to(dev)
        vc[perm[j // BS], :, j % BS] = torch.as_tensor(v[j]).to(dt).to(dev)
    return kc, vc, i32([perm.tolist()], dev)


def run_attention(q, kc, vc, bt, pos0, mode, window, scale, kind, pb=None,
                  gate=None, tiled=False):
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
        q, kc, vc, bt, i32([0] * n, dev), pos, scale, window=window,
        tiles=tiles, sigmoid_bias=None if pb is None else f32(pb, dev),
        sinks=torch.zeros(q.size(1), device=dev) if kind == "sink" else None,
        gate=gate)


def weights_of(kind, pb):
    return (lambda n, s: V.sigmoid_weights(s, pb[n])) if kind == "sigmoid" \
        else (lambda n, s: V.sink_weights(s))


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("kind", ["sigmoid", "sink"])
@pytest.mark.parametrize("heads,kv,dim,vdim,window", [
    (6, 2, 64, 64, 21), (4, 4, 24, 40, 1), (5, 1, 32, 16, 200),
    (8, 1, 128, 32, 33), (2, 2, 18, 10, 16), (3, 1, 64, 128, 17)])
def test_attention_weights(mode, kind, heads, kv, dim, vdim, window):
    """Whole sequences and single rows, with and without query tiles: sizes
    of the matrix-core kernel, of the vector kernel and of neither; windows
    of one key, a page, a page and one, and longer than the sequence."""
    dev, dt = mode
    rng = np.random.default_rng(heads * 100 + window)
    n, scale = 75, 0.4
    qt, q = act(rng.normal(0, 1, (n, heads, dim)), mode)
    _, k = act(rng.normal(0, 1, (n, kv, dim)), mode)
    _, v = act(rng.normal(0, 1, (n, kv, vdim)), mode)
    pb = rng.normal(-1.0, 1.5, heads)
    pb = np.float32(pb).astype(np.float64)
    gt, g = act(rng.normal(0, 2, (n, heads + 3)), mode)   # a row-strided view
    want = V.attend(q, k, v, scale, window, weights_of(kind, pb))
    want = want * V.sigmoid(g[:, 2:2 + heads])[:, :, None]
    kc, vc, bt = paged(k, v, mode, rng)
    kw = dict(pb=pb if kind == "sigmoid" else None)
    size = np.abs(want).max()
    for tiled in (False, True):
        got = run_attention(qt, kc, vc, bt, 0, mode, window, scale, kind,
                            gate=gt[:, 2:2 + heads], tiled=tiled, **kw)
        close(got, want, dt, scale=size)
        part = run_attention(qt[41:].contiguous(), kc, vc, bt, 41, mode,
                             window, scale, kind, gate=gt[41:, 2:2 + heads],
                             tiled=tiled, **kw)
        close(part, want[41:], dt, scale=size)
    one = run_attention(qt[74:].contiguous(), kc, vc, bt, 74, mode, window,
                        scale, kind, gate=gt[74:, 2:2 + heads], **kw)
    close(one, want[74:], dt, scale=size)


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("kind", ["sigmoid", "sink"])
@pytest.mark.parametrize("window", [15, 16, 17, 32, 70])
def test_window_edge_key_is_seen_and_the_next_is_not(mode, kind, window):
    """Key p matches every query strongly and every other key not at all:
    rows p .. p + window - 1 carry its value, the row after does not, bit
    for bit as if the key were absent. Prompt rows, tiled rows and single
    rows; keys at page borders, the first token and far ahead."""
    dev, dt = mode
    n, D, Vd = 120, 64, 64
    q = torch.zeros(n, 2, D, dtype=dt, device=dev)
    q[:, :, 0] = 4.0
    rng = np.random.default_rng(3)
    base_v = rng.normal(0, 0.05, (n, 1, Vd))
    pb = [-8.0, -8.0]
    for p in (0, 15, 16, 37):
        k = np.zeros((n, 1, D))
        k[:, :, 0] = -4.0
        plain = np.array(k)
        k[p, 0, 0] = 4.0
        v = np.array(base_v)
        v[p] = 1.0
        outs = []
        for keys in (k, plain):
            kc, vc, bt = paged(keys, v, mode, np.random.default_rng(5))
            for tiled in (False, True):
                outs.append(run_attention(q, kc, vc, bt, 0, mode, window,
                                          1.0, kind, pb=pb
                                          if kind == "sigmoid" else None,
                                          tiled=tiled))
        for with_key, without in ((outs[0], outs[2]), (outs[1], outs[3])):
            seen = with_key[:, :, 0].float().cpu()
            end = min(p + window, n)
            assert (seen[p:end] > 0.9).all()
            same = torch.ones(n, dtype=torch.bool)
            same[p:end] = False
            assert torch.equal(with_key.cpu()[same], without.cpu()[same])
        for row in {p, min(p + window - 1, n - 1), min(p + window, n - 1)}:
            kc, vc, bt = paged(k, v, mode, np.random.default_rng(6))
            one = run_attention(q[row:row + 1], kc, vc, bt, row, mode, window,
                                1.0, kind, pb=pb if kind == "sigmoid"
                                else None)
            assert (one[0, :, 0].float().cpu() > 0.9).all() == \
                (row - p < window)


@pytest.mark.parametrize("mode", MODES)
def test_far_key_among_hundreds(mode):
    """One key 700 positions back stands out of a window of 1000."""
    dev, dt = mode
    n, D, Vd = 800, 32, 16
    rng = np.random.default_rng(1)
    k = np.zeros((n, 1, D))
    k[:, 0, 1] = -1.0
    k[99, 0, 1] = 3.0
    v = rng.normal(0, 0.1, (n, 1, Vd))
    v[99] = 2.0
    qn = np.zeros((1, 2, D))
    qn[:, :, 1] = 4.0
    qt, q = act(qn, mode)
    for kind, pb in (("sigmoid", np.array([-6.0, 3.0])), ("sink", None)):
        kc, vc, bt = paged(k, v, mode, rng)
        got = run_attention(qt, kc, vc, bt, n - 1, mode, 1000, 1.0, kind,
                            pb=pb)
        _, vh = act(v, mode)
        s = k[:, 0] @ q[0, 0]
        for h in range(2):
            w = V.sigmoid_weights(s, pb[h]) if pb is not None \
                else V.sink_weights(s)
            close(got[0, h], w @ vh[:, 0], dt)


@pytest.mark.parametrize("mode", MODES)
def test_weights_are_not_normalised(mode):
    """Closed form: equal scores give count * sigmoid(score + bias) times
    the common value, and count / (count + exp(-score)) under the unit
    sink."""
    dev, dt = mode
    q = torch.ones(12, 2, 8, dtype=dt, device=dev)
    k, v = np.full((12, 1, 8), 0.25), np.full((12, 1, 8), 1.5)
    pb = np.array([-3.0, 0.5])
    kc, vc, bt = paged(k, v, mode, np.random.default_rng(0))
    got = run_attention(q, kc, vc, bt, 0, mode, 7, 0.5, "sigmoid", pb=pb)
    sink = run_attention(q, kc, vc, bt, 0, mode, 7, 0.5, "sink")
    for i in range(12):
        n = min(i + 1, 7)
        for h in range(2):
            close(got[i, h], np.full(8, 1.5 * n / (1 + np.exp(-1.0 - pb[h]))),
                  dt)
            close(sink[i, h], np.full(8, 1.5 * n / (n + np.exp(-1.0))), dt)


def attention_module(kind, mx, W, mode, width, eps):
    from kaito_amd.models.hybrid_config import _vemenex_layer
    from kaito_amd.models.mixers import RotaryWindowAttention
    dev, dt = mode
    spec = _vemenex_layer({"type": kind, "mixer": mx, "mlp": None}).rattn
    m = RotaryWindowAttention(width, spec, dt, eps).to(dev)
    names = ("q", "k", "v") + (("g",) if spec.head_gate else ())
    with torch.no_grad():
        m.qkv_proj.zero_()
        m.qkv_proj[:m.in_rows].copy_(torch.cat(
            [f32(W["m." + x], dev) for x in names], 0))
        m.o_proj.copy_(f32(W["m.o"], dev))
        if spec.sigmoid_scores:
            m.score_bias.copy_(f32(W["m.pb"], dev))
    return m


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("kind", ["attention", "attention_2"])
@pytest.mark.parametrize("dim,vdim", [(20, 12), (64, 32)])
def test_attention_mixer_in_portions(mode, kind, dim, vdim):
    """The whole mixer (projections, rotation, norm, pages, weights, gate,
    output projection): portions of many sizes against the whole."""
    dev, dt = mode
    rng = np.random.default_rng(dim)
    H, G, width, eps, n = 4, 2, 48, 1e-4, 61
    mx = {"heads": H, "kv_heads": G, "dim": dim, "vdim": vdim, "scale": 0.3,
          "mask": {"size": 19}, "rot": {"base": 300.0, "dims": dim // 2}}
    if kind == "attention":
        mx["rot"]["scaling"] = {"factor": 3.0}
    W = {}
    for name, rows, cols in (("q", H * dim, width), ("k", G * dim, width),
                             ("v", G * vdim, width), ("g", H, width),
                             ("o", width, H * vdim)):
        W["m." + name] = V._bf16_round(
            rng.normal(0, 1.0 / np.sqrt(cols), (rows, cols)))
    W["m.pb"] = V._bf16_round(rng.normal(-1, 1, H))
    m = attention_module(kind, mx, W, mode, width, eps)
    ht, h = act(rng.normal(0, 1, (n, width)), mode)
    fn = V.sigmoid_attention if kind == "attention" else \
        V.gated_sink_attention
    want = fn(h, W, "m.", mx, eps)
    for sizes in ([n], [1] * n, [2, 17, 1, 2, 30, 9], [33, 2, 2, 24]):
        cache = m.alloc_cache(8, BS, 4, dev)
        bt = i32([[6, 1, 4, 2]], dev)
        out, at = [], 0
        for c in sizes:
            pos = torch.arange(at, at + c, device=dev)
            ts, tq = ops.build_query_tiles([c], dev)
            meta = SimpleNamespace(
                cu_seqlens=i32([0, c], dev), state_slots=i32([1], dev),
                seq_starts=i32([at], dev), token_seq=i32([0] * c, dev),
                block_tables=bt, slot_mapping=(
                    bt[0].long()[pos // BS] * BS + pos % BS),
                tile_seq=ts if c > 1 else None, tile_qbase=tq,
                layer_shared={})
            out.append(m(ht[at:at + c].contiguous(), pos, cache, meta))
            at += c
        close(torch.cat(out, 0), want, dt, bf16=3e-2)


# ---- streams -----------------------------------------------------------------------

@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("width", [64, 75, 1028, 8196])
def test_stream_write_and_next_read(mode, S, width):
    dev, dt = mode
    rng = np.random.default_rng(S * width)
    T, eps = 3, 1e-3
    x = np.float32(rng.normal(0, 2, (T, S, width))).astype(np.float64)
    mix = np.float32(rng.normal(0, 1, (S, S))).astype(np.float64)
    w_in, w_out, nxt = (np.float32(rng.normal(0.3, 1, S)).astype(np.float64)
                        for _ in range(3))
    yt, y = act(rng.normal(0, 1, (T, width)), mode)
    want = V.stream_write(x, mix, w_out, 1.0, y)
    u = V.stream_read(want, nxt)
    args = [f32(a, dev) for a in (mix, w_out, nxt)]
    for w in (np.array([1.3]), rng.uniform(0.5, 1.5, width)):
        for yy in (yt, yt.float()):         # routed sums arrive in f32
            xt = f32(x, dev)
            h = ops.stream_mix_norm(xt, yy, *args, f32(w, dev), eps, dt)
            close(xt, want, torch.float32)
            close(h, V.rms(u, eps) * np.float32(w), dt)
            assert h.dtype == dt
    # the last sub-layer: the plain sum, streams stored or not
    for store in (True, False):
        xt = f32(x, dev)
        s = ops.stream_mix_norm(xt, yt, args[0], args[1],
                                torch.ones(S, device=dev), None, eps,
                                torch.float32, write_x=store)
        close(s, want.sum(1), torch.float32)
        close(xt, want if store else x, torch.float32)
    # a row-strided sub-layer output
    wide = torch.zeros(T, width + 5, dtype=dt, device=dev)
    wide[:, 3:3 + width] = yt
    xt = f32(x, dev)
    ops.stream_mix_norm(xt, wide[:, 3:3 + width], *args, f32([0.7], dev),
                        eps, dt)
    close(xt, want, torch.float32)


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("S,width", [(1, 136), (3, 75), (5, 3000),
                                     (2, 8200)])
def test_stream_embedding(mode, S, width):
    dev, dt = mode
    rng = np.random.default_rng(S)
    vocab, eps = 11, 1e-2
    tt, table = act(rng.normal(0, 0.2, (vocab, width)), mode)
    w_in = np.float32(rng.normal(0.4, 1, S)).astype(np.float64)
    ids = [4, 0, 10, 4, 7]
    x, h = ops.stream_embed(torch.tensor(ids, device=dev), tt,
                            f32([1.4], dev), f32(w_in, dev), f32([0.6], dev),
                            eps)
    e = V.rms(table[ids], eps) * np.float32(1.4)
    want = np.stack([e] * S, 1)
    close(x, want, torch.float32)
    close(h, V.rms(V.stream_read(want, w_in), eps) * np.float32(0.6), dt)
    assert x.dtype == torch.float32 and h.dtype == dt


def test_mix_matrix_is_indexed_from_to():
    """One entry: stream 2 flows into stream 0 and into no other."""
    x = np.random.default_rng(0).normal(0, 1, (1, 3, 4))
    mix = np.zeros((3, 3))
    mix[2, 0] = 1.0
    xt = f32(x, "cpu")
    ops.stream_mix_norm(xt, torch.zeros(1, 4), f32(mix, "cpu"),
                        torch.zeros(3), torch.ones(3), torch.ones(1), 1e-5,
                        torch.float32)
    close(xt[:, 0], x[:, 2], torch.float32)
    assert xt[:, 1:].eq(0).all()


# ---- feed-forwards -----------------------------------------------------------------

@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("ff", [40, 33])
def test_relu_gated_feed_forward(mode, ff):
    from kaito_amd.models.hybrid_config import GLUSpec
    from kaito_amd.models.mixers import GatedFF
    dev, dt = mode
    rng = np.random.default_rng(ff)
    gt, g = act(rng.normal(0, 1, (5, 2 * ff)), mode)
    close(ops.relu_glu(gt), np.maximum(g[:, :ff], 0) * g[:, ff:], dt)
    W = {k: V._bf16_round(rng.normal(0, 0.3, s)) for k, s in (
        ("f.gate", (ff, 24)), ("f.up", (ff, 24)), ("f.down", (24, ff)))}
    m = GatedFF(24, GLUSpec(ff, "relu"), dt).to(dev)
    with torch.no_grad():
        m.gate_up.copy_(f32(np.concatenate([W["f.gate"], W["f.up"]]), dev))
        m.down.copy_(f32(W["f.down"], dev))
    ht, h = act(rng.normal(0, 1, (7, 24)), mode)
    close(m(ht), V.relu_glu(h, W, "f."), dt, bf16=3e-2)


def moe_module(mode, width, mlp, W, pre):
    from kaito_amd.engine.config import ModelConfig
    from kaito_amd.models.hybrid_config import _vemenex_ff, layer_moe_config
    from kaito_amd.models.loader import _load_routed
    from kaito_amd.models.moe import MoEMLP
    from kaito_amd.parallel.state import init_parallel
    init_parallel(1)
    dev, dt = mode
    cfg = ModelConfig(name="t", hidden_size=width, dtype=dt)
    m = MoEMLP(layer_moe_config(cfg, _vemenex_ff(mlp)[1])).to(dev)

    def put(p, t):
        assert tuple(p.shape) == tuple(t.shape)
        with torch.no_grad():
            p.copy_(t)
    _load_routed(SimpleNamespace(get=lambda n: f32(W[n], dev), put=put), m,
                 pre)
    return m


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("N,real,top,groups,keep", [
    (14, 12, 3, 2, 1), (9, 9, 1, 1, 1), (12, 7, 4, 4, 2), (8, 5, 8, 1, 1),
    (70, 66, 5, 7, 3), (130, 128, 6, 10, 4), (300, 256, 8, 60, 7), (5, 0, 2, 5, 3)])
def test_expert_choice(device, N, real, top, groups, keep):
    """Indices, weights, the identity share and the sort, with corrections
    large enough to make choices negative and to override scores."""
    rng = np.random.default_rng(N + top)
    T = 37
    z = np.float32(rng.normal(0, 2, (T, N))).astype(np.float64)
    corr = np.float32(rng.normal(-0.2, 0.3, N)).astype(np.float64)
    for renorm, scale in ((True, 1.0), (False, 1.7)):
        topi, topw, w_id = ops.moe_route(f32(z, device), f32(corr, device),
                                         top, real, groups, keep, renorm,
                                         scale)
        for t in range(T):
            s = V.softmax(z[t])
            want = V.choose(s, corr, top, groups, keep)
            assert topi[t].tolist() == want
            w = s[want] * scale / ((s[want].sum() + 1e-20) if renorm else 1.0)
            close(topw[t], w, torch.float32, scale=w.max())
            close(w_id[t], sum(x for x, e in zip(w, want) if e >= real),
                  torch.float32, scale=1.0)
    tok, gates, off = ops.moe_sort(topi, topw, N)
    flat = topi.reshape(-1).cpu().numpy()
    assert off.tolist() == np.concatenate(
        [[0], np.cumsum(np.bincount(flat, minlength=N))]).tolist()
    for e in range(N):
        a, b = int(off[e]), int(off[e + 1])
        got = sorted(zip(tok[a:b].tolist(), gates[a:b].tolist()))
        want = sorted((t, float(topw[t, k])) for t in range(T)
                      for k in range(top) if int(topi[t, k]) == e)
        assert got == want


def test_negative_choices_stay_ahead_of_excluded_groups():
    """All choices of the kept group are negative: outputs of the other
    groups must still not be taken (excluded means minus infinity)."""
    z = torch.zeros(1, 4)
    corr = torch.tensor([-0.3, -0.9, -1.0, -0.8])
    topi, _, _ = ops.moe_route(z, corr, 2, 4, 2, 1, True, 1.0)
    assert topi[0].tolist() == [0, 1]


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("width,ff,experts,identity,top,groups,T", [
    (40, 24, 6, 2, 3, (2, 1), 9),     # per-expert path
    (64, 64, 7, 1, 2, (4, 3), 70),    # fused grouped products in bf16
    (128, 40, 5, 0, 2, (1, 1), 21),   # experts padded to the tile, no identity
    (64, 64, 2, 6, 4, (2, 2), 33)])   # mostly identity
def test_routed_experts(mode, width, ff, experts, identity, top, groups, T):
    dev, dt = mode
    rng = np.random.default_rng(width + ff)
    mlp = V.moe(experts, top, ff, identity, groups, limit=0.6)
    W = {}
    for e in range(experts):
        for n, shape in (("gate", (ff, width)), ("up", (ff, width)),
                         ("down", (width, ff))):
            W[f"r.e{e}.{n}"] = V._bf16_round(
                rng.normal(0, 1.3 / np.sqrt(shape[1]), shape))
    W["r.router"] = V._bf16_round(
        rng.normal(0, 3 / np.sqrt(width), (experts + identity, width)))
    W["r.correction"] = V._bf16_round(rng.normal(0, 0.2, experts + identity))
    m = moe_module(mode, width, mlp, W, "r.")
    ht, h = act(rng.normal(0, 1, (T, width)), mode)
    want = V.routed_experts(h, W, "r.", mlp)
    out = m(ht, keep_f32=True)
    assert out.dtype == torch.float32
    close(out, want, dt, bf16=3e-2)
    close(m(ht), want, dt, bf16=3e-2)
    if dev == "cuda" and dt == torch.bfloat16 and width % 64 == 0:
        # the per-expert path of large prompts agrees with the fused one
        m.FUSED_MAX_TOKENS = 0
        close(m(ht, keep_f32=True), want, dt, bf16=3e-2)


def test_identity_expert_returns_its_input():
    """Every choice forced onto the identity outputs: the layer is the
    identity map, weights summing to one."""
    mlp = V.moe(3, 2, 8, identity=2)
    W = {f"r.e{e}.{n}": np.ones(s) for e in range(3) for n, s in (
        ("gate", (8, 16)), ("up", (8, 16)), ("down", (16, 8)))}
    W["r.router"] = np.random.default_rng(0).normal(0, 1, (5, 16))
    W["r.correction"] = np.array([-5.0, -5.0, -5.0, 0.0, 0.0])
    m = moe_module(("cpu", torch.float32), 16, mlp, W, "r.")
    h = torch.randn(6, 16)
    close(m(h), h.double().numpy(), torch.float32)
