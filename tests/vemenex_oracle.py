"""Plain restatement of the Vemenex design for tests: float64 numpy, token
loops, one function per mechanism, operating on checkpoint-named tensors.
Nothing here is shared with the package; it exists to be obviously right,
not fast.

Notation: h is a sub-layer's normed input row, W[name] a checkpoint tensor
(linear maps stored [out, in]), rms(v) = v / sqrt(mean(v^2) + eps).
"""
from __future__ import annotations

import json
import os

import numpy as np


def rms(v, eps):
    return v / np.sqrt(np.mean(v * v, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    out = np.empty_like(z)
    up = z >= 0
    out[up] = 1.0 / (1.0 + np.exp(-z[up]))
    e = np.exp(z[~up])
    out[~up] = e / (1.0 + e)
    return out


def softmax(z):
    e = np.exp(z - np.max(z, axis=-1, keepdims=True))
    return e / np.sum(e, axis=-1, keepdims=True)


# ---- streams --------------------------------------------------------------------

def stream_read(X, w_in):
    """X [T, S, width] -> sum over streams of w_in[s] X[:, s]."""
    out = np.zeros_like(X[:, 0])
    for s in range(X.shape[1]):
        out += w_in[s] * X[:, s]
    return out


def stream_write(X, mix, w_out, m, y):
    """New stream t = sum over s of mix[s, t] X[:, s], plus m w_out[t] y."""
    S = X.shape[1]
    new = np.zeros_like(X)
    for to in range(S):
        for frm in range(S):
            new[:, to] += mix[frm, to] * X[:, frm]
        new[:, to] += m * w_out[to] * y
    return new


# ---- attention ------------------------------------------------------------------

def rotate(x, positions, rot, interleaved):
    """x [T, heads, n], rotated in its first `dims` dimensions; the pairs
    are (2i, 2i+1) or (i, i + dims/2)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    factor = float((rot.get("scaling") or {}).get("factor", 1.0))
    out = x.copy()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        ang = np.asarray(positions, dtype=np.float64) \
            * (base ** (-2.0 * i / dims) / factor)
        c, s = np.cos(ang)[:, None], np.sin(ang)[:, None]
        out[..., a] = x[..., a] * c - x[..., b] * s
        out[..., b] = x[..., b] * c + x[..., a] * s
    return out


def visible(i, window):
    """Key positions query i sees."""
    return [j for j in range(i + 1) if i - j < window]


def sigmoid_weights(scores, bias):
    return sigmoid(scores + bias)


def sink_weights(scores):
    """Softmax with one more term exp(0) in the denominator."""
    top = max(0.0, float(np.max(scores)))
    e = np.exp(scores - top)
    return e / (np.exp(-top) + np.sum(e))


def project_qkv(h, W, pre, mx, eps, interleaved, positions=None):
    H, G, D, V = (int(mx[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    T = h.shape[0]
    positions = np.arange(T) if positions is None else positions
    q = (h @ W[pre + "q"].T).reshape(T, H, D)
    k = (h @ W[pre + "k"].T).reshape(T, G, D)
    v = (h @ W[pre + "v"].T).reshape(T, G, V)
    q = rms(rotate(q, positions, mx["rot"], interleaved), eps)
    k = rms(rotate(k, positions, mx["rot"], interleaved), eps)
    return q, k, v


def attend(q, k, v, scale, window, weights_of):
    """q [T, H, D], k [T, G, D], v [T, G, V]; weights_of(head, scores)."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for n in range(H):
        g = n // rep
        for i in range(T):
            js = visible(i, window)
            w = weights_of(n, (k[js, g] @ q[i, n]) * scale)
            out[i, n] = w @ v[js, g]
    return out


def sigmoid_attention(h, W, pre, mx, eps):
    q, k, v = project_qkv(h, W, pre, mx, eps, True)
    o = attend(q, k, v, float(mx["scale"]), int(mx["mask"]["size"]),
               lambda n, s: sigmoid_weights(s, W[pre + "pb"][n]))
    return o.reshape(h.shape[0], -1) @ W[pre + "o"].T


def gated_sink_attention(h, W, pre, mx, eps):
    q, k, v = project_qkv(h, W, pre, mx, eps, False)
    o = attend(q, k, v, float(mx["scale"]), int(mx["mask"]["size"]),
               lambda n, s: sink_weights(s))
    o = o * sigmoid(h @ W[pre + "g"].T)[:, :, None]
    return o.reshape(h.shape[0], -1) @ W[pre + "o"].T


# ---- feed-forwards --------------------------------------------------------------

def relu_glu(h, W, pre):
    return (np.maximum(h @ W[pre + "gate"].T, 0.0)
            * (h @ W[pre + "up"].T)) @ W[pre + "down"].T


def clamped_expert(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def choose(scores, correction, top, groups, keep):
    """Indices of one token's chosen outputs."""
    choice = scores + correction
    n = len(choice) // groups
    best = sorted(range(groups),
                  key=lambda g: -np.max(choice[g * n:(g + 1) * n]))[:keep]
    allowed = [e for g in best for e in range(g * n, (g + 1) * n)]
    return sorted(allowed, key=lambda e: -choice[e])[:top]


def routed_experts(h, W, pre, mlp):
    r = mlp["router"]
    E, limit = int(r["experts"]), float(mlp["expert"]["limit"])
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ W[pre + "router"].T
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        s = softmax(z[t])
        picked = choose(s, W[pre + "correction"], int(r["top"]),
                        int(groups["count"]), int(groups["keep"]))
        total = sum(s[e] for e in picked) + 1e-20
        for e in picked:
            if e >= E:                                  # identity
                y = h[t]
            else:
                y = clamped_expert(h[t], W[f"{pre}e{e}.gate"],
                                   W[f"{pre}e{e}.up"],
                                   W[f"{pre}e{e}.down"], limit)
            out[t] += s[e] / total * y
    return out


# ---- the stack ------------------------------------------------------------------

def forward(cfg, W, tokens, streams_out=None):
    """Logits [T, vocab]; `streams_out` receives the sum of the streams
    after every layer."""
    eps, m = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x = rms(W["embed"][list(tokens)], eps) * W["embed.norm"]
    X = np.stack([x] * int(cfg["streams"]), 1)
    for i, layer in enumerate(cfg["layers"]):
        pre, mx = f"l{i}.", layer["mixer"]

        def sub(q, norm, f):
            u = stream_read(X, W[f"{pre}hc{q}.in"])
            y = f(rms(u, eps) * W[pre + norm])
            return stream_write(X, W[f"{pre}hc{q}.mix"],
                                W[f"{pre}hc{q}.out"], m, y)
        mixer = {"attention": sigmoid_attention,
                 "attention_2": gated_sink_attention}[layer["type"]]
        X = sub(1, "norm1", lambda h: mixer(h, W, pre + "mix.", mx, eps))
        mlp = layer.get("mlp")
        if mlp is not None:
            if mlp["kind"] == "dense":
                X = sub(2, "norm2", lambda h: relu_glu(h, W, pre + "mlp."))
            else:
                X = sub(2, "norm2",
                        lambda h: routed_experts(h, W, pre + "mlp.", mlp))
        if streams_out is not None:
            streams_out.append(X.sum(1))
    return (rms(X.sum(1), eps) * W["final.norm"]) @ W["head"].T


# ---- configurations and random checkpoints --------------------------------------

def _attn(kind, heads, kv_heads, dim, vdim, window, rot_dims, base, scale,
          factor, mlp):
    rot = {"base": base, "dims": rot_dims}
    if factor is not None:
        rot["scaling"] = {"factor": factor}
    return {"type": kind, "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "mask": {"size": window}, "rot": rot,
        "scale": dim ** -0.5 if scale is None else scale}}


def sigmoid_layer(heads, kv_heads, dim, vdim, window, rot_dims=None,
                  base=10000.0, scale=None, factor=2.0, mlp=None):
    return _attn("attention", heads, kv_heads, dim, vdim, window,
                 dim if rot_dims is None else rot_dims, base, scale, factor,
                 mlp)


def sink_layer(heads, kv_heads, dim, vdim, window, rot_dims=None,
               base=10000.0, scale=None, mlp=None):
    return _attn("attention_2", heads, kv_heads, dim, vdim, window,
                 dim if rot_dims is None else rot_dims, base, scale, None,
                 mlp)


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, identity=0, groups=(1, 1), limit=2.0):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "top": top, "identity": identity,
                       "groups": {"count": groups[0], "keep": groups[1]}}}


def make_config(layers, width, vocab, streams, eps=1e-5, residual_mult=0.5):
    return {"architecture": "Vemenex", "layers": layers,
            "norm": {"eps": eps}, "residual_mult": residual_mult,
            "streams": streams, "vocab": vocab, "width": width}


def _bf16_round(a):
    """Values a bfloat16 file can hold, as float64 (the checkpoint is
    written in bf16, so oracle and engine must start from equal weights)."""
    import torch
    return torch.tensor(np.asarray(a), dtype=torch.float32).to(
        torch.bfloat16).double().numpy()


def random_weights(cfg, seed=0):
    rng = np.random.default_rng(seed)
    width, vocab, S = (int(cfg[k]) for k in ("width", "vocab", "streams"))
    W = {}

    def lin(name, out, inn, gain=1.0):
        W[name] = _bf16_round(rng.normal(0, gain / np.sqrt(inn), (out, inn)))

    def vec(name, shape, lo, hi):
        W[name] = _bf16_round(rng.uniform(lo, hi, shape))

    W["embed"] = _bf16_round(rng.normal(0, 1.5, (vocab, width)))
    vec("embed.norm", (), 0.7, 1.4)
    vec("final.norm", (), 0.7, 1.4)
    lin("head", vocab, width)
    for i, layer in enumerate(cfg["layers"]):
        pre, mx, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        H, G, D, V = (int(mx[k]) for k in ("heads", "kv_heads", "dim",
                                           "vdim"))
        mp = pre + "mix."
        for q in (1, 2) if mlp is not None else (1,):
            vec(f"{pre}norm{q}", (), 0.7, 1.4)
            vec(f"{pre}hc{q}.in", (S,), -0.3, 1.2)
            vec(f"{pre}hc{q}.out", (S,), -0.5, 1.5)
            # near the identity, clearly asymmetric
            W[f"{pre}hc{q}.mix"] = _bf16_round(
                np.eye(S) * 0.8 + rng.normal(0, 0.25, (S, S)))
        lin(mp + "q", H * D, width)
        lin(mp + "k", G * D, width)
        lin(mp + "v", G * V, width)
        if layer["type"] == "attention":
            W[mp + "pb"] = _bf16_round(rng.normal(-2.0, 1.0, H))
        else:
            lin(mp + "g", H, width, 1.5)
        lin(mp + "o", width, H * V)
        if mlp is None:
            continue
        fp = pre + "mlp."
        if mlp["kind"] == "dense":
            ff = int(mlp["ff"])
            lin(fp + "gate", ff, width, 1.5)
            lin(fp + "up", ff, width, 1.5)
            lin(fp + "down", width, ff)
            continue
        ff, r = int(mlp["expert"]["ff"]), mlp["router"]
        for e in range(int(r["experts"])):
            lin(f"{fp}e{e}.gate", ff, width, 1.5)
            lin(f"{fp}e{e}.up", ff, width, 1.5)
            lin(f"{fp}e{e}.down", width, ff)
        n = int(r["experts"]) + int(r.get("identity", 0))
        lin(fp + "router", n, width, 3.0)
        W[fp + "correction"] = _bf16_round(rng.normal(0, 0.1, n))
    return W


def write_checkpoint(folder, cfg, W):
    """config.json + model.safetensors (bfloat16) as a served folder."""
    import torch
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: torch.tensor(np.asarray(v), dtype=torch.float32).to(
        torch.bfloat16).contiguous() for k, v in W.items()},
        os.path.join(folder, "model.safetensors"))
    return folder


def model_logits(cfg, W, tokens, streams=None):
    """Logits [T, vocab] as a float64 torch tensor; `streams`, if a list,
    receives the summed streams after every layer."""
    import torch
    raw = [] if streams is not None else None
    out = torch.from_numpy(forward(cfg, W, tokens, raw))
    if streams is not None:
        streams.extend(torch.from_numpy(x) for x in raw)
    return out
