"""Plain restatement of the Labirax design for tests: float64 numpy, token
loops, one function per mechanism, operating on checkpoint-named tensors.
Nothing here is shared with the package; it exists to be obviously right,
not fast.

Notation: h is a sub-layer's normed input row, W[name] a checkpoint tensor
(linear maps stored [out, in]), rms(v) = v / sqrt(mean(v^2) + eps).
"""
from __future__ import annotations

import json
import math
import os

import numpy as np


def rms(v, eps):
    return v / np.sqrt(np.mean(v * v, axis=-1, keepdims=True) + eps)


def layer_norm(v, w, b, eps):
    c = v - np.mean(v, axis=-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * w + b


def sigmoid(z):
    z = np.asarray(z, dtype=np.float64)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softmax(z):
    e = np.exp(z - np.max(z, axis=-1, keepdims=True))
    return e / np.sum(e, axis=-1, keepdims=True)


# ---- attention with a learned distance bias --------------------------------------

def bucket(n, buckets, bias_max):
    """Distance -> row of the bias table: one row per distance in the
    lower half, logarithmic up to bias_max in the upper half."""
    half = buckets // 2
    if n < half:
        return n
    step = math.log(n / half) / math.log(bias_max / half) * (buckets - half)
    return min(buckets - 1, half + int(math.floor(step)))


def temperature(p, coef, every):
    """Factor of the query at position p."""
    return 1.0 + coef * math.log((p + 1) // every + 1)


def biased_attention(h, W, pre, mx):
    H, G, D, V = (int(mx[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    T = h.shape[0]
    q = (h @ W[pre + "q"].T + W[pre + "q.b"]).reshape(T, H, D)
    k = (h @ W[pre + "k"].T + W[pre + "k.b"]).reshape(T, G, D)
    v = (h @ W[pre + "v"].T + W[pre + "v.b"]).reshape(T, G, V)
    rel = W[pre + "rel"]
    row = [bucket(n, rel.shape[0], float(mx["bias_max"])) for n in range(T)]
    out = np.zeros((T, H, V))
    for i in range(T):
        qi = q[i] * temperature(i, float(mx["q_temp"]["coef"]),
                                int(mx["q_temp"]["every"]))
        for n in range(H):
            g = n // (H // G)
            s = (k[:i + 1, g] @ qi[n]) * float(mx["scale"])
            s = s + rel[[row[i - j] for j in range(i + 1)], n]
            out[i, n] = softmax(s) @ v[:i + 1, g]
    return out.reshape(T, -1) @ W[pre + "o"].T


# ---- gated linear attention ------------------------------------------------------

def gla_decay(h, W, pre, tau):
    z = (h @ W[pre + "a1"].T) @ W[pre + "a2"].T + W[pre + "a2.b"]
    return sigmoid(z) ** (1.0 / tau)


def gla_recurrence(q, k, v, alpha, S=None):
    """q, k, alpha [T, heads, dim], v [T, heads, vdim] -> (o, state)."""
    T, H, D = q.shape
    V = v.shape[2]
    S = np.zeros((H, D, V)) if S is None else S.copy()
    out = np.zeros((T, H, V))
    for t in range(T):
        for n in range(H):
            S[n] = alpha[t, n][:, None] * S[n] + np.outer(k[t, n], v[t, n])
            out[t, n] = S[n].T @ q[t, n]
    return out, S


def gla(h, W, pre, mx, eps):
    H, D, V = (int(mx[k]) for k in ("heads", "dim", "vdim"))
    T = h.shape[0]
    q = (h @ W[pre + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ W[pre + "k"].T).reshape(T, H, D)
    v = (h @ W[pre + "v"].T).reshape(T, H, V)
    alpha = gla_decay(h, W, pre, float(mx["tau"])).reshape(T, H, D)
    o, _ = gla_recurrence(q, k, v, alpha)
    o = rms(o, eps) * W[pre + "norm"]
    return (o.reshape(T, -1) * silu(h @ W[pre + "g"].T)) @ W[pre + "o"].T


# ---- windowed latent attention ---------------------------------------------------

def rotate_halves(x, positions, base):
    """x [T, ..., n]: dimension i paired with i + n/2."""
    n = x.shape[-1]
    out = x.copy()
    shape = (-1,) + (1,) * (x.ndim - 2)
    for i in range(n // 2):
        a = np.asarray(positions, dtype=np.float64) * base ** (-2.0 * i / n)
        c, s = np.cos(a).reshape(shape), np.sin(a).reshape(shape)
        u, v = x[..., i], x[..., i + n // 2]
        out[..., i] = u * c - v * s
        out[..., i + n // 2] = v * c + u * s
    return out


def latent_attention(h, W, pre, mx, eps):
    H, D, P, V, R = (int(mx[k]) for k in ("heads", "dim", "rot_dim", "vdim",
                                          "kv_rank"))
    base, window = float(mx["rot"]["base"]), int(mx["mask"]["size"])
    T = h.shape[0]
    pos = np.arange(T)
    cq = rms(h @ W[pre + "dq"].T, eps) * W[pre + "dq.norm"]
    q = (cq @ W[pre + "uq"].T).reshape(T, H, D + P)
    qn, qr = q[..., :D], rotate_halves(q[..., D:], pos, base)
    down = h @ W[pre + "dkv"].T
    c = rms(down[:, :R], eps) * W[pre + "dkv.norm"]
    kr = rotate_halves(down[:, R:], pos, base)
    kn = (c @ W[pre + "uk"].T).reshape(T, H, D)
    v = (c @ W[pre + "uv"].T).reshape(T, H, V)
    out = np.zeros((T, H, V))
    for i in range(T):
        lo = max(0, i - window + 1)
        for n in range(H):
            s = kn[lo:i + 1, n] @ qn[i, n] + kr[lo:i + 1] @ qr[i, n]
            out[i, n] = softmax(s * float(mx["scale"])) @ v[lo:i + 1, n]
    gate = sigmoid(h @ W[pre + "g"].T)
    return (out.reshape(T, -1) * gate) @ W[pre + "o"].T


# ---- feed-forward ----------------------------------------------------------------

def expert(h, W, pre):
    return (silu(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) \
        @ W[pre + "down"].T


def routed_experts(h, W, pre, mlp):
    E, top = (int(mlp["router"][k]) for k in ("experts", "top"))
    z = h @ W[pre + "router"].T
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        s = softmax(z[t])
        picked = sorted(range(E), key=lambda e: -s[e])[:top]
        total = sum(s[e] for e in picked) + 1e-20
        for e in picked:
            out[t] += s[e] / total * expert(h[t], W, f"{pre}e{e}.")
    if mlp.get("shared"):
        out += expert(h, W, pre + "shared.")
    return out


# ---- the stack -------------------------------------------------------------------

def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab]; `layers_out` receives the stream after every
    layer."""
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][list(tokens)] * float(cfg["embedding"]["scale"])

    def norm(v, name):
        return layer_norm(v, W[name], W[name + ".b"], eps)
    for i, layer in enumerate(cfg["layers"]):
        src = layer.get("weights_of")
        pre = f"l{i if src is None else src}."
        mx, mlp, kind = layer["mixer"], layer.get("mlp"), layer["type"]
        h = norm(x, pre + "norm1")
        if kind == "gla":
            y = gla(h, W, pre + "mix.", mx, eps)
        elif kind == "latent_attention":
            y = latent_attention(h, W, pre + "mix.", mx, eps)
        else:
            y = biased_attention(h, W, pre + "mix.", mx)
        x = x + norm(y, pre + "norm1b")
        if mlp is not None:
            y = routed_experts(norm(x, pre + "norm2"), W, pre + "mlp.", mlp)
            x = x + norm(y, pre + "norm2b")
        if layers_out is not None:
            layers_out.append(x.copy())
    logits = norm(x, "final.norm") @ W["head"].T * float(cfg["logit_scale"])
    cap = float(cfg["logit_softcap"])
    return cap * np.tanh(logits / cap)


# ---- configurations and random checkpoints ---------------------------------------

def attention_layer(heads, kv_heads, dim, vdim, bias_max, scale=None,
                    temp=(0.3, 16), mlp=None):
    return {"type": "attention", "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "bias_max": bias_max, "scale": dim ** -0.5 if scale is None else scale,
        "q_temp": {"coef": temp[0], "every": temp[1]}}}


def gla_layer(heads, dim, vdim, tau=8.0, mlp=None):
    return {"type": "gla", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def latent_layer(heads, dim, rot_dim, vdim, kv_rank, q_rank, window,
                 base=10000.0, scale=None, mlp=None):
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
        "kv_rank": kv_rank, "q_rank": q_rank, "mask": {"size": window},
        "rot": {"base": base, "dims": rot_dim},
        "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}}


def moe(experts, top, ff, shared):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top},
            "shared": {"ff": shared}}


def again(layers, i):
    """One more run of layer i on its weights."""
    return dict(layers[i], weights_of=i)


def make_config(layers, width, vocab, eps=1e-5, embed_scale=0.8,
                logit_scale=1.7, softcap=12.0):
    return {"architecture": "Labirax", "embedding": {"scale": embed_scale},
            "layers": layers, "logit_scale": logit_scale,
            "logit_softcap": softcap, "norm": {"eps": eps}, "vocab": vocab,
            "width": width}


def bf16_round(a):
    """Values a bfloat16 file can hold, as float64 (the checkpoint is
    written in bf16, so oracle and engine must start from equal weights)."""
    import torch
    return torch.tensor(np.asarray(a), dtype=torch.float32).to(
        torch.bfloat16).double().numpy()


def random_weights(cfg, seed=0, buckets=8, decay_rank=5):
    rng = np.random.default_rng(seed)
    width, vocab = int(cfg["width"]), int(cfg["vocab"])
    W = {}

    def lin(name, out, inn, gain=1.0):
        W[name] = bf16_round(rng.normal(0, gain / np.sqrt(inn), (out, inn)))

    def vec(name, n, lo=0.6, hi=1.4):
        W[name] = bf16_round(rng.uniform(lo, hi, n))

    def gauss(name, shape, std, mean=0.0):
        W[name] = bf16_round(rng.normal(mean, std, shape))

    def norm(name):
        vec(name, width)
        gauss(name + ".b", width, 0.3)

    gauss("embed", (vocab, width), 1.2)
    norm("final.norm")
    lin("head", vocab, width)
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        pre, mx, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        mp, kind = pre + "mix.", layer["type"]
        H = int(mx["heads"])
        norm(pre + "norm1")
        norm(pre + "norm1b")
        if kind == "gla":
            D, V = int(mx["dim"]), int(mx["vdim"])
            for n, out in (("q", H * D), ("k", H * D), ("v", H * V),
                           ("g", H * V)):
                lin(mp + n, out, width)
            lin(mp + "a1", decay_rank, width)
            lin(mp + "a2", H * D, decay_rank, 2.0)
            gauss(mp + "a2.b", H * D, 1.5, 1.0)
            vec(mp + "norm", V)
            lin(mp + "o", width, H * V)
        elif kind == "latent_attention":
            D, P, V, R, Q = (int(mx[k]) for k in ("dim", "rot_dim", "vdim",
                                                  "kv_rank", "q_rank"))
            lin(mp + "dq", Q, width)
            vec(mp + "dq.norm", Q)
            lin(mp + "uq", H * (D + P), Q, 1.5)
            lin(mp + "dkv", R + P, width)
            vec(mp + "dkv.norm", R)
            lin(mp + "uk", H * D, R, 1.5)
            lin(mp + "uv", H * V, R)
            lin(mp + "g", H * V, width, 1.5)
            lin(mp + "o", width, H * V)
        else:
            G, D, V = (int(mx[k]) for k in ("kv_heads", "dim", "vdim"))
            for n, out in (("q", H * D), ("k", G * D), ("v", G * V)):
                lin(mp + n, out, width)
                gauss(mp + n + ".b", out, 0.4)
            gauss(mp + "rel", (buckets, H), 1.0)
            lin(mp + "o", width, H * V)
        if mlp is None:
            continue
        norm(pre + "norm2")
        norm(pre + "norm2b")
        fp = pre + "mlp."
        ffs = [(f"e{e}", int(mlp["expert"]["ff"]))
               for e in range(int(mlp["router"]["experts"]))]
        if mlp.get("shared"):
            ffs.append(("shared", int(mlp["shared"]["ff"])))
        for n, ff in ffs:
            lin(f"{fp}{n}.gate", ff, width, 1.5)
            lin(f"{fp}{n}.up", ff, width, 1.5)
            lin(f"{fp}{n}.down", width, ff)
        lin(fp + "router", int(mlp["router"]["experts"]), width, 3.0)
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


def model_logits(cfg, W, tokens, layers=None):
    """Logits [T, vocab] as a float64 torch tensor; `layers`, if a list,
    receives the stream after every layer."""
    import torch
    raw = [] if layers is not None else None
    out = torch.from_numpy(forward(cfg, W, tokens, raw))
    if layers is not None:
        layers.extend(torch.from_numpy(x) for x in raw)
    return out
