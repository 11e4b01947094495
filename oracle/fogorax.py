"""TEST INFRASTRUCTURE: the Fogorax language model from its equations, slow and plain (float64 on the CPU), one function per
mechanism, a sequence at a time, no cache: every call computes a whole sequence from its first token."""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm_scalar(x, g, eps):
    """one gain for all coordinates"""
    return rms(x, eps) * g


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def token_shift(h, s):
    """h (T, D): every row moves towards the row in front of it by s, element by element (a zero row in front of the first)"""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * s


def visible(i, size, keep):
    """the keys position i sees: the last `size` up to itself, and the first `keep` of the sequence"""
    return [j for j in range(i + 1) if i - j < size or j < keep]


def window_attention(q, k, v, scale, size, keep, start=0):
    """q (T, H, d) behind `start` earlier tokens; k (start + T, G, d), v (start + T, G, e); query head h reads key head h // (H / G)"""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        see = torch.tensor(visible(start + i, size, keep))
        for h in range(H):
            g = h // (H // G)
            s = (k[see, g] @ q[i, h]) * scale
            e = torch.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[see, g]
    return out


def project_kv(h, w, G, d, e):
    T = h.shape[0]
    return (h @ w["k"].T).view(T, G, d), (h @ w["v"].T).view(T, G, e)


def gated_attention(h, k, v, w, mx):
    T, H, d = h.shape[0], mx["heads"], mx["dim"]
    q = (h @ w["q"].T).view(T, H, d)
    o = window_attention(q, k, v, mx["scale"], mx["mask"]["size"], mx["mask"]["keep_first"]).reshape(T, -1)
    return (o * sigmoid(h @ w["g"].T)) @ w["o"].T


def dense_glu(h, w):
    a = gelu_tanh(h @ w["gate"].T + w["gate.b"]) * (h @ w["up"].T + w["up.b"])
    return a @ w["down"].T + w["down.b"]


def token_side(x, e, gate, proj, norm, eps):
    """x (T, D), e (T, n): what the tokens' own rows add behind a layer"""
    y = (gelu_tanh(x @ gate.T) * e) @ proj.T
    return x + rms(y, eps) * norm


def model(cfg: dict, tensors: dict, tokens, trace=None):
    """logits (T, vocab) of one sequence; cfg: a config.json dict, tensors: checkpoint names -> tensors"""
    W = {k: t.double() for k, t in tensors.items()}
    ids = torch.as_tensor(tokens)
    eps, n = cfg["norm"]["eps"], cfg["token_side"]["dim"]
    x = W["embed"][ids] + W["pos"][:len(ids)]
    held = {}
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        sub = lambda part: {k[len(p + part):]: t for k, t in W.items() if k.startswith(p + part)}
        h = norm_scalar(x, W[p + "norm1"], eps)
        hs = token_shift(h, W[p + "shift"])
        if mx.get("kv_from") is None:
            held[i] = project_kv(hs, sub("mix."), mx["kv_heads"], mx["dim"], mx["vdim"])
        k, v = held[i if mx.get("kv_from") is None else mx["kv_from"]]
        u = gated_attention(hs, k, v, sub("mix."), mx)
        if layer.get("mlp") is not None:
            u = u + dense_glu(h, sub("mlp."))
        x = x + u
        x = token_side(x, W["side.embed"][ids][:, i * n:(i + 1) * n], W[p + "side.gate"], W[p + "side.proj"], W[p + "side.norm"], eps)
        if trace is not None:
            trace.append(x)
    return norm_scalar(x, W["final.norm"], eps) @ W["head"].T


def tensor_shapes(cfg: dict):
    """checkpoint names -> shapes of a configuration"""
    D, V, L, n = cfg["width"], cfg["vocab"], len(cfg["layers"]), cfg["token_side"]["dim"]
    out = {"embed": (V, D), "pos": (cfg["max_positions"], D), "side.embed": (V, L * n), "final.norm": (), "head": (V, D)}
    for i, layer in enumerate(cfg["layers"]):
        mx, p = layer["mixer"], f"l{i}."
        H, G, d, e = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        out.update({p + "norm1": (), p + "shift": (D,), p + "mix.q": (H * d, D), p + "mix.g": (H * e, D), p + "mix.o": (D, H * e)})
        if mx.get("kv_from") is None:
            out.update({p + "mix.k": (G * d, D), p + "mix.v": (G * e, D)})
        if layer.get("mlp") is not None:
            ff = layer["mlp"]["ff"]
            for name in ("gate", "up"):
                out.update({p + f"mlp.{name}": (ff, D), p + f"mlp.{name}.b": (ff,)})
            out.update({p + "mlp.down": (D, ff), p + "mlp.down.b": (D,)})
        out.update({p + "side.gate": (n, D), p + "side.proj": (D, n), p + "side.norm": (D,)})
    return out


def random_tensors(cfg: dict, seed=0):
    """bf16 weights at which every mechanism matters: matrices that keep the size of their input, scores that stand apart, gains
    away from 1, biases and shifts away from 0"""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        if name.endswith(("norm1", "final.norm", "side.norm")):
            t = 1 + 0.2 * t
        elif name.endswith(".shift"):
            t = 0.5 + 0.4 * t
        elif name.endswith(".b") or name == "pos":
            t = 0.3 * t
        elif name.endswith(("mix.q", "mix.k")):
            t = 1.5 * t / math.sqrt(shape[-1])
        elif name not in ("embed", "side.embed"):
            t = t / math.sqrt(shape[-1])
        out[name] = t.bfloat16()
    return out
