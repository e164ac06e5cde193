"""Plain, slow implementation of the Kabanex decoder, one function per mechanism, float64 on the CPU.

It recomputes a whole sequence from its tokens every time (no cache, no pages, no batching) and
shares no code with the package: the tests compare the framework's kernels, cache, state slots and
scheduler with it.

Notation: x [n, d] residual rows of one sequence, position p = row index.
"""
import math

import torch

F = torch.float64


def layer_norm(x, w, b, eps):
    mu = x.mean(-1, keepdim=True)
    dev = x - mu
    return dev / torch.sqrt((dev * dev).mean(-1, keepdim=True) + eps) * w + b


def rotate(x, base, dims, first=0):
    """x [n, heads, dim]: pairs (i, i + dims/2) of the first ``dims`` dimensions turned by p * base^(-2i/dims)."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        f = base ** (-2.0 * i / dims)
        for p in range(x.shape[0]):
            a = (first + p) * f
            c, s = math.cos(a), math.sin(a)
            u, v = x[p, :, i], x[p, :, i + half]
            out[p, :, i] = u * c - v * s
            out[p, :, i + half] = v * c + u * s
    return out


def visible(i, j, size, keep):
    """Does position i see position j: causal, inside the last ``size`` positions or among the first ``keep``."""
    return j <= i and (i - j < size or j < keep)


def mask(n, size, keep):
    m = torch.zeros(n, n, dtype=torch.bool)
    for i in range(n):
        for j in range(i + 1):
            m[i, j] = visible(i, j, size, keep)
    return m


def softmax_weights(q, k, scale, m):
    """q [n, H, dim], k [n, G, dim] -> [H, n, n]; query head h reads key head h // (H / G)."""
    n, H, _ = q.shape
    rep = H // k.shape[1]
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // rep].T) * scale
        s = s.masked_fill(~m, float("-inf"))
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out.append(e / e.sum(-1, keepdim=True))
    return torch.stack(out)


def talk(weights, T):
    """weights [H, n, n] -> head h gets sum_g T[h, g] weights[g]."""
    return torch.stack([sum(T[h, g] * weights[g] for g in range(T.shape[1])) for h in range(T.shape[0])])


def attention(h, w, c):
    """h [n, d] -> the left mixer's output [n, d]; w: tensors by short name, c: its configuration."""
    n = h.shape[0]
    H, G, dim, vdim = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = (h @ w["q"].T).view(n, H, dim)
    k = (h @ w["k"].T).view(n, G, dim)
    v = (h @ w["v"].T).view(n, G, vdim)
    q = rotate(q, c["rot"]["base"], c["rot"]["dims"])
    k = rotate(k, c["rot"]["base"], c["rot"]["dims"])
    p = softmax_weights(q, k, c["scale"], mask(n, c["mask"]["size"], c["mask"]["keep_first"]))
    p = talk(p, w["talk"])
    gate = torch.sigmoid(h @ w["g"].T)
    heads = [gate[:, i : i + 1] * (p[i] @ v[:, i // (H // G)]) for i in range(H)]
    return torch.cat(heads, -1) @ w["o"].T


def min_gru(z_pre, u, state=None):
    """z_pre, u [n, width] -> (states [n, width]); S <- (1 - z) S + z cand."""
    S = torch.zeros(u.shape[1], dtype=u.dtype) if state is None else state
    out = []
    for t in range(u.shape[0]):
        z = torch.sigmoid(z_pre[t])
        cand = torch.where(u[t] >= 0, u[t] + 0.5, torch.sigmoid(u[t]))
        S = (1 - z) * S + z * cand
        out.append(S)
    return torch.stack(out)


def silu(x):
    return x * torch.sigmoid(x)


def recurrent(h, w):
    S = min_gru(h @ w["z"].T + w["z.b"], h @ w["x"].T + w["x.b"])
    return (S * silu(h @ w["g"].T)) @ w["o"].T


def feed_forward(h, w):
    a = torch.relu(h @ w["up"].T)
    return (a * a) @ w["down"].T


def _sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, layers=False):
    """cfg: the parsed config.json; weights: name -> tensor.  -> logits [n, vocab] (and, with
    ``layers``, the residual after every layer)."""
    w = {k: v.to(F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    res = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        mx = L["mixer"]
        y = mx["left_scale"] * attention(h, _sub(w, p + "mix.left."), mx["left"]) \
            + mx["right_scale"] * recurrent(h, _sub(w, p + "mix.right."))
        if L.get("mlp"):
            y = y + feed_forward(h, _sub(w, p + "mlp."))
        x = x + y
        res.append(x)
    logits = layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T
    return (logits, res) if layers else logits


# ----------------------------------------------------------------------------- test models
def layer_config(heads, kv_heads, dim, vdim, rot_dims, window, keep, width, ff, base=10000.0, scale=None, ls=0.9, rs=0.6):
    return {"type": "parallel",
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                               "mask": {"size": window, "keep_first": keep}, "rot": {"base": base, "dims": rot_dims},
                               "scale": dim ** -0.5 if scale is None else scale},
                      "right": {"width": width}, "left_scale": ls, "right_scale": rs},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model_config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Kabanex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def random_weights(cfg, seed=0, dtype=torch.bfloat16):
    """Weights that keep every mechanism visible: spread-out scores, strong mixing and gates, slow and
    fast recurrent channels."""
    gen = torch.Generator().manual_seed(seed)
    r = lambda *s, std=1.0: (torch.randn(*s, generator=gen) * std).to(dtype)  # noqa: E731
    d = cfg["width"]
    w = {"embed": r(cfg["vocab"], d), "final.norm": (1 + r(d, std=0.2).float()).to(dtype), "final.norm.b": r(d, std=0.2),
         "head": r(cfg["vocab"], d, std=d ** -0.5)}
    for i, L in enumerate(cfg["layers"]):
        a, W, p = L["mixer"]["left"], L["mixer"]["right"]["width"], f"l{i}."
        w[p + "norm1"], w[p + "norm1.b"] = (1 + r(d, std=0.2).float()).to(dtype), r(d, std=0.2)
        H, G, m = a["heads"], a["kv_heads"], p + "mix."
        s = d ** -0.5
        w.update({m + "left.q": r(H * a["dim"], d, std=1.6 * s), m + "left.k": r(G * a["dim"], d, std=1.6 * s),
                  m + "left.v": r(G * a["vdim"], d, std=s), m + "left.talk": (torch.eye(H) + r(H, H, std=0.4).float()).to(dtype),
                  m + "left.g": r(H, d, std=s), m + "left.o": r(d, H * a["vdim"], std=(H * a["vdim"]) ** -0.5),
                  m + "right.z": r(W, d, std=2 * s), m + "right.z.b": r(W, std=3.0), m + "right.x": r(W, d, std=s),
                  m + "right.x.b": r(W, std=0.3), m + "right.g": r(W, d, std=s), m + "right.o": r(d, W, std=W ** -0.5)})
        if L["mlp"]:
            f = L["mlp"]["ff"]
            w.update({p + "mlp.up": r(f, d, std=s), p + "mlp.down": r(d, f, std=f ** -0.5)})
    return w


def save_model(path, cfg, weights):
    import json
    import os

    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))


def logit_error(got, want):
    """Per row: RMS over the vocabulary of the difference (its mean taken off), relative to the logits' spread."""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.std()
