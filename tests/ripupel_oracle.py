"""Plain, slow implementation of the Ripupel decoder, one function per mechanism, float64 on the CPU.

It recomputes a whole sequence from its tokens every time (no cache, no pages, no batching, no absorbed
projections) and shares no code with the package: the tests compare the framework's kernels, cache,
state slots and scheduler with it.

Notation: x [n, d] residual rows of one sequence, position p = row index.
"""
import math

import torch

F = torch.float64


def layer_norm(x, w, eps):
    mu = x.mean(-1, keepdim=True)
    dev = x - mu
    return dev / torch.sqrt((dev * dev).mean(-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate(x, base, first=0):
    """x [n, heads, r]: pairs (i, i + r/2) turned by p * base^(-2i/r)."""
    out = x.clone()
    r = x.shape[-1]
    for i in range(r // 2):
        f = base ** (-2.0 * i / r)
        for p in range(x.shape[0]):
            a = (first + p) * f
            c, s = math.cos(a), math.sin(a)
            u, v = x[p, :, i], x[p, :, i + r // 2]
            out[p, :, i] = u * c - v * s
            out[p, :, i + r // 2] = v * c + u * s
    return out


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp_min(0)


# ----------------------------------------------------------------------------- recurrent block
def causal_conv(x, w, b, before=None):
    """x [n, C], w [C, taps] (last column: the current token), ``before`` [taps - 1, C] the inputs ahead."""
    taps = w.shape[1]
    pad = torch.zeros(taps - 1, x.shape[1], dtype=x.dtype) if before is None else before
    xs = torch.cat([pad, x])
    return torch.stack([sum(xs[t + k] * w[:, k] for k in range(taps)) + b for t in range(x.shape[0])])


def block_linear(u, m):
    """u [n, nb * s], m [nb, out, in] -> [n, nb * out]: every part by its own matrix."""
    nb, o, s = m.shape
    return torch.cat([u[:, b * s : (b + 1) * s] @ m[b].T for b in range(nb)], -1)


def gated_linear_recurrence(u, r, i, lam, state=None):
    """u, r, i [n, W] -> (states [n, W]): S <- a S + sqrt(1 - a^2) i u with log a = -8 r softplus(lam)."""
    S = torch.zeros(u.shape[1], dtype=u.dtype) if state is None else state
    out = []
    for t in range(u.shape[0]):
        la = -8.0 * r[t] * softplus(lam)
        S = torch.exp(la) * S + torch.sqrt(-torch.expm1(2 * la)) * i[t] * u[t]
        out.append(S)
    return torch.stack(out)


def recurrent_block(h, w):
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = causal_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    r = sigmoid(block_linear(u, w["ra"]) + w["ra.b"].reshape(-1))
    i = sigmoid(block_linear(u, w["ri"]) + w["ri.b"].reshape(-1))
    return (gated_linear_recurrence(u, r, i, w["lam"]) * y) @ w["o"].T


# ----------------------------------------------------------------------------- latent attention
def latent(h, w, c, eps):
    """-> (c [n, rank] normed latent, [n, rot] rotated key part)."""
    z = h @ w["dkv"].T
    lat = rms_norm(z[:, : c["kv_rank"]], w["dkv.norm"], eps)
    return lat, rotate(z[:, None, c["kv_rank"] :], c["rot"]["base"])[:, 0]


def sink_softmax(s, sink):
    """Rows of scores s [n, n] (-inf: not visible): exp(s_j) / (exp(sink) + sum exp(s))."""
    m = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def latent_attention(h, w, c, lat, krot):
    n, H, dim, rot, vd = h.shape[0], c["heads"], c["dim"], c["rot_dim"], c["vdim"]
    q = (h @ w["q"].T).view(n, H, dim + rot)
    qr = rotate(q[..., dim:], c["rot"]["base"])
    k = (lat @ w["uk"].T).view(n, H, dim)
    v = (lat @ w["uv"].T).view(n, H, vd)
    causal = torch.ones(n, n).tril().bool()
    heads = []
    for i in range(H):
        s = (q[:, i, :dim] @ k[:, i].T + qr[:, i] @ krot.T) * c["scale"]
        heads.append(sink_softmax(s.masked_fill(~causal, float("-inf")), w["sink"][i]) @ v[:, i])
    return (torch.cat(heads, -1) * sigmoid(h @ w["g"].T)) @ w["o"].T


# ----------------------------------------------------------------------------- feed-forwards
def expert(x, w):
    return (silu(x @ w["gate"].T) * (x @ w["up"].T)) @ w["down"].T


def route(h, router, top):
    """-> (chosen [n, top] experts, their scores)."""
    s = sigmoid(h @ router.T)
    val, idx = torch.topk(s, top, dim=-1)
    return idx, val


def mixture(h, w, n_experts, top):
    idx, val = route(h, w["router"], top)
    ex = [_sub(w, f"e{e}.") for e in range(n_experts)]
    return torch.stack([sum(expert(val[t, k] * h[t], ex[int(idx[t, k])]) for k in range(top)) for t in range(h.shape[0])])


def _sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, layers=False):
    """cfg: the parsed config.json; weights: name -> tensor.  -> logits [n, vocab] (and, with
    ``layers``, the residual after every layer)."""
    w = {k: v.to(F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    res, kept = [], {}
    for i, L in enumerate(cfg["layers"]):
        p, c = f"l{i}.", L["mixer"]
        h = layer_norm(x, w[p + "norm1"], eps)
        m = _sub(w, p + "mix.")
        if L["type"] == "rglru":
            y = recurrent_block(h, m)
        else:
            if "kv_from" not in c:
                kept[i] = latent(h, m, c, eps)
            y = latent_attention(h, m, c, *kept[c.get("kv_from", i)])
        x = x + layer_norm(y, w[p + "norm1b"], eps)
        f = L.get("mlp")
        if f:
            h = layer_norm(x, w[p + "norm2"], eps)
            m = _sub(w, p + "mlp.")
            y = expert(h, m) if f["kind"] == "dense" else mixture(h, m, f["router"]["experts"], f["router"]["top"])
            x = x + layer_norm(y, w[p + "norm2b"], eps)
        res.append(x)
    logits = layer_norm(x, w["final.norm"], eps) @ w["embed"].T
    return (logits, res) if layers else logits


# ----------------------------------------------------------------------------- test models
def rglru_layer(width, blocks, conv, mlp):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": mlp}


def latent_layer(heads, dim, rot_dim, vdim, kv_rank, mlp, base=10000.0, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
         "rot": {"base": base, "dims": rot_dim}, "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def model_config(width, vocab, layers, eps=1e-5, scale=0.7):
    return {"architecture": "Ripupel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


def random_weights(cfg, seed=0, dtype=torch.bfloat16):
    """Weights that keep every mechanism visible: spread-out attention scores, sinks of the scores' size, strong
    gates, slow and fast recurrent channels.  The first coordinates of a token's embedding rank the experts with
    wide margins and the branches hardly touch them, so no choice of experts is a close call."""
    gen = torch.Generator().manual_seed(seed)
    r = lambda *s, std=1.0, mean=0.0: (mean + torch.randn(*s, generator=gen) * std).to(dtype)  # noqa: E731
    d, V = cfg["width"], cfg["vocab"]
    s = d ** -0.5
    n_exp = max([0] + [L["mlp"]["router"]["experts"] for L in cfg["layers"] if L["mlp"] and L["mlp"]["kind"] == "moe"])
    embed = r(V, d, std=1.5).float()
    for t in range(V):
        for k in range(n_exp):
            embed[t, (t * 7 + k) % n_exp] = 4.0 - 8.0 * k / max(1, n_exp - 1)
    w = {"embed": embed.to(dtype), "final.norm": r(d, mean=1, std=0.2)}

    def out_norm():
        n = r(d, mean=1, std=0.2)
        n[:n_exp] = n[:n_exp] * 0.02
        return n

    for i, L in enumerate(cfg["layers"]):
        p, m, c = f"l{i}.", f"l{i}.mix.", L["mixer"]
        w[p + "norm1"], w[p + "norm1b"] = r(d, mean=1, std=0.2), out_norm()
        if L["type"] == "rglru":
            W, nb = c["width"], c["blocks"]
            k = W // nb
            w.update({m + "y": r(W, d, std=s), m + "y.b": r(W, std=0.3), m + "x": r(W, d, std=s), m + "x.b": r(W, std=0.3),
                      m + "conv": r(W, c["conv"], std=0.6), m + "conv.b": r(W, std=0.3), m + "ra": r(nb, k, k, std=2 * k ** -0.5),
                      m + "ra.b": r(nb, k), m + "ri": r(nb, k, k, std=2 * k ** -0.5), m + "ri.b": r(nb, k),
                      m + "lam": r(W, mean=-4.0, std=2.0), m + "o": r(d, W, std=W ** -0.5)})
        else:
            H, n = c["heads"], c["kv_rank"]
            w.update({m + "q": r(H * (c["dim"] + c["rot_dim"]), d, std=1.6 * s), m + "uk": r(H * c["dim"], n, std=1.6 * n ** -0.5),
                      m + "uv": r(H * c["vdim"], n, std=n ** -0.5), m + "sink": r(H, mean=1.0), m + "g": r(H * c["vdim"], d, std=s),
                      m + "o": r(d, H * c["vdim"], std=(H * c["vdim"]) ** -0.5)})
            if "kv_from" not in c:
                w.update({m + "dkv": r(n + c["rot_dim"], d, std=1.6 * s), m + "dkv.norm": r(n, mean=1, std=0.2)})
        f = L["mlp"]
        if not f:
            continue
        w[p + "norm2"], w[p + "norm2b"] = r(d, mean=1, std=0.2), out_norm()
        w[p + "norm2"][:n_exp] = 1.0
        names, ff = [p + "mlp."], f.get("ff")
        if f["kind"] == "moe":
            E, ff = f["router"]["experts"], f["expert"]["ff"]
            router = r(E, d, std=0.02 * s).float()
            for e in range(E):
                router[e, e] += 1.0
            w[p + "mlp.router"] = router.to(dtype)
            names = [p + f"mlp.e{e}." for e in range(E)]
        for q in names:
            w.update({q + "gate": r(ff, d, std=s), q + "up": r(ff, d, std=s), q + "down": r(d, ff, std=ff ** -0.5)})
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
