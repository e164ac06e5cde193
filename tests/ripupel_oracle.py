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
