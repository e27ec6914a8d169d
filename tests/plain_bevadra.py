"""A plain, slow Bevadra in float64 torch on the CPU: the oracle of the Bevadra tests.

One function per mechanism, written from the equations; nothing here is shared with the
package.  ``cfg`` is the config.json dict, ``w`` a dict of float64 tensors by checkpoint name.
Sequences are handled one at a time and whole.

    x_0     = E[token]                        L(v) = (v - mean) / sqrt(mean((v - mean)^2) + eps) g + b
    h       = L_1(x)
    x'      = x + Mixer(h) + FeedForward(h)   one norm for both; a layer may have no feed-forward
    logits  = c tanh(E L_f(x_L) / c)          the embedding table is the output matrix
"""

import math

import torch

F64 = torch.float64


# ----------------------------------------------------------------------------- small functions

def layer_norm(x, weight, bias, eps):
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * weight + bias


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def slopes(heads):
    """What head h = 0 .. heads - 1 loses per position of distance."""
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def sees(i, j, window):
    """Whether the query at position i reads the key at j: itself and the window - 1 before it
    (window 0: all of them)."""
    return j <= i and (not window or i - j < window)


def window_of(m):
    return int((m.get("mask") or {}).get("size", 0))


def visible(n, window):
    """[n, n]: ``sees`` for every pair of positions."""
    back = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (back >= 0) & (back < (window or n + 1))


def rotate_halves(x, positions, rot):
    """x [n, heads, d]: element i of the first rot.dims of a head turns with element i + dims / 2 by
    p * base^(-2 i / dims)."""
    dims = int(rot["dims"])
    half = dims // 2
    freq = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(half)], dtype=F64)
    ang = torch.as_tensor(positions, dtype=F64)[:, None] * freq[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    out = x.clone()
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


# ----------------------------------------------------------------------------- attention with slopes, a sink and a gate

def softmax_with_sink(scores, sink):
    """Rows of scores (-inf: not seen); the denominator has one more term, exp(sink)."""
    top = torch.maximum(scores.max(-1, keepdim=True).values, torch.as_tensor(sink, dtype=F64))
    e = torch.exp(scores - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def project(h, w, name):
    return h @ w[name].T + w[name + ".b"]


def keys_and_values(h, w, p, m):
    n, G = h.shape[0], m["kv_heads"]
    return project(h, w, p + ".k").reshape(n, G, m["dim"]), project(h, w, p + ".v").reshape(n, G, m["vdim"])


def attend(q, k, v, scale, window, sink):
    """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]; the distance bias is taken off the scaled
    score, the sink gets neither."""
    n, H, _ = q.shape
    G = k.shape[1]
    mask = visible(n, window)
    distance = torch.arange(n, dtype=F64)[:, None] - torch.arange(n, dtype=F64)[None, :]
    out = torch.zeros(n, H, v.shape[2], dtype=F64)
    for h, slope in enumerate(slopes(H)):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * float(scale) - slope * distance
        out[:, h] = softmax_with_sink(s.masked_fill(~mask, float("-inf")), sink[h]) @ v[:, g]
    return out


def attention(h, w, p, m, kv):
    """``kv``: the keys and values this layer reads (its own, or those of the layer it names)."""
    n, H = h.shape[0], m["heads"]
    q = project(h, w, p + ".q").reshape(n, H, m["dim"])
    out = attend(q, kv[0], kv[1], m["scale"], window_of(m), w[p + ".sink"]).reshape(n, H * m["vdim"])
    return project(out * torch.sigmoid(h @ w[p + ".g"].T), w, p + ".o")


# ----------------------------------------------------------------------------- attention through latents

def latent_attention(h, w, p, m, eps, positions):
    H, d, dr, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    n = h.shape[0]
    cq = rms_norm(h @ w[p + ".dq"].T, w[p + ".dq.norm"], eps)
    q = (cq @ w[p + ".uq"].T).reshape(n, H, d + dr)
    down = h @ w[p + ".dkv"].T
    c = rms_norm(down[:, :rank], w[p + ".dkv.norm"], eps)
    k_rot = rotate_halves(down[:, rank:].reshape(n, 1, dr), positions, m["rot"])[:, 0]
    q_rot = rotate_halves(q[..., d:], positions, m["rot"])
    k = (c @ w[p + ".uk"].T).reshape(n, H, d)
    v = (c @ w[p + ".uv"].T).reshape(n, H, dv)
    mask = visible(n, window_of(m))
    out = torch.zeros(n, H, dv, dtype=F64)
    for i in range(H):
        s = (q[:, i, :d] @ k[:, i].T + q_rot[:, i] @ k_rot.T) * float(m["scale"])
        out[:, i] = torch.softmax(s.masked_fill(~mask, float("-inf")), -1) @ v[:, i]
    gate = torch.sigmoid(h @ w[p + ".g"].T)                     # one number a head
    return (out * gate[:, :, None]).reshape(n, H * dv) @ w[p + ".o"].T


# ----------------------------------------------------------------------------- layers and model

def feed_forward(h, w, p):
    return (gelu_tanh(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def forward(cfg, w, tokens, taps=None, rounded=lambda t: t):
    """Logits [n, vocab] of one whole sequence from position 0; ``taps`` (a list) receives the
    stream after every layer; ``rounded`` is applied to what the products of a layer read."""
    eps = float(cfg["norm"]["eps"])
    positions = list(range(len(tokens)))
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    kept = {}                                                   # layer -> its keys and values
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix", layer["mixer"]
        h = rounded(layer_norm(x, w[f"l{i}.norm1"], w[f"l{i}.norm1.b"], eps))
        if layer["type"] == "attention":
            source = m.get("kv_from")
            kept[i] = keys_and_values(h, w, p, m) if source is None else kept[source]
            y = attention(h, w, p, m, kept[i])
        else:
            y = latent_attention(h, w, p, m, eps, positions)
        if layer.get("mlp") is not None:
            y = y + feed_forward(h, w, f"l{i}.mlp")
        x = x + y
        if taps is not None:
            taps.append(x.clone())
    return soft_cap(rounded(layer_norm(x, w["final.norm"], w["final.norm.b"], eps)) @ w["embed"].T,
                    float(cfg["logit_softcap"]))


def greedy(cfg, w, prompt, steps):
    """The ``steps`` tokens that follow ``prompt`` when the likeliest is taken each time."""
    toks = list(prompt)
    for _ in range(steps):
        toks.append(int(torch.argmax(forward(cfg, w, toks)[-1])))
    return toks[len(prompt):]


# ----------------------------------------------------------------------------- random weights

def random_weights(cfg, seed):
    """Weights of a size that keeps every mechanism in play: products of unit scale, sinks and gates
    spread over both sides, means that are not zero."""
    g = torch.Generator().manual_seed(seed)
    d = cfg["width"]

    def mat(o, k):
        return torch.randn(o, k, generator=g, dtype=F64) / math.sqrt(k)

    def vec(n, mean=0.0, spread=0.2):
        return mean + spread * torch.randn(n, generator=g, dtype=F64)

    w = {"embed": 0.4 + 1.3 * torch.randn(cfg["vocab"], d, generator=g, dtype=F64),
         "final.norm": vec(d, 1.0), "final.norm.b": vec(d)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix", layer["mixer"]
        H = m["heads"]
        w[f"l{i}.norm1"], w[f"l{i}.norm1.b"] = vec(d, 1.0), vec(d, 0.0, 0.3)
        if layer["type"] == "attention":
            G, dk, dv = m["kv_heads"], m["dim"], m["vdim"]
            rows = {"q": H * dk}
            if m.get("kv_from") is None:
                rows.update(k=G * dk, v=G * dv)
            for t, n in rows.items():
                w[f"{p}.{t}"], w[f"{p}.{t}.b"] = mat(n, d), vec(n, 0.0, 0.4)
            w[p + ".sink"] = vec(H, 0.5, 1.5)
            w[p + ".g"] = 1.5 * mat(H * dv, d)
            w[p + ".o"], w[p + ".o.b"] = mat(d, H * dv), vec(d, 0.0, 0.3)
        else:
            dk, dr, dv, qr, rank = m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"]
            w[p + ".dq"], w[p + ".uq"] = mat(qr, d), mat(H * (dk + dr), qr)
            w[p + ".dkv"] = mat(rank + dr, d)
            w[p + ".uk"], w[p + ".uv"] = mat(H * dk, rank), mat(H * dv, rank)
            w[p + ".g"], w[p + ".o"] = 1.5 * mat(H, d), mat(d, H * dv)
            w[p + ".dq.norm"], w[p + ".dkv.norm"] = vec(qr, 1.0), vec(rank, 1.0)
        if layer.get("mlp") is not None:
            f = layer["mlp"]["ff"]
            for t, (o, k) in {"gate": (f, d), "up": (f, d), "down": (d, f)}.items():
                w[f"l{i}.mlp.{t}"] = mat(o, k)
    return w
