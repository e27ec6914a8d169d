"""Small Bevadra configurations for the tests, each unlike the others in every size and constant,
helpers to write them as model folders, configurations drawn from a seed, and weights whose
queries look along one chosen key.

B1: both mixers and a reader: attention of 4 heads of 24 on 2 KV heads with values of 40 behind a
    window of 20; latents of 24 and 40 for 3 heads of 16 + 8 with values of 20, window 33; a layer
    that reads the first one's keys and values through a wider window (50).
B2: latent attention first, without feed-forward; readers in front of and behind a layer with keys
    of its own, one of them with a narrower window; a head of 64, values of 64.
B3: no masks at all (every earlier position is read), heads of 128 on one KV head, a soft cap that bites.
B4: nothing a multiple of 4 or 8: width 50, five heads of 10 with values of 14, windows 7 and 1, latents
    of 22 and 14 for five heads of 6 + 6.
B5: windows of one page, of two tokens and of 130; one head; a reader without a window on a layer that has one.
A1, L1: one mixer each, alone, without feed-forward.  R1: a reader behind its source.
B6, B7: sizes nearer to a real model's layers (heads of 64 and 128, latents of 160 and 448, 20 heads).
"""

import json
import math
import os
import random

import torch

import plain_bevadra as P


def attn(heads, kv, dim, vdim=None, window=0, source=None, scale=None, ff=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim or dim, "scale": scale or 1.2 * dim ** -0.5}
    if window:
        m["mask"] = {"size": window}
    if source is not None:
        m["kv_from"] = source
    return _layer("attention", m, ff)


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, window=0, base=10000.0, scale=None, ff=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": scale or 1.1 * (dim + rot_dim) ** -0.5, "rot": {"dims": rot_dim, "base": base}}
    if window:
        m["mask"] = {"size": window}
    return _layer("latent_attention", m, ff)


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def _cfg(vocab, width, eps, cap, layers):
    return {"architecture": "Bevadra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_softcap": cap,
            "layers": layers}


CONFIGS = {
    "B1": _cfg(90, 64, 1e-6, 20.0, [
        attn(4, 2, 24, 40, window=20, ff=80),
        latent(3, 16, 8, 20, 24, 40, window=33, base=2000.0, ff=96),
        attn(4, 2, 24, 40, window=50, source=0, scale=0.3, ff=56)]),
    "B2": _cfg(128, 128, 1e-5, 30.0, [
        latent(4, 32, 16, 48, 64, 80, window=40),
        attn(4, 1, 64, window=48, ff=72),
        attn(4, 1, 64, window=17, source=1, ff=160),
        attn(8, 8, 16, 32, window=64),
        attn(8, 8, 16, 32, window=64, source=3, ff=64),
        attn(4, 1, 64, window=48, source=1)]),
    "B3": _cfg(101, 72, 1e-4, 4.0, [
        attn(2, 1, 128, ff=40),
        latent(2, 64, 32, 32, 36, 96, base=300.0, ff=56)]),
    "B4": _cfg(61, 50, 1e-5, 12.0, [
        attn(5, 5, 10, 14, window=7, ff=34),
        latent(5, 6, 6, 14, 22, 14, window=9, base=50.0, ff=30),
        attn(5, 5, 10, 14, window=1, source=0, ff=22)]),
    "B5": _cfg(77, 48, 1e-3, 9.0, [
        attn(1, 1, 32, window=16, ff=56),
        latent(1, 8, 4, 8, 12, 20, window=2, ff=40),
        attn(1, 1, 32, source=0, ff=24),
        latent(2, 16, 16, 16, 24, 32, window=130)]),
    "A1": _cfg(50, 32, 1e-5, 25.0, [attn(6, 2, 40, 24, window=20)]),
    "L1": _cfg(50, 40, 1e-5, 25.0, [latent(2, 24, 16, 12, 20, 36, window=21)]),
    "R1": _cfg(50, 40, 1e-5, 25.0, [attn(2, 2, 48, 16, window=11), attn(2, 2, 48, 16, window=30, source=0)]),
    "B6": _cfg(200, 192, 1e-6, 15.0, [
        attn(6, 2, 64, window=100, ff=128),
        latent(6, 64, 32, 64, 96, 160, window=70, base=3000.0, ff=160),
        attn(6, 2, 64, window=100, source=0, ff=128),
        latent(6, 64, 32, 64, 96, 160, window=70, base=3000.0, ff=160),
        attn(6, 2, 64, window=100, source=0, ff=128)]),
    "B7": _cfg(160, 128, 1e-5, 50.0, [
        latent(20, 128, 64, 32, 72, 448, window=140, ff=96),
        attn(4, 4, 128, 96, window=90),
        attn(16, 4, 128, 96, window=200, source=1, ff=72)]),
}


def random_config(seed):
    """A configuration drawn from a seed: two to five layers in any order, every size and constant drawn
    anew (also the values that configurations written by hand tend to make equal or 1)."""
    r = random.Random(seed)
    pick = r.choice
    windows = [0, 1, 2, 5, 16, 17, 31, 32, 33, 50, 64, 100]

    def feed_forward():
        return pick([None, 8, 24, 50, 64, 130])

    layers, owners = [], []
    for i in range(r.randint(2, 5)):
        kind = r.random()
        if owners and kind < 0.35:
            j = pick(owners)
            m = layers[j]["mixer"]
            layers.append(attn(m["kv_heads"] * pick([1, 2, 3]), m["kv_heads"], m["dim"], m["vdim"], window=pick(windows), source=j,
                               scale=r.uniform(0.6, 1.6) * m["dim"] ** -0.5, ff=feed_forward()))
        elif kind < 0.7:
            kv, dim = pick([1, 2, 3, 4]), pick([8, 12, 16, 24, 32, 40, 64, 80, 128])
            owners.append(i)
            layers.append(attn(kv * pick([1, 2, 3]), kv, dim, pick([dim, 8, 20, 48, min(2 * dim, 256)]), window=pick(windows),
                               scale=r.uniform(0.6, 1.6) * dim ** -0.5, ff=feed_forward()))
        else:
            dim, dr = pick([4, 10, 16, 32, 64]), pick([2, 4, 8, 16, 24, 32])
            layers.append(latent(pick([1, 2, 3, 5, 8, 17]), dim, dr, pick([8, 12, 16, 48, 64]), pick([1, 6, 16, 40, 96]),
                                 pick([8, 14, 16, 32, 80, 96, 160]), window=pick(windows), base=pick([30.0, 1000.0, 500000.0]),
                                 scale=r.uniform(0.6, 1.6) * (dim + dr) ** -0.5, ff=feed_forward()))
    return _cfg(pick([40, 97, 256]), pick([24, 32, 50, 64, 96]), pick([1e-6, 1e-5, 1e-3]), pick([3.0, 10.0, 50.0]), layers)


def write_model(out_dir, cfg, seed, store="float32", weights=None):
    """A model folder written with the safetensors library."""
    from safetensors.torch import save_file
    w = weights if weights is not None else P.random_weights(cfg, seed)
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[store]
    os.makedirs(out_dir, exist_ok=True)
    save_file({k: v.to(dt).contiguous() for k, v in w.items()}, os.path.join(out_dir, "model.safetensors"))
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(cfg, f)
    return out_dir


def read_weights(model_dir, as_stored_in=None):
    """The folder's weights as float64 CPU tensors; with as_stored_in="bfloat16" the matrices of the
    products are rounded first, as a bfloat16 engine keeps them (norms, biases and sinks stay in
    32-bit)."""
    from safetensors.torch import load_file
    out = {}
    for k, v in load_file(os.path.join(model_dir, "model.safetensors")).items():
        v = v.float()
        if as_stored_in == "bfloat16" and v.dim() == 2:
            v = v.to(torch.bfloat16).float()
        out[k] = v.double()
    return out


def tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


# ----------------------------------------------------------------------------- aimed weights

def _own_channels(cfg, w, query_token, key_token, layers):
    """Channel 0 of the stream is the query token's own and channel 1 the key token's: every other
    token has (nearly) nothing there behind the norm of any of ``layers``, and no layer in front of
    the last of them writes there."""
    e = w["embed"]
    e -= e.mean(-1, keepdim=True)
    e[:, :2] = 0.0
    e[query_token, 0] = 6.0
    e[key_token, 1] = 6.0
    for i in layers:
        w[f"l{i}.norm1"][:2], w[f"l{i}.norm1.b"][:2] = 1.0, 0.0
    for i in range(max(layers)):
        for t in (f"l{i}.mix.o", f"l{i}.mix.o.b", f"l{i}.mlp.down"):
            if t in w:
                w[t][:2] = 0.0


def aimed_attention(cfg, w, query_token, key_token, layer=0, score=30.0):
    """Changes ``w`` so that in attention layer ``layer`` the query of ``query_token`` looks along the key
    of ``key_token`` wherever it stands, with a score of about ``score``, and finds a value unlike any
    other there.  The keys and values may be those of the layer that ``layer`` reads."""
    m = cfg["layers"][layer]["mixer"]
    source = m.get("kv_from", layer)
    _own_channels(cfg, w, query_token, key_token, sorted({layer, source}))
    g = torch.Generator().manual_seed(99)
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    u = torch.randn(d, generator=g, dtype=torch.float64)
    u = u / u.norm()
    height = 6.0 / 1.4                                 # of the own channel behind the norm, about
    amp = math.sqrt(score / float(m["scale"])) / height
    q, k, v = f"l{layer}.mix.q", f"l{source}.mix.k", f"l{source}.mix.v"
    w[q][:, 0], w[k][:, 1] = amp * u.repeat(H), amp * u.repeat(G)
    w[v][:, 1] = 2.0 * torch.randn(w[v].shape[0], generator=g, dtype=torch.float64)
    return w


def aimed_latent(cfg, w, query_token, key_token, layer=0, score=30.0):
    """The same for latent attention: channel 0 of both latents is the aimed tokens' own, and the
    up-projections turn it into one vector in the unrotated part of every head."""
    m = cfg["layers"][layer]["mixer"]
    H, d, dr, rank, q_rank = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"], m["q_rank"]
    _own_channels(cfg, w, query_token, key_token, [layer])
    g = torch.Generator().manual_seed(98)
    p = f"l{layer}.mix"
    for t, channel in (("dq", 0), ("dkv", 1)):
        w[f"{p}.{t}"][0] = 0.0
        w[f"{p}.{t}"][1:, channel] = 0.0
        w[f"{p}.{t}"][0, channel] = 12.0
    u = torch.randn(d, generator=g, dtype=torch.float64)
    u = u / u.norm()
    # behind the norms channel 0 holds about sqrt(rank) times the norm's weight
    amp = math.sqrt(score / (float(m["scale"]) * math.sqrt(q_rank * rank)
                             * abs(float(w[p + ".dq.norm"][0] * w[p + ".dkv.norm"][0]))))
    for h in range(H):
        w[p + ".uq"][h * (d + dr):h * (d + dr) + d, 0] = amp * u
        w[p + ".uq"][h * (d + dr) + d:(h + 1) * (d + dr), 0] = 0.0
        w[p + ".uk"][h * d:(h + 1) * d, 0] = amp * u
    w[p + ".uv"][:, 0] = 1.5 * torch.randn(w[p + ".uv"].shape[0], generator=g, dtype=torch.float64)
    return w
