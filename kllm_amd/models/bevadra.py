"""The Bevadra decoder, put together from parts.

Token embedding; layers in the order the configuration lists them, each with one layer norm (mean,
variance, weight and bias) whose output both the mixer and the feed-forward read (x' = x + mixer +
feed-forward).  A mixer is one of two.  ``attention``: projections with biases, no rotation, a
distance bias, a window, a learned sink per head in the softmax and a gate per element on the
output; a layer may read the keys and values that an earlier one cached (with a window of its
own).  ``latent_attention``: attention through low-rank latents behind a window, with a gate per
head.  The feed-forward is dense and gated (the tanh form of gelu), or absent.  A final layer norm,
the embedding table as the output matrix, and a soft cap on the logits.  Tensor names: ``embed``,
``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``; a bias is its weight's name with ``.b``.
"""

from __future__ import annotations

from ..config.bevadra import BevadraConfig
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, Run

# The distance bias of head h of H is 2^(-8 (h + 1) / H) per position.
DISTANCE_SLOPE_BITS = 8


def build_bevadra(cfg: BevadraConfig) -> ModelSpec:
    d = cfg.width

    def norm(name):
        return PartSpec("layer_norm", size=d, eps=cfg.norm_eps, names={"weight": name, "bias": name + ".b"})

    positions = {}      # mixers that rotate alike share one position part (and its tables of a step)

    def position(dims, base):
        if (dims, base) not in positions:
            positions[dims, base] = PartSpec("rotary_scaled", rotary_dim=dims, base=base, interleaved=False)
        return positions[dims, base]

    def attention(p, m):
        own = m.kv_from is None
        names = {f"{t}.weight": f"{p}.{t}" for t in ("q", "k", "v", "g", "o")}
        names.update({f"{t}.bias": f"{p}.{t}.b" for t in ("q", "k", "v", "o")})
        names["sink"] = f"{p}.sink"
        return PartSpec("attention_bias", p, hidden=d, heads=m.heads, kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim,
                        scale=m.scale, window=m.window, distance_slope_bits=DISTANCE_SLOPE_BITS, sink="learned", gate=True,
                        own_kv=own, names=names)

    def latent(p, m):
        names = {f"{t}.weight": f"{p}.{t}" for t in ("dq", "uq", "dkv", "uk", "uv", "g", "o")}
        names.update({"dq.norm": f"{p}.dq.norm", "dkv.norm": f"{p}.dkv.norm"})
        return PartSpec("latent_attention", p, hidden=d, heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim,
                        value_dim=m.vdim, q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale, eps=cfg.norm_eps,
                        window=m.window, gate="head", position=position(m.rot_dim, m.rot_base), names=names)

    layers, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.mix", layer.mixer
        mixer = attention(p, m) if layer.type == "attention" else latent(p, m)
        ff = None
        if layer.ff is not None:
            f = f"l{i}.mlp"
            ff = PartSpec("gated_mlp", f, hidden=d, intermediate=layer.ff, activation="gelu_tanh",
                          names={f"{t}_proj.weight": f"{f}.{t}" for t in ("gate", "up", "down")})
        layers.append(LayerSpec(mixer=mixer, feed_forward=ff, norm_mixer=norm(f"l{i}.norm1"), block="parallel"))
        schedule.append(Run(i, cache_of=getattr(m, "kv_from", None)))
    return ModelSpec(
        embedding=PartSpec("token_embedding", vocab=cfg.vocab, hidden=d, names={"weight": "embed"}),
        layers=layers,
        schedule=schedule,
        final_norm=norm("final.norm"),
        head=PartSpec("linear_head", vocab=cfg.vocab, hidden=d, soft_cap=cfg.logit_softcap, names={"weight": "embed"}),
        vocab_size=cfg.vocab,
        hidden_size=d,
    )


register_architecture("Bevadra", BevadraConfig, build_bevadra)
