"""The plain Bevadra (tests/plain_bevadra.py) against identities of its own, and the configuration
reader, the model builder and the plan of shared caches, without a GPU."""

import copy
import math

import pytest
import torch

import bevadra_tiny as T
import plain_bevadra as P

F64 = torch.float64


def randn(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_layer_norm_takes_off_the_mean_and_divides_by_the_deviation():
    x = 3.0 + 2.0 * randn(5, 40)
    y = P.layer_norm(x, torch.ones(40, dtype=F64), torch.zeros(40, dtype=F64), 1e-9)
    assert y.mean(-1).abs().max() < 1e-12 and (y.var(-1, unbiased=False) - 1).abs().max() < 1e-6
    w, b = randn(40, seed=1), randn(40, seed=2)
    assert torch.allclose(P.layer_norm(x, w, b, 1e-3), torch.nn.functional.layer_norm(x, (40,), w, b, 1e-3), atol=1e-12)
    assert torch.allclose(P.layer_norm(x + 17.0, w, b, 1e-3), P.layer_norm(x, w, b, 1e-3), atol=1e-10)


def test_the_window_counts_the_position_itself():
    assert P.sees(100, 100, 8) and P.sees(100, 93, 8) and not P.sees(100, 92, 8) and not P.sees(5, 6, 8)
    assert all(P.sees(50, j, 0) for j in range(51))
    for window in (0, 1, 7, 40):
        got = P.visible(30, window)
        assert all(bool(got[i, j]) == P.sees(i, j, window) for i in range(30) for j in range(30))


def test_slopes_fall_from_head_to_head():
    assert P.slopes(8) == [2.0 ** -(h + 1) for h in range(8)]
    assert P.slopes(1) == [2.0 ** -8] and abs(P.slopes(3)[0] - 2.0 ** (-8 / 3)) < 1e-15


def test_a_sink_is_a_key_with_a_score_of_its_own_and_no_value():
    s = randn(4, 9)
    p = P.softmax_with_sink(s, torch.tensor(0.7, dtype=F64))
    full = torch.softmax(torch.cat([s, torch.full((4, 1), 0.7, dtype=F64)], dim=1), -1)
    assert torch.allclose(p, full[:, :9], atol=1e-14) and (p.sum(-1) < 1).all()
    # far below the scores it does nothing, far above them it takes everything
    assert torch.allclose(P.softmax_with_sink(s, torch.tensor(-900.0, dtype=F64)), torch.softmax(s, -1))
    assert P.softmax_with_sink(s, torch.tensor(900.0, dtype=F64)).max() == 0.0


def test_with_a_sink_the_bias_must_be_taken_of_the_distance():
    """Without a sink, slope * (i - j) and -slope * j are the same softmax; with one they are not."""
    n, d = 30, 8
    q, k, v = randn(n, 2, d, seed=3), randn(n, 1, d, seed=4), randn(n, 1, d, seed=5)
    none, some = torch.full((2,), -1e9, dtype=F64), torch.zeros(2, dtype=F64)

    def other_form(sink):
        out = torch.zeros(n, 2, d, dtype=F64)
        for h, slope in enumerate(P.slopes(2)):
            s = (q[:, h] @ k[:, 0].T) * 0.3 + slope * torch.arange(n, dtype=F64)[None, :]
            out[:, h] = P.softmax_with_sink(s.masked_fill(~P.visible(n, 9), float("-inf")), sink[h]) @ v[:, 0]
        return out
    assert torch.allclose(P.attend(q, k, v, 0.3, 9, none), other_form(none), atol=1e-12)
    assert (P.attend(q, k, v, 0.3, 9, some) - other_form(some)).abs().max() > 1e-2


def test_soft_cap():
    z = torch.tensor([-1e9, -3.0, 0.0, 1e-6, 3.0, 1e9], dtype=F64)
    y = P.soft_cap(z, 5.0)
    assert y[0] == -5.0 and y[-1] == 5.0 and abs(y[3] - 1e-6) < 1e-15 and abs(y[4] - 5 * math.tanh(0.6)) < 1e-15


def test_rotation_keeps_lengths_and_scores_depend_on_the_distance():
    rot = {"dims": 8, "base": 100.0}
    x, y = randn(1, 1, 12, seed=6), randn(1, 1, 12, seed=7)
    a = (P.rotate_halves(x, [5], rot) * P.rotate_halves(y, [2], rot)).sum()
    b = (P.rotate_halves(x, [105], rot) * P.rotate_halves(y, [102], rot)).sum()
    assert abs(a - b) < 1e-9 and torch.equal(P.rotate_halves(x, [7], rot)[..., 8:], x[..., 8:])
    assert abs(P.rotate_halves(x, [7], rot).norm() - x.norm()) < 1e-12


def test_latent_attention_with_folded_products():
    """The score against the latent itself and the value product behind the softmax give the
    numbers of the definition."""
    cfg = T.CONFIGS["L1"]
    w = P.random_weights(cfg, 9)
    m, p, eps, n = cfg["layers"][0]["mixer"], "l0.mix", cfg["norm"]["eps"], 33
    h = randn(n, cfg["width"], seed=4)
    want = P.latent_attention(h, w, p, m, eps, list(range(n)))
    H, d, dr, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (P.rms_norm(h @ w[p + ".dq"].T, w[p + ".dq.norm"], eps) @ w[p + ".uq"].T).reshape(n, H, d + dr)
    down = h @ w[p + ".dkv"].T
    c = P.rms_norm(down[:, :rank], w[p + ".dkv.norm"], eps)
    kr = P.rotate_halves(down[:, rank:].reshape(n, 1, dr), list(range(n)), m["rot"])[:, 0]
    qr = P.rotate_halves(q[..., d:], list(range(n)), m["rot"])
    gate = torch.sigmoid(h @ w[p + ".g"].T)
    out = torch.zeros(n, H, dv, dtype=F64)
    for hd in range(H):
        folded = q[:, hd, :d] @ w[p + ".uk"][hd * d:(hd + 1) * d]
        s = (folded @ c.T + qr[:, hd] @ kr.T) * m["scale"]
        s = s.masked_fill(~P.visible(n, m["mask"]["size"]), float("-inf"))
        out[:, hd] = gate[:, hd:hd + 1] * ((torch.softmax(s, -1) @ c) @ w[p + ".uv"][hd * dv:(hd + 1) * dv].T)
    assert torch.allclose(out.reshape(n, H * dv) @ w[p + ".o"].T, want, atol=1e-10)


def test_a_reader_uses_its_sources_keys_and_values():
    """A layer that reads another's keys and values equals one with those tensors of its own only if it
    also saw the source's input."""
    cfg = T.CONFIGS["R1"]
    w = P.random_weights(cfg, 3)
    assert not any(k.startswith(("l1.mix.k", "l1.mix.v")) for k in w) and "l1.mix.sink" in w
    h0, h1 = randn(20, cfg["width"], seed=1), randn(20, cfg["width"], seed=2)
    m = cfg["layers"][1]["mixer"]
    kv = P.keys_and_values(h0, w, "l0.mix", m)
    y = P.attention(h1, w, "l1.mix", m, kv)
    own = dict(w)
    own.update({f"l1.mix.{t}": w[f"l0.mix.{t}"] for t in ("k", "k.b", "v", "v.b")})
    assert not torch.allclose(y, P.attention(h1, own, "l1.mix", m, P.keys_and_values(h1, own, "l1.mix", m)))
    assert torch.allclose(P.attention(h0, w, "l1.mix", m, kv),
                          P.attention(h0, own, "l1.mix", m, P.keys_and_values(h0, own, "l1.mix", m)))


def test_both_sublayers_read_the_same_norm():
    cfg = T.CONFIGS["B3"]
    w = P.random_weights(cfg, 4)
    toks, taps = T.tokens(cfg, 6, 1), []
    P.forward(cfg, w, toks, taps)
    x0 = w["embed"][torch.tensor(toks)]
    h = P.layer_norm(x0, w["l0.norm1"], w["l0.norm1.b"], cfg["norm"]["eps"])
    m = cfg["layers"][0]["mixer"]
    y = P.attention(h, w, "l0.mix", m, P.keys_and_values(h, w, "l0.mix", m)) + P.feed_forward(h, w, "l0.mlp")
    assert torch.allclose(taps[0], x0 + y, atol=1e-12)


# ----------------------------------------------------------------------------- configuration and builder

@pytest.mark.parametrize("name", sorted(T.CONFIGS) + [f"seed{i}" for i in range(8)])
def test_configuration_round_trip_and_tensor_list(name):
    from kllm_amd.config import config_from_dict
    from kllm_amd.config.registry import resolve_architecture
    from kllm_amd.engine.model import collect_weight_specs
    raw = T.CONFIGS[name] if name in T.CONFIGS else T.random_config(int(name[4:]))
    cfg = config_from_dict(raw)
    assert cfg.to_dict() == raw
    spec = resolve_architecture(raw).build(cfg)
    specs = {s.name: tuple(s.shape) for s in collect_weight_specs(spec)}
    assert specs == {k: tuple(v.shape) for k, v in P.random_weights(raw, 1).items()}
    assert [r.layer for r in spec.schedule] == list(range(len(raw["layers"])))
    assert [r.cache_of for r in spec.schedule] == [l["mixer"].get("kv_from") for l in raw["layers"]]


def _set(*path):
    *keys, last, value = path

    def change(c):
        for k in keys:
            c = c[k]
        c[last] = value
    return change


@pytest.mark.parametrize("change,word", [
    (_set("layers", 0, "type", "delta"), "type"),
    (_set("layers", 2, "mixer", "kv_from", 2), "kv_from"),
    (_set("layers", 2, "mixer", "kv_from", 9), "kv_from"),
    (_set("layers", 2, "mixer", "kv_from", 1), "kv_from"),
    (_set("layers", 2, "mixer", "kv_heads", 4), "kv_heads"),
    (_set("layers", 2, "mixer", "vdim", 24), "vdim"),
    (_set("layers", 0, "mixer", "kv_heads", 3), "kv_heads"),
    (_set("layers", 1, "mixer", "rot", "dims", 6), "rot_dim"),
    (_set("layers", 1, "mixer", "rot_dim", 7), "rot_dim"),
    (_set("layers", 0, "mixer", "mask", "size", 0), "size"),
    (_set("layers", 0, "mlp", "kind", "moe"), "dense"),
    (lambda c: c.pop("logit_softcap"), "logit_softcap"),
    (lambda c: c["layers"][1]["mixer"].pop("q_rank"), "q_rank"),
])
def test_configurations_that_are_refused(change, word):
    from kllm_amd.config import ConfigError, config_from_dict
    raw = copy.deepcopy(T.CONFIGS["B1"])
    change(raw)
    with pytest.raises(ConfigError) as e:
        config_from_dict(raw)
    assert word in str(e.value)


def _plan(raw):
    from kllm_amd.config import config_from_dict
    from kllm_amd.config.registry import resolve_architecture
    from kllm_amd.engine.model import Model
    from kllm_amd.parts.base import Runtime
    return Model(resolve_architecture(raw).build(config_from_dict(raw)), Runtime(torch.device("cpu"), torch.float32)).cache_plan


def test_a_shared_cache_is_kept_for_the_widest_reader():
    plan = _plan(T.CONFIGS["B1"])
    g, entry, writes = plan.runs[0]
    assert writes and plan.runs[2] == (g, entry, False)
    assert plan.groups[g].need.window == 50 and plan.groups[g].entries == 1           # the reader's, not its own 20
    # one page width for keys of 24 and values of 40
    assert (plan.groups[g].need.head_dim, plan.groups[g].need.value_width) == (64, 64)
    latent = plan.groups[plan.runs[1][0]].need
    assert (latent.window, latent.kv_heads, latent.head_dim, latent.value_width) == (33, 1, 48, 40)
    plan = _plan(T.CONFIGS["B5"])
    assert plan.groups[plan.runs[0][0]].need.window == 0          # the reader has no window: every position is kept
    plan = _plan(T.CONFIGS["B2"])
    assert [r[2] for r in plan.runs] == [True, True, False, True, False, False]
    assert plan.runs[2][:2] == plan.runs[1][:2] == plan.runs[5][:2]
    assert plan.groups[plan.runs[1][0]].need.window == 48         # a narrower reader changes nothing
    assert plan.runs[4][:2] == plan.runs[3][:2]


def test_needs_that_differ_in_more_than_the_window_share_no_cache():
    from kllm_amd.parts.spec import CacheNeed
    a = CacheNeed("paged", kv_heads=2, head_dim=64, window=20)
    assert a.alike(CacheNeed("paged", kv_heads=2, head_dim=64, window=0)) and not a.alike(CacheNeed("paged", kv_heads=2, head_dim=32))
    assert not a.alike(CacheNeed("state", state_shape=(4,)))
    assert a.covering(CacheNeed("paged", kv_heads=2, head_dim=64, window=33)).window == 33
    assert a.covering(CacheNeed("paged", kv_heads=2, head_dim=64, window=7)).window == 20
    whole = a.covering(CacheNeed("paged", kv_heads=2, head_dim=64, window=0, keep_first=3))
    assert (whole.window, whole.keep_first) == (0, 0)
    kept = a.covering(CacheNeed("paged", kv_heads=2, head_dim=64, window=9, keep_first=3))
    assert (kept.window, kept.keep_first) == (20, 3)


# ----------------------------------------------------------------------------- the aimed weights do aim

@pytest.mark.parametrize("name,layer,kind", [("B1", 0, "attention"), ("B1", 2, "attention"), ("L1", 0, "latent")])
def test_aimed_queries_find_their_key(name, layer, kind):
    cfg = T.CONFIGS[name]
    w = (T.aimed_attention if kind == "attention" else T.aimed_latent)(cfg, P.random_weights(cfg, 2), 1, 2, layer)
    W = P.window_of(cfg["layers"][layer]["mixer"])
    toks = [3 + t % (cfg["vocab"] - 3) for t in T.tokens(cfg, W + 20, 3)]
    toks[W + 9] = 1
    plain = P.forward(cfg, w, toks)[W + 9]
    seen = list(toks)
    seen[10] = 2                                                # the window's oldest position
    assert (P.forward(cfg, w, seen)[W + 9] - plain).norm() > 0.3 * plain.norm()
