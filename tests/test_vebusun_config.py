"""The Vebusun configuration reader and plan, on the CPU: what the file's keys become, what is refused, what a file
may leave out, ranks that only the tensors name, the cache manager's pages behind a window and the first ones that
stay, and the plain implementation against sums written out."""
import copy

import pytest
import torch

import plain_vebusun as plain
from imparo_amd.cache.pages import CacheManager, FixedSpec, PagedSpec, kv_spec
from imparo_amd.config import plan_from_config
from imparo_amd.config.errors import BadValue, Inconsistent, MissingKey
from imparo_amd.engine.model import declared_tensors
from imparo_amd.weights import load_weights
from imparo_amd.weights.loader import FreeDim, WeightsError
from vebusun_models import CONFIGS, RANKS, random_weights, write_model


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_plan_declares_the_tensors_the_model_has(name):
    cfg, seed = CONFIGS[name]
    typed, plan = plan_from_config(cfg)
    assert typed.unread_keys == []
    declared = declared_tensors(plan)
    have = random_weights(cfg, seed, RANKS[name])
    assert set(declared) == set(have)
    for k, (decl, _) in declared.items():
        assert len(decl.shape) == have[k].dim(), k
        assert all(isinstance(d, FreeDim) or d == n for d, n in zip(decl.shape, have[k].shape)), k
    assert [c.layer for c in plan.order] == plain.run_order(cfg)


def test_plan_of_a():
    typed, plan = plan_from_config(CONFIGS["A"][0])
    assert (typed.residual_mult, typed.embedding_scale) == (0.45, 2.5)
    assert [c.layer for c in plan.order] == [0, 1, 2, 1, 2, 3]
    assert all(c.cache_of is None for c in plan.order)          # each pass of the loop has a cache or state of its own
    assert [l.mixer.kind for l in plan.layers] == ["channel_delta", "mixer_pair", "channel_delta", "mixer_pair"]
    assert all(l.arrangement == "pre_norm" and l.mixer_norm.kind == "dynamic_tanh" for l in plan.layers)
    assert plan.final_norm.kind == "dynamic_tanh" and plan.embedding["scale"] == 2.5
    assert "ffn" not in plan.layers[2].parts
    a, b = plan.layers[1].mixer["left"], plan.layers[1].mixer["right"]
    assert (a.kind, a["window"], a["keep_first"], a["softcap"], a["scale"], a["sink"]) == ("attention", 21, 5, 6.0, 0.4, "sink")
    assert (a["position"].kind, a["position"]["rotary_dim"], a["position"]["base"]) == ("rope_neox", 8, 500.0)
    # the factors of the sides carry the residual multiplier
    assert a["out_scale"] == pytest.approx(1.3 * 0.45) and b["out_scale"] == pytest.approx(0.7 * 0.45)
    assert (b.kind, b["decay"], b["silu_in"], b["key_scale"], b["gate"]) == ("retention", [0.7, 0.95, 0.999], True, 1.0, "sigmoid")
    assert plan.layers[0].mixer["out_scale"] == 0.45 and plan.layers[0].ffn["out_scale"] == 0.45


def test_what_a_file_leaves_out_is_not_there():
    typed, plan = plan_from_config(CONFIGS["B"][0])
    assert (typed.residual_mult, typed.embedding_scale) == (1.0, 1.0)
    assert [c.layer for c in plan.order] == [0, 1, 2, 3, 4]
    a = plan.layers[0].mixer["left"]
    assert (a["window"], a["keep_first"], a["softcap"], a["position"], a["out_scale"]) == (None, 0, None, None, 1.0)
    c = plan.layers[2].mixer["left"]
    assert (c["window"], c["keep_first"]) == (1, 0)


def _broken(change):
    cfg = copy.deepcopy(CONFIGS["A"][0])
    change(cfg)
    return cfg


@pytest.mark.parametrize("change,error", [
    (lambda c: c.pop("norm"), MissingKey),
    (lambda c: c["layers"][0]["mixer"].pop("kv_heads"), MissingKey),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), MissingKey),
    (lambda c: c["layers"][1]["mixer"].pop("right"), MissingKey),
    (lambda c: c["layers"][1]["mixer"].pop("left_scale"), MissingKey),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("scale"), MissingKey),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].pop("size"), MissingKey),
    (lambda c: c["layers"][1]["mlp"].pop("ff"), MissingKey),
    (lambda c: c["loop"].pop("times"), MissingKey),
    (lambda c: c["layers"][0].update(type="delta"), BadValue),
    (lambda c: c["layers"][1]["mlp"].update(kind="moe"), BadValue),
    (lambda c: c["layers"][1]["mixer"]["left"].update(softcap=0.0), BadValue),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), BadValue),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(keep_first=-1), BadValue),
    (lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.9]), BadValue),
    (lambda c: c["loop"].update(times=0), BadValue),
    (lambda c: c["loop"].update(stop=5), Inconsistent),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), Inconsistent),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=18), Inconsistent),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), Inconsistent),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), Inconsistent),
])
def test_refused_files(change, error):
    with pytest.raises(error):
        plan_from_config(_broken(change))


def test_unknown_keys_are_listed():
    typed, _ = plan_from_config(_broken(lambda c: c.update(dropout=0.1)))
    assert typed.unread_keys == ["dropout"]


def test_inner_ranks_come_from_the_tensors(tmp_path):
    """Any rank loads; a tensor of another number of dimensions or another fixed size does not."""
    cfg, seed = CONFIGS["A"]
    _, plan = plan_from_config(cfg)
    declared = {k: d for k, (d, _) in declared_tensors(plan).items()}
    for ranks in ((1, 7), (40, 3)):
        got = load_weights(write_model(cfg, seed, str(tmp_path / f"r{ranks[0]}"), ranks=ranks), declared)
        assert got["l0.mix.a1"].shape == (ranks[0], 64) and got["l0.mix.g2"].shape == (96, ranks[1])
    bad = write_model(cfg, seed, str(tmp_path / "bad"), overrides={"l0.mix.a1": torch.zeros(12, 63)})
    with pytest.raises(WeightsError, match="l0.mix.a1"):
        load_weights(bad, declared)
    flat = write_model(cfg, seed, str(tmp_path / "flat"), overrides={"l0.mix.a1": torch.zeros(12 * 64)})
    with pytest.raises(WeightsError, match="l0.mix.a1"):
        load_weights(flat, declared)


def test_random_weights_mode_draws_a_model(tmp_path):
    from imparo_amd.weights.random_init import write_random_model
    cfg, _ = CONFIGS["C"]
    d = write_random_model(cfg, 3, str(tmp_path / "m"))
    _, plan = plan_from_config(cfg)
    tensors = load_weights(d, {k: v for k, (v, _) in declared_tensors(plan).items()})
    assert tensors["l0.mix.a1"].shape[0] == tensors["l0.mix.a2"].shape[1]
    assert tensors["final.norm.alpha"].shape == ()
    logits = plain.PlainVebusun(d).logits([1, 2, 3])
    assert torch.isfinite(logits).all()


def test_pages_of_the_first_tokens_stay():
    """Pages wholly behind the window go back to the pool, those that hold first tokens stay until the request ends."""
    spec = kv_spec(2, 16, window=12, keep_first=10)
    assert (spec.window, spec.keep_first) == (12, 10)
    with pytest.raises(ValueError):
        PagedSpec(spec.arrays, keep_first=4)              # without a window everything stays anyway
    m = CacheManager([spec, FixedSpec((3, 4))], page_size=8, n_pages=12, n_slots=2)
    m.admit("a")
    m.reserve("a", 30)
    m.commit("a", 30)                       # the next query, 30, sees 19..30 and 0..9: page 2 (16..23) is still needed
    assert m.table(0, "a") == [0, 1, 2, 3]
    m.reserve("a", 37)
    m.commit("a", 37)                       # the next query, 37, sees 26..37: page 2 has passed, pages 0 and 1 stay
    assert m.table(0, "a") == [0, 1, -1, 3, 4]
    m.reserve("a", 70)
    m.commit("a", 70)
    table = m.table(0, "a")
    assert table[:2] == [0, 1] and table[2:7] == [-1] * 5 and all(p >= 0 for p in table[7:])
    m.check()
    m.release("a")
    assert m.free_pages() == [12]
    # fewer tokens than the first ones that stay: nothing to give back, nothing taken twice
    m.admit("b")
    for n in range(1, 20):
        m.reserve("b", n)
        m.commit("b", n)
    assert m.table(0, "b") == [0, 1, 2]
    m.release("b")
    m.check()
    # beside a group that keeps none: other requests use the pages that came back
    both = CacheManager([spec, kv_spec(2, 16, window=12)], page_size=8, n_pages=6, n_slots=2)
    both.admit("a")
    for n in range(1, 100):
        both.reserve("a", n)
        both.commit("a", n)
    assert both.held_pages("a")[0] == both.held_pages("a")[1] + 2
    both.check()


def test_plain_statements_agree():
    """The plain implementation's mechanisms against sums written out: the mask against loops, the sink and the cap
    as a weighted sum, the linear attention as a sum over earlier tokens, the channel rule as dense matrices."""
    torch.manual_seed(0)
    T, d, dv = 9, 4, 3
    f64 = torch.float64
    pos = torch.arange(T)
    seen = plain.seen_mask(pos, 4, 2)
    for i in range(T):
        for j in range(T):
            assert bool(seen[i, j]) == (j <= i and (i - j < 4 or j < 2))
    q, k, v = torch.randn(T, 2, d, dtype=f64), torch.randn(T, 1, d, dtype=f64), torch.randn(T, 1, dv, dtype=f64)
    sink = torch.tensor([0.3, -1.0], dtype=f64)
    out = plain.capped_sink_attention(q, k, v, seen, 0.7, 1.5, sink)
    for i in range(T):
        for h in range(2):
            s = {j: 1.5 * torch.tanh((q[i, h] @ k[j, 0]) * 0.7 / 1.5) for j in range(T) if seen[i, j]}
            z = sum(torch.exp(x) for x in s.values()) + torch.exp(sink[h])
            assert torch.allclose(out[i, h * dv:(h + 1) * dv], sum(torch.exp(x) / z * v[j, 0] for j, x in s.items()))
    # the channel rule: S_t = (I - b k k^T) diag(g) S_(t-1) + b k v^T, from one model's layer
    cfg, seed = CONFIGS["A"]
    w = {n: t.to(f64) for n, t in random_weights(cfg, seed).items()}
    mx = cfg["layers"][2]["mixer"]
    h = torch.randn(7, 64, dtype=f64)
    got = plain.channel_delta(h, w, "l2", mx, 1e-6)
    H, dk, dvv = mx["heads"], mx["dim"], mx["vdim"]
    proj = lambda n, c: plain.silu(plain.causal_conv(h @ w[f"l2.mix.{n}"].T, w[f"l2.mix.{n}.conv"])).reshape(7, c, -1)
    Q, K, V = proj("q", H), proj("k", H), proj("v", H)
    Q = Q / torch.sqrt((Q * Q).sum(-1, keepdim=True) + 1e-6) / dk ** 0.5
    K = K / torch.sqrt((K * K).sum(-1, keepdim=True) + 1e-6)
    dt = plain.softplus(h @ w["l2.mix.a1"].T @ w["l2.mix.a2"].T + w["l2.mix.dt_bias"])
    beta = torch.sigmoid(h @ w["l2.mix.b"].T)
    o = torch.zeros(7, H, dvv, dtype=f64)
    for hd in range(H):
        S = torch.zeros(dk, dvv, dtype=f64)
        for t in range(7):
            g = torch.exp(-torch.exp(w["l2.mix.A_log"][hd]) * dt[t, hd * dk:(hd + 1) * dk])
            kk = K[t, hd]
            S = (torch.eye(dk, dtype=f64) - beta[t, hd] * torch.outer(kk, kk)) @ torch.diag(g) @ S + beta[t, hd] * torch.outer(kk, V[t, hd])
            o[t, hd] = S.T @ Q[t, hd]
    o = plain.unit_rms(o, 1e-6) * w["l2.mix.norm"]
    want = (o.reshape(7, -1) * torch.sigmoid(h @ w["l2.mix.g1"].T @ w["l2.mix.g2"].T)) @ w["l2.mix.o"].T
    assert torch.allclose(got, want)
