"""The numpy statement of the Ludalix mechanisms pinned to closed forms, and its configuration reader."""
from __future__ import annotations

import copy

import numpy as np
import pytest

import ludalix_fixture as lf
import ludalix_oracle as lo
from homura_amd import runtime


def test_position_waves():
    w = lo.position_waves([0, 3], 5)
    assert np.allclose(w[0], [0, 1, 0, 1, 0])
    a = 10000.0 ** (-2 / 5)
    assert np.allclose(w[1], [np.sin(3), np.cos(3), np.sin(3 * a), np.cos(3 * a), np.sin(3 * a * a)])


def test_unit_rms_has_eps_inside_the_root():
    assert np.allclose(lo.unit_rms(np.array([[3.0, 4.0]]), 0.0), [[3 / np.sqrt(12.5), 4 / np.sqrt(12.5)]])
    assert np.allclose(lo.unit_rms(np.full((1, 2), 1e-3), 3e-6), 1e-3 / np.sqrt(4e-6))


def plain_memory(q, k, v, i, f):
    """The unstabilised sums: e^m cancels except in the floor of the divisor."""
    T = len(q)
    out = np.zeros_like(v)
    for t in range(T):
        w = np.array([np.exp(i[s] + f[s + 1:t + 1].sum()) for s in range(t + 1)])
        dots = (k[:t + 1] @ q[t]) * w
        top = max(f[:t + 1].sum(), max(i[s] + f[s + 1:t + 1].sum() for s in range(t + 1)))
        scale = np.exp(-top)
        out[t] = scale * (dots @ v[:t + 1]) / (max(abs(scale * dots.sum()), scale) + 1e-6)
    return out


@pytest.mark.parametrize("level", [-4.0, 0.0, 5.0])
def test_matrix_memory_closed_form(level):
    rng = np.random.default_rng(3)
    q, k = rng.standard_normal((2, 9, 4))
    v = rng.standard_normal((9, 3))
    i, f = level + rng.standard_normal(9), lo.log_sigmoid(rng.standard_normal(9))
    assert np.allclose(lo.matrix_memory(q, k, v, i, f), plain_memory(q, k, v, i, f))


def test_the_running_maximum_starts_at_zero():
    one = np.ones((1, 1))
    assert np.isclose(lo.matrix_memory(one, one, one, np.array([-3.0]), np.array([0.0]))[0, 0], np.exp(-3) / (1 + 1e-6))
    assert np.isclose(lo.matrix_memory(one, one, one, np.array([-3.0]), np.array([-2.0]))[0, 0], np.exp(-1) / (np.exp(2) + 1e-6))
    assert np.isclose(lo.matrix_memory(one, one, one, np.array([3.0]), np.array([0.0]))[0, 0], 1 / (1 + 1e-6))


def test_gate_functions():
    z = np.linspace(-40, 40, 17)
    assert np.allclose(lo.log_sigmoid(z), -np.logaddexp(0, -z))
    assert np.allclose(lo.soft_cap(z, 3.0), 3 * np.tanh(z / 3))


def test_who_sees_whom():
    seen = lo.visible(8, 3, 2)
    for i in range(8):
        assert [j for j in range(8) if seen[i, j]] == sorted({j for j in range(i + 1) if i - j < 3 or j < 2})
    assert np.array_equal(lo.visible(5, 0, 0), np.tri(5, dtype=bool))


def test_query_heads_share_key_heads_in_order():
    cfg = lf.config([lf.attn(heads=4, kv_heads=2, dim=3, vdim=2, window=None)], width=8)
    w = {k: np.asarray(v, np.float64) for k, v in lf.weights(cfg, 1).items()}
    h = np.random.default_rng(0).standard_normal((1, 8))
    t = {k[7:]: v for k, v in w.items() if k.startswith("l0.mix.")}
    k, v = lo.attention_keys(h, cfg["layers"][0]["mixer"], t, 1e-6)
    t["o"] = np.eye(8)  # one token: every head returns its value head
    assert np.allclose(lo.attention(h, cfg["layers"][0]["mixer"], t, 1e-6, k, v)[0], np.concatenate([v[0, 0], v[0, 0], v[0, 1], v[0, 1]]))


def test_clamped_glu():
    one = np.ones((1, 1))
    y = lambda g, u, limit=2.0: lo.clamped_glu(np.array([[g, u]]), np.array([[1.0, 0]]), np.array([[0, 1.0]]), one, limit)[0, 0]
    s = lambda z: z / (1 + np.exp(-1.702 * z))
    assert np.isclose(y(1.0, 0.5), s(1.0) * 1.5)
    assert np.isclose(y(9.0, 0.5), s(2.0) * 1.5) and np.isclose(y(-9.0, 0.5), s(-9.0) * 1.5)
    assert np.isclose(y(1.0, 9.0), s(1.0) * 3) and np.isclose(y(1.0, -9.0), -s(1.0))


def test_experts_see_their_weight_on_the_input():
    rng = np.random.default_rng(5)
    h, router = rng.standard_normal((4, 6)), rng.standard_normal((3, 6))
    t = {"router": router}
    for e in range(3):
        t |= {f"e{e}.gate": rng.standard_normal((2, 6)), f"e{e}.up": rng.standard_normal((2, 6)), f"e{e}.down": rng.standard_normal((6, 2))}
    chosen, weight = lo.route(h, router, 2)
    for r in range(4):
        order = np.argsort(-(router @ h[r]))
        assert list(chosen[r]) == list(order[:2]) and np.allclose(weight[r], lo.sigmoid(router @ h[r])[order[:2]])
    y = lo.mixture(h, {"router": {"experts": 3, "top": 2}}, t)
    want = sum(weight[0, p] and lo.expert(weight[0, p] * h[0], *(t[f"e{chosen[0, p]}.{n}"] for n in ("gate", "up", "down"))) for p in range(2))
    assert np.allclose(y[0], want)


def test_positions_only_see_the_past_and_shared_keys_are_the_source_layers():
    layers = [lf.memory(mlp=lf.dense()), lf.attn(mlp=lf.moe()), lf.attn(kv_from=1, window=4, keep=1)]
    cfg = lf.config(layers)
    w = lf.weights(cfg, 4)
    toks = np.random.default_rng(4).integers(0, cfg["vocab"], 12)
    full, trail = lo.forward(cfg, w, toks)
    assert trail.shape == (3, 12, cfg["width"])
    assert np.allclose(full[:7], lo.forward(cfg, w, toks[:7])[0])
    changed = dict(w, **{"l1.mix.v": 2 * w["l1.mix.v"]})
    other = lo.forward(dict(cfg, layers=layers), changed, toks)[1]
    assert np.allclose(other[0], trail[0]) and not np.allclose(other[2] - other[1], trail[2] - trail[1])


# ── configuration reader ──

def test_config_reader_takes_the_design():
    layers = [lf.memory(mlp=lf.moe()), lf.attn(mlp=lf.dense()), lf.attn(kv_from=1, window=None), lf.attn(window=3, keep=0)]
    assert runtime.block_layer_runs(lf.config(layers)) == [0, 1, 2, 3]


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda c: c["layers"][0]["mixer"].update(gate_cap=0), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=0), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(dim=21), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "mlp.kind"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=6), "top"),
    (lambda c: c["layers"][1]["mlp"].pop("expert"), "expert.ff"),
    (lambda c: c.update(architecture="Unheard"), "Unheard"),
])
def test_config_reader_names_what_is_wrong(change, message):
    cfg = lf.config([lf.memory(mlp=lf.dense()), lf.attn(mlp=lf.moe()), lf.attn(kv_from=1), lf.attn(kv_from=1)])
    bad = copy.deepcopy(cfg)
    change(bad)
    runtime.block_layer_runs(cfg)
    with pytest.raises(ValueError, match=message):
        runtime.block_layer_runs(bad)
