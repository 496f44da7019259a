"""The Pumozen design without a GPU: its config.json reader, its plan over the library's parts, what its layers ask of the
cache, and the plain implementation's own mechanisms against closed forms."""
import copy
import math

import numpy as np
import pytest

import plain_pumozen as plain
from pumozen_cases import CASES, random_case, tensors
from turboquant_cpp_amd.config.base import ConfigError
from turboquant_cpp_amd.config.plan import PartSpec
from turboquant_cpp_amd.config.registry import config_from_dict
from turboquant_cpp_amd.engine.model import model_from_config
from turboquant_cpp_amd.parts.base import build_part


@pytest.mark.parametrize("case", sorted(CASES))
def test_config_round_trip_and_tensor_table(case):
    cfg = CASES[case]
    arch, typed = config_from_dict(cfg)
    assert arch.name == "Pumozen" and arch.config_to_json(typed) == cfg
    table = model_from_config(cfg, "float32").tensor_table()
    w = tensors(cfg, 0)
    assert set(table) == set(w)
    for name, (shape, _role) in table.items():
        assert tuple(shape) == w[name].shape, name


def test_random_cases_are_read():
    for seed in range(60):
        cfg = random_case(seed)
        arch, typed = config_from_dict(cfg)
        assert arch.config_to_json(typed) == cfg
        table, w = model_from_config(cfg, "bfloat16").tensor_table(), tensors(cfg, seed)
        assert {n: tuple(s) for n, (s, _) in table.items()} == {n: a.shape for n, a in w.items()}


def test_what_the_reader_refuses():
    good = CASES["odd"]

    def broken(change):
        cfg = copy.deepcopy(good)
        change(cfg)
        with pytest.raises(ConfigError):
            config_from_dict(cfg)
    mixer = lambda i, **kw: (lambda c: c["layers"][i]["mixer"].update(**kw))
    broken(lambda c: c["layers"][0].update(type="linear"))
    broken(lambda c: c["layers"][0].pop("mixer"))
    broken(mixer(0, kv_heads=4))
    broken(mixer(0, vdim=16))                               # the values are the keys
    broken(mixer(0, rot={"dims": 22, "base": 1e4}))
    broken(mixer(0, rot={"dims": 7, "base": 1e4}))
    broken(mixer(0, rot={"dims": 8}))
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    broken(mixer(1, groups=4))
    broken(mixer(1, norm_groups=5))
    broken(mixer(1, conv=0))
    broken(lambda c: c["layers"][1]["mixer"].pop("state"))
    broken(mixer(2, q_temp={"coef": 0.1, "every": 0}))
    broken(lambda c: c["layers"][2]["mixer"].pop("diff"))
    broken(mixer(3, kv_from=3))
    broken(mixer(3, kv_from=0))                             # a layer of another type
    broken(mixer(6, kv_from=3))                             # which has no keys of its own
    broken(mixer(3, dim=16))
    broken(lambda c: c["layers"][1]["mlp"].pop("limit"))
    broken(lambda c: c["layers"][1]["mlp"].update(kind="glu"))
    broken(lambda c: c["layers"][2]["mlp"]["router"].update(top=9))
    broken(lambda c: c["layers"][2]["mlp"]["shared"].pop("limit"))
    broken(lambda c: c["layers"][2]["mlp"]["expert"].update(limit=-1.0))
    broken(lambda c: c["token_side"].update(dim=0))
    broken(lambda c: c["norm"].pop("eps"))
    broken(lambda c: c.update(layers=[]))


def test_what_its_layers_keep():
    model = model_from_config(CASES["odd"], "float32")
    needs = model.cache_needs()
    for (kv, state, of), layer in zip(needs, CASES["odd"]["layers"]):
        m = layer["mixer"]
        assert of == m.get("kv_from")
        if layer["type"] == "mamba2":
            C = m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            floats = m["heads"] * m["state"] * m["vdim"] + C * (m["conv"] - 1)
            assert kv is None and state.shape == (-(-floats // 4) * 4,)
        else:
            assert state is None and kv.num_kv_heads == m["kv_heads"] and kv.window is None
            wide = m["dim"] if layer["type"] == "attention" else 2 * max(m["dim"], math.ceil(m["vdim"] / 2))
            assert wide <= kv.head_dim < wide + 32 and kv.head_dim % 16 == 0
    assert model.plan.token_table_width == 7 * 12
    bare = model_from_config(CASES["attention_only"], "float32")
    assert bare.plan.token_table is None and bare.blocks[0].side is None and bare.blocks[0].ffn is None


def test_parts_that_do_not_fit_are_refused():
    attn = dict(hidden_size=32, num_heads=2, num_kv_heads=1, head_dim=16, position=PartSpec("none"), separate_qkv=True)
    for bad in (dict(values_are_keys=True), dict(row_norm_eps=1e-5, qk_norm_eps=1e-5), dict(row_norm_eps=-1.0), dict(unit_sink=True, sink=True),
                dict(row_norm_eps=1e-5, values_are_keys=True, value_dim=8), dict(row_norm_eps=1e-5, head_gate=True)):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("gqa_attention", {**attn, **bad}))
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("gqa_attention", {**attn, "separate_qkv": False, "unit_sink": True}))
    diff = dict(hidden_size=32, num_heads=4, num_kv_heads=2, head_dim=8, value_dim=16, eps=1e-5, diff=0.5)
    for bad in (dict(num_kv_heads=3), dict(temperature=(0.1, 0.0))):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("differential_attention", {**diff, **bad}))
    ssd = dict(hidden_size=32, num_heads=4, value_dim=8, state_dim=16, groups=2, conv_taps=4, norm_parts=2, eps=1e-5)
    for bad in (dict(groups=3), dict(norm_parts=3), dict(state_dim=0), dict(conv_taps=0)):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("ssd", {**ssd, **bad}))
    with pytest.raises(ValueError):
        build_part("ffn", PartSpec("dense_swiglu", dict(hidden_size=8, inner_size=8, pair_limit=0.0)))
    with pytest.raises(ValueError):
        build_part("ffn", PartSpec("moe_swiglu", dict(hidden_size=8, num_experts=4, top_k=2, expert_size=8, weight_scale=2.0)))


def test_the_plain_state_space_is_the_sum_it_stands_for():
    """The recurrence against the sum it stands for: with F_t the sum of -exp(A_log) dt up to t, token s weighs
    e^(F_t - F_s) dt_s (C_t . B_s) at t; and a run that goes on from a state is the rest of the whole run."""
    rng = np.random.default_rng(0)
    T, H, V, N, G = 17, 4, 3, 5, 2
    x, B, C = rng.normal(size=(T, H, V)), rng.normal(size=(T, G, N)), rng.normal(size=(T, G, N))
    dt, a_log, D = plain.softplus(rng.normal(size=(T, H))), rng.normal(size=H), rng.normal(size=H)
    y, S = plain.ssd_scan(x, B, C, dt, a_log, D)
    for h in range(H):
        F = np.cumsum(-np.exp(a_log[h]) * dt[:, h])
        for t in range(T):
            wt = np.exp(F[t] - F[:t + 1]) * dt[:t + 1, h] * (B[:t + 1, h // 2] @ C[t, h // 2])
            assert np.allclose(y[t, h], wt @ x[:t + 1, h] + D[h] * x[t, h])
    y1, S1 = plain.ssd_scan(x[:6], B[:6], C[:6], dt[:6], a_log, D)
    y2, S2 = plain.ssd_scan(x[6:], B[6:], C[6:], dt[6:], a_log, D, S1)
    assert np.allclose(np.concatenate([y1, y2]), y) and np.allclose(S2, S)
    c = rng.normal(size=(9, 2))
    w = np.array([[1.0, 2.0, 3.0], [0.0, 0.0, 1.0]])
    out = plain.short_convolution(c, w, np.array([0.5, -1.0]))
    assert np.allclose(out[0], [3 * c[0, 0] + 0.5, c[0, 1] - 1.0])
    assert np.allclose(out[5, 0], c[3, 0] + 2 * c[4, 0] + 3 * c[5, 0] + 0.5)
    assert np.allclose(plain.short_convolution(c[4:], w, np.array([0.5, -1.0]), c[2:4]), out[4:])


def test_sinks_rotations_temperatures_and_choices_of_the_plain_implementation():
    p = plain.causal_softmax(np.zeros((3, 3)), True)
    assert np.allclose(p, [[1 / 2, 0, 0], [1 / 3, 1 / 3, 0], [1 / 4, 1 / 4, 1 / 4]])
    assert np.allclose(plain.causal_softmax(np.full((2, 2), -800.0), True), 0.0)
    assert np.allclose(plain.causal_softmax(np.full((2, 2), 800.0), True), [[1, 0], [0.5, 0.5]])
    assert np.allclose(plain.causal_softmax(np.zeros((2, 2)), False), [[1, 0], [0.5, 0.5]])
    x = np.zeros((3, 1, 6))
    x[:, 0, 0], x[:, 0, 5] = 1.0, 7.0
    r = plain.rotate(x, {"dims": 4, "base": 100.0})           # numbers 0 and 2 are a pair, 4 and 5 pass
    assert np.allclose(r[2, 0], [math.cos(2), 0, math.sin(2), 0, 0, 7.0])
    x[:, 0, 0], x[:, 0, 1] = 0.0, 1.0
    assert np.allclose(plain.rotate(x, {"dims": 4, "base": 100.0})[2, 0], [0, math.cos(0.2), 0, math.sin(0.2), 0, 7.0])
    t = plain.temperature(9, {"coef": 0.5, "every": 4})
    assert np.allclose(t[:3], 1.0) and np.allclose(t[3:7], 1 + 0.5 * math.log(2)) and np.allclose(t[7:], 1 + 0.5 * math.log(3))
    w = {"gate": np.array([[5.0], [-5.0], [0.5]]), "up": np.array([[9.0], [-9.0], [0.25]]), "down": np.eye(3)}
    y = plain.pair(np.array([[1.0]]), {"e." + k: v for k, v in w.items()}, "e.", 2.0)[0]
    sw = lambda g: g / (1 + math.exp(-1.702 * g))
    assert np.allclose(y, [sw(2.0) * 3.0, sw(-5.0) * -1.0, sw(0.5) * 1.25])
    ids, weights = plain.choose(np.log(np.array([[1.0, 4.0, 2.0, 3.0]])), {"top": 2, "scale": 3.0})
    assert ids.tolist() == [[1, 3]] and np.allclose(weights, [[3 * 4 / 7, 3 * 3 / 7]])
    z = plain.layer_norm(np.array([[1.0, 3.0]]), np.array([2.0, 4.0]), np.array([10.0, 20.0]), 0.0)
    assert np.allclose(z, [[8.0, 24.0]])


def test_what_a_layer_reads_shows_in_the_logits():
    """Each of the design's inputs and constants changes the plain logits by far more than the bound the library is held to."""
    cfg = CASES["regular"]
    w = tensors(cfg, 2)
    toks = list(range(40, 160))
    base = plain.forward(cfg, w, toks)
    scale = np.sqrt(np.mean(base ** 2))

    def changed(change, weights=None):
        c = copy.deepcopy(cfg)
        change(c)
        return np.abs(plain.forward(c, {**w, **(weights or {})}, toks) - base)[110:].max() / scale
    assert changed(lambda c: c["layers"][0]["mixer"].pop("rot")) > 0.01
    assert changed(lambda c: c["layers"][1]["mixer"].pop("q_temp")) > 0.005
    assert changed(lambda c: c["layers"][1]["mixer"].update(diff=0.55)) > 0.005
    assert changed(lambda c: c["layers"][0]["mlp"].update(limit=1.8)) > 0.005
    assert changed(lambda c: c["layers"][1]["mlp"]["shared"].update(limit=1.2)) > 0.005
    assert changed(lambda c: c["layers"][1]["mlp"]["router"].update(scale=1.0)) > 0.005
    for name in ("side.embed", "l0.norm1.b", "l1.mix.lq2", "l1.mix.g", "l2.mix.conv.b", "l2.mix.D", "l1.mlp.shared.sg", "l3.side.gate"):
        assert changed(lambda c: None, {name: np.zeros_like(w[name])}) > 0.005, name
