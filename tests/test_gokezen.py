"""The Gokezen design without a GPU: its config.json reader, its plan over the library's parts, what its layer runs ask of the
cache, and the plain implementation's own mechanisms against closed forms."""
import copy
import math

import numpy as np
import pytest

import plain_gokezen as plain
from gokezen_cases import CASES, config, dense, mixer, moe, random_case, tensors
from turboquant_cpp_amd.config.base import ConfigError
from turboquant_cpp_amd.config.registry import config_from_dict
from turboquant_cpp_amd.engine.model import model_from_config


@pytest.mark.parametrize("case", sorted(CASES))
def test_config_round_trip_and_tensor_table(case):
    cfg = CASES[case]
    arch, typed = config_from_dict(cfg)
    assert arch.name == "Gokezen" and arch.config_to_json(typed) == cfg
    table = model_from_config(cfg, "float32").tensor_table()
    w = tensors(cfg, 0)
    assert set(table) == set(w)
    for name, (shape, _role) in table.items():
        assert tuple(shape) == w[name].shape, name


def test_random_cases_are_read():
    for seed in range(40):
        cfg = random_case(seed)
        arch, typed = config_from_dict(cfg)
        assert arch.config_to_json(typed) == cfg
        assert set(model_from_config(cfg, "bfloat16").tensor_table()) == set(tensors(cfg, seed))


def test_what_the_reader_refuses():
    good = CASES["odd"]

    def broken(change):
        cfg = copy.deepcopy(good)
        change(cfg)
        with pytest.raises(ConfigError):
            config_from_dict(cfg)
    broken(lambda c: c["layers"][0].update(type="serial"))
    broken(lambda c: c["layers"][0]["mixer"].pop("right"))
    broken(lambda c: c["layers"][0]["mixer"].pop("left_scale"))
    broken(lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4))
    broken(lambda c: c["layers"][0]["mixer"]["left"].update(mask={"size": 0}))
    broken(lambda c: c["layers"][0]["mixer"]["right"].update(gate_cap=0.0))
    broken(lambda c: c["layers"][0]["mixer"]["right"].pop("gate_cap"))
    broken(lambda c: c["layers"][2]["mlp"]["router"].update(top=5))          # four groups of one expert are kept
    broken(lambda c: c["layers"][2]["mlp"]["router"].update(groups={"count": 3, "keep": 1}))
    broken(lambda c: c["layers"][2]["mlp"]["shared"].pop("limit"))
    broken(lambda c: c["layers"][2]["mlp"]["expert"].update(limit=-1.0))
    broken(lambda c: c["layers"][1]["mlp"].update(kind="glu"))
    broken(lambda c: c["loop"].update(stop=6))
    broken(lambda c: c["loop"].update(start=4))
    broken(lambda c: c["loop"].update(times=0))
    broken(lambda c: c.pop("max_positions"))
    broken(lambda c: c["norm"].pop("eps"))


def test_the_schedule_of_a_loop_and_what_its_runs_keep():
    model = model_from_config(CASES["odd"], "float32")          # layers 1, 2, 3 twice
    assert [(e.layer, e.step_vector) for e in model.schedule] == \
        [(0, None), (1, 0), (2, None), (3, None), (1, 1), (2, None), (3, None), (4, None)] == plain.runs(CASES["odd"])
    needs = model.cache_needs()
    for (kv, state, of), e in zip(needs, model.schedule):
        m = CASES["odd"]["layers"][e.layer]["mixer"]
        H, D, V = (m["right"][k] for k in ("heads", "dim", "vdim"))
        assert of is None and kv.window == m["left"].get("mask", {}).get("size") and kv.num_kv_heads == m["left"]["kv_heads"]
        assert state.shape == (-(-(H * D * V + H * D + H) // 4) * 4,)
    # two passes over one layer: two places in the cache, two rows of state
    cache = model_from_config(CASES["odd"], "float32").cache_needs()
    assert len(cache) == 8
    for case in CASES:
        model = model_from_config(CASES[case], "float32")
        assert [(e.layer, e.step_vector) for e in model.schedule] == plain.runs(CASES[case])
    # a model without a loop has no step vectors, and a loop of one pass has one
    assert model_from_config(CASES["dense_only"], "float32").plan.step_vectors is None
    assert model_from_config(CASES["ragged"], "float32").tensor_table()["loop.step"][0] == (1, 50)


def test_two_mixers_that_both_keep_the_same_kind_are_refused():
    from turboquant_cpp_amd.config.plan import PartSpec
    from turboquant_cpp_amd.parts.base import build_part
    memory = PartSpec("matrix_memory", dict(hidden_size=8, num_heads=1, head_dim=4, value_dim=4, gate_cap=1.0, eps=1e-5))
    attn = PartSpec("gqa_attention", dict(hidden_size=8, num_heads=1, num_kv_heads=1, head_dim=16, position=PartSpec("none")))
    for a, b in ((memory, memory), (attn, attn)):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("parallel", dict(left=a, right=b)))
    both = build_part("mixer", PartSpec("parallel", dict(left=memory, right=attn)))      # either side may be either kind
    assert both.cache_need() is not None and both.state_need() is not None
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("matrix_memory", dict(hidden_size=8, num_heads=1, head_dim=4, value_dim=4, gate_cap=0.0, eps=1e-5)))


def test_the_plain_memory_is_the_sum_it_stands_for():
    """The recurrence with its running maximum against the sums it stands for: with F_t the sum of f up to t, the weight of
    token s at t is e^(F_t - F_s + i_s), that of the empty start e^(F_t), and the running maximum cancels except against 1."""
    cfg = CASES["memory_only"]
    w = tensors(cfg, 1)
    m, p = cfg["layers"][0]["mixer"]["right"], "l0.mix.right."
    rng = np.random.default_rng(0)
    h = rng.normal(size=(19, cfg["width"]))
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(-1, H, D) / math.sqrt(D)
    k = (h @ w[p + "k"].T).reshape(-1, H, D)
    v = (h @ w[p + "v"].T).reshape(-1, H, V)
    i, f = plain.memory_gates(h, m, w, p)
    assert np.all(f < 0) and np.all(np.abs(i) < m["gate_cap"])
    o = np.zeros((19, H, V))
    for head in range(H):
        F = np.cumsum(f[:, head])
        for t in range(19):
            wt = np.exp(F[t] - F[:t + 1] + i[:t + 1, head]) * (k[:t + 1, head] @ q[t, head])
            # the maximum of what the weights and the start's e^F_t could have been, whichever token it came from
            top = np.exp(max(F[t], (F[t] - F[:t + 1] + i[:t + 1, head]).max()))
            o[t, head] = (wt @ v[:t + 1, head] / top) / (max(abs(wt.sum() / top), 1.0 / top) + 1e-6)
    want = plain.rms_norm(o, None, 1e-5).reshape(19, -1) * w[p + "norm"] * plain.sigmoid(h @ w[p + "g"].T) @ w[p + "o"].T
    whole = plain.matrix_memory(h, m, w, p, 1e-5)
    assert np.abs(whole - want).max() < 1e-9
    first, state = plain.matrix_memory(h[:7], m, w, p, 1e-5, return_state=True)
    rest = plain.matrix_memory(h[7:], m, w, p, 1e-5, state=state)
    assert np.abs(np.concatenate([first, rest]) - whole).max() < 1e-12


def test_windows_limits_and_choices_of_the_plain_implementation():
    p = plain.masked_softmax(np.zeros((6, 6)), 3)
    assert np.allclose(p[5], [0, 0, 0, 1 / 3, 1 / 3, 1 / 3]) and np.allclose(p[1], [0.5, 0.5, 0, 0, 0, 0]) and p[0, 0] == 1.0
    w = {"gate": np.array([[5.0], [-5.0], [0.5]]), "up": np.array([[9.0], [-9.0], [0.25]]), "down": np.eye(3)}
    y = plain.expert(np.array([[1.0]]), {"e." + k: v for k, v in w.items()}, "e.", 2.0)[0]
    sw = lambda g: g / (1 + math.exp(-1.702 * g))
    assert np.allclose(y, [sw(2.0) * 3.0, sw(-5.0) * -1.0, sw(0.5) * 1.25])
    # the best single score lies in a group that loses by its two best
    s = np.array([[0.9, 0.1, 0.2, 0.6, 0.55, 0.0]])
    ids, weights = plain.choose(s, {"top": 2, "scale": 3.0, "groups": {"count": 2, "keep": 1}})
    assert ids.tolist() == [[3, 4]] and np.allclose(weights, [[3 * 0.6 / 1.15, 3 * 0.55 / 1.15]])
    assert plain.choose(s, {"top": 2, "scale": 1.0, "groups": {"count": 2, "keep": 2}})[0].tolist() == [[0, 3]]
    assert plain.choose(s, {"top": 2, "scale": 1.0})[0].tolist() == [[0, 3]]
    assert plain.choose(s, {"top": 2, "scale": 1.0, "groups": {"count": 6, "keep": 3}})[0].tolist() == [[0, 3]]


def test_passes_of_a_loop_differ_by_their_vectors():
    """Taking the step vectors away changes the logits, and each pass has a history of its own: a layer run twice in a row is
    not the layer run once over a history twice as long."""
    cfg = CASES["loop_only"]
    w = tensors(cfg, 2)
    toks = list(range(12))
    a = plain.forward(cfg, w, toks)
    b = plain.forward(cfg, dict(w, **{"loop.step": np.zeros_like(w["loop.step"])}), toks)
    assert np.abs(a - b).max() > 0.1
    flat = dict(cfg, layers=cfg["layers"] * 3)
    del flat["loop"]
    same = {k.replace("l0.", f"l{i}.", 1): v for k, v in w.items() for i in range(3) if k.startswith("l0.")}
    c = plain.forward(flat, dict(w, **same), toks)
    assert np.abs(b - c).max() < 1e-12
