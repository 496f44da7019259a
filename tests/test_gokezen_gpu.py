"""The Gokezen design in the engine against the plain implementation in ``plain_gokezen.py``: every mechanism alone, whole
prompts, the stream behind every layer run, decoding through the cache and the state, prompts in portions, unequal batches,
slots and pages that are used again, keys far away, at the borders of pages and just inside and outside a window (also in a
second pass over the same layer), the first tokens of a sequence, long decoding, a memory that still holds the first token
hundreds of tokens later, sizes of many kinds, the kernels one by one, greedy generation through the library's entry point,
the command line, and the trace runner as a program."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

import plain_gokezen as plain
from gokezen_cases import CASES, config, dense, mixer, moe, random_case, tensors, tokens, write_folder

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32_BOUND = 1e-4        # of the logits' root mean square, per position, mean taken off


@pytest.fixture(scope="module")
def made(tmp_path_factory):
    """(case, seed, peaky) -> (folder, config, weights), each written once."""
    cache = {}

    def get(case: str, seed: int = 0, peaky: float = 1.0):
        key = (case, seed, peaky)
        if key not in cache:
            cfg = CASES[case]
            w = tensors(cfg, seed, peaky)
            cache[key] = (write_folder(str(tmp_path_factory.mktemp(f"gokezen_{case}")), cfg, w), cfg, w)
        return cache[key]
    return get


def engine_of(folder: str, dtype: str = "float32", max_tokens: int = 4096, **kw):
    from turboquant_cpp_amd.engine.model import load_model
    from turboquant_cpp_amd.engine.step import Engine
    return Engine(load_model(folder, act=dtype), max_tokens=max_tokens, page_size=64, **kw)


def errors(got, want: np.ndarray) -> np.ndarray:
    """Per position: root mean square of the difference with its mean taken off, over that of the wanted logits."""
    got = got.detach().double().cpu().numpy() if isinstance(got, torch.Tensor) else np.asarray(got, dtype=np.float64)
    d = got - want
    d = d - d.mean(axis=1, keepdims=True)
    scale = np.sqrt(np.mean((want - want.mean(axis=1, keepdims=True)) ** 2))
    return np.sqrt(np.mean(d * d, axis=1)) / scale


def check(got, want, dtype="float32", what="", clear=None):
    """``clear``: the positions whose experts were chosen by a margin that rounding to bfloat16 cannot turn (all of them for
    None): at the others a choice, and with it the row, may differ by more than rounding, so they count for the quantiles only."""
    e = errors(got, want)
    worst = e.max() if clear is None else e[clear].max()
    if dtype == "float32":
        assert e.max() < F32_BOUND, f"{what}: position {int(e.argmax())} differs by {e.max():.2e}"
    elif dtype == "bfloat16":       # rounding of bfloat16 products and activations through all layers of a narrow model
        assert worst < 0.2 and np.quantile(e, 0.9) < 0.06 and np.median(e) < 0.03, \
            f"{what}: median {np.median(e):.3f}, 90 % {np.quantile(e, 0.9):.3f}, worst {worst:.3f}"
    else:       # "same path": the engine against itself on another schedule, in bfloat16
        assert np.quantile(e, 0.9) < 0.02 and worst < 0.3, \
            f"{what}: 90 % {np.quantile(e, 0.9):.3f}, worst {worst:.2e}"


def clear_choices(cfg, w, toks, margin: float = 0.02):
    """Positions at which no layer's choice of experts or groups hung on less than ``margin`` (scores lie within 0 and 1)."""
    return plain.forward(cfg, w, toks, return_margins=True)[1] > margin


def all_places(n):
    return list(range(n))


def wanted(eng, cfg, w, toks, dtype):
    """In float32 the plain implementation; in bfloat16 the engine's own logits for the whole sequence in one step, alone
    (which test_whole_prompt_bfloat16 holds against the plain implementation)."""
    if dtype == "float32":
        return plain.forward(cfg, w, toks), dtype
    slot = eng.open(1)
    out = eng.step(slot, [toks], [all_places(len(toks))]).double().cpu().numpy()
    eng.close(slot)
    return out, "same path"


def prompt_then_decode(eng, toks, cut):
    slot = eng.open(1)
    rows = [eng.step(slot, [toks[:cut]], [all_places(cut)])] + [eng.step(slot, [[t]]) for t in toks[cut:]]
    eng.close(slot)
    return torch.cat(rows)


# ---------------------------------------------------------------- whole prompts, every configuration
@pytest.mark.parametrize("case", sorted(CASES))
def test_whole_prompt(made, case):
    d, cfg, w = made(case)
    eng = engine_of(d)
    for seed, n in ((1, 1), (2, 150), (3, 67), (4, 2)):
        toks = tokens(cfg, n, seed)
        slot = eng.open(1)
        got = eng.step(slot, [toks], [all_places(n)])
        eng.close(slot)
        check(got, plain.forward(cfg, w, toks), what=f"{case}, {n} tokens")


@pytest.mark.parametrize("case", ["regular", "odd", "ragged", "wide"])
def test_whole_prompt_bfloat16(made, case):
    d, cfg, w = made(case)
    eng = engine_of(d, "bfloat16")
    toks = tokens(cfg, 200, 4)
    slot = eng.open(1)
    got = eng.step(slot, [toks], [all_places(len(toks))])
    check(got, plain.forward(cfg, w, toks), "bfloat16", case, clear_choices(cfg, w, toks))


@pytest.mark.parametrize("seed", range(12))
def test_sizes_of_many_kinds(tmp_path, seed):
    """Configurations drawn at random: a prompt in two portions and a few decoded tokens, two requests side by side, in
    true 32-bit against the plain implementation at every position, and in bfloat16."""
    cfg = random_case(seed)
    w = tensors(cfg, seed)
    d = write_folder(str(tmp_path), cfg, w)
    a, b = tokens(cfg, 140, seed), tokens(cfg, 31, 100 + seed)
    wa, wb = plain.forward(cfg, w, a), plain.forward(cfg, w, b)
    for dtype in ("float32", "bfloat16"):
        eng = engine_of(d, dtype)
        sa, sb = eng.open(2)
        out = eng.step([sa, sb], [a[:70], b[:3]], [all_places(70), all_places(3)])
        rows_a, rows_b = [out[:70]], [out[70:]]
        out = eng.step([sa, sb], [a[70:130], b[3:]], [all_places(60), all_places(len(b) - 3)])
        rows_a.append(out[:60])
        rows_b.append(out[60:])
        eng.close([sb])
        rows_a += [eng.step([sa], [[t]]) for t in a[130:]]
        ga, gb = torch.cat(rows_a), torch.cat(rows_b)
        assert bool(torch.isfinite(ga).all()) and bool(torch.isfinite(gb).all())
        if dtype == "float32":
            check(ga, wa, what=f"seed {seed}: {json.dumps(cfg['layers'])}")
            check(gb, wb, what=f"seed {seed}, second request")
        else:
            assert np.median(errors(ga, wa)) < 0.05, f"seed {seed}: median {np.median(errors(ga, wa)):.3f}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_prompt_of_a_thousand_tokens(made, dtype):
    """Long enough for the plain products of the bfloat16 path to go to the vendor's library, over many pages and several
    windows, then decoded on."""
    d, cfg, w = made("regular", seed=7)
    eng = engine_of(d, dtype)
    toks = tokens(cfg, 1010, 13)
    check(prompt_then_decode(eng, toks, 1000), plain.forward(cfg, w, toks), dtype, "1,000 tokens", clear_choices(cfg, w, toks))


@pytest.mark.parametrize("case", ["odd", "ragged"])
def test_layers_one_by_one(made, case):
    """The residual stream behind every layer run, before the vector that comes ahead of the next pass."""
    d, cfg, w = made(case)
    eng = engine_of(d)
    seen = []
    eng.layer_hook = lambda entry, hidden, batch: seen.append(hidden.double().cpu().numpy())
    toks = tokens(cfg, 120, 5)
    eng.step(eng.open(1), [toks], [[]])
    _, streams = plain.forward(cfg, w, toks, return_layers=True)
    assert len(seen) == len(plain.runs(cfg)) == len(streams)
    for i, (a, b) in enumerate(zip(seen, streams)):
        assert np.abs(a - b).max() < 2e-4 * max(1.0, np.abs(b).max()), f"layer run {i}"


# ---------------------------------------------------------------- decoding, portions, batches
@pytest.mark.parametrize("case,dtype", [("odd", "float32"), ("ragged", "float32"), ("regular", "float32"),
                                        ("regular", "bfloat16"), ("odd", "bfloat16"), ("ragged", "bfloat16"),
                                        ("wide", "float32"), ("wide", "bfloat16"), ("attention_only", "float32"),
                                        ("memory_only", "float32"), ("experts_only", "float32"), ("dense_only", "float32"),
                                        ("loop_only", "float32")])
def test_prompt_then_token_by_token(made, case, dtype):
    """Most of a sequence in one step, the rest one token a step (the later steps replayed as graphs), across the edges of
    pages and of windows."""
    d, cfg, w = made(case)
    eng = engine_of(d, dtype)
    toks = tokens(cfg, 150, 6)
    want, how = wanted(eng, cfg, w, toks, dtype)
    check(prompt_then_decode(eng, toks, 58), want, how, case, clear_choices(cfg, w, toks))


def test_token_by_token_from_the_first(made):
    """No prompt step at all: the first tokens of a sequence through the decode kernels, an empty state, a softmax over
    one key, windows that are not yet full."""
    for case in ("odd", "ragged", "regular"):
        d, cfg, w = made(case)
        eng = engine_of(d)
        toks = tokens(cfg, 110, 16)
        check(prompt_then_decode(eng, toks, 1), plain.forward(cfg, w, toks), what=case)


@pytest.mark.parametrize("case", ["odd", "ragged", "regular"])
def test_portions(made, case):
    """The logits do not depend on how a prompt was cut: portions of two tokens and more, of one, of a page and over."""
    d, cfg, w = made(case)
    eng = engine_of(d)
    toks = tokens(cfg, 190, 7)
    want = plain.forward(cfg, w, toks)
    for cuts in ([2, 3, 1, 5, 2, 64, 7, 2, 33, 71], [17, 2, 2, 100, 69], [95, 95], [64, 64, 62], [2] * 95):
        assert sum(cuts) == len(toks)
        slot, rows, at = eng.open(1), [], 0
        for c in cuts:
            rows.append(eng.step(slot, [toks[at:at + c]], [all_places(c)]))
            at += c
        eng.close(slot)
        check(torch.cat(rows), want, what=f"{case}, cuts {cuts[:12]}")


def test_portions_bfloat16(made):
    d, cfg, w = made("regular")
    eng = engine_of(d, "bfloat16")
    toks = tokens(cfg, 190, 7)
    want, how = wanted(eng, cfg, w, toks, "bfloat16")
    slot, rows, at = eng.open(1), [], 0
    for c in [2, 3, 1, 5, 2, 64, 7, 2, 33, 71]:
        rows.append(eng.step(slot, [toks[at:at + c]], [all_places(c)]))
        at += c
    check(torch.cat(rows), want, how, "portions", clear_choices(cfg, w, toks))


@pytest.mark.parametrize("case,dtype", [("odd", "float32"), ("regular", "float32"), ("regular", "bfloat16"),
                                        ("ragged", "float32"), ("wide", "bfloat16"), ("odd", "bfloat16")])
def test_unequal_batch(made, case, dtype):
    """Requests of unequal lengths in one step and decoded together, the shorter ones ending earlier, against each alone."""
    d, cfg, w = made(case)
    eng = engine_of(d, dtype)
    lengths, prompts = [1, 37, 131, 64, 90], [1, 20, 100, 64, 61]
    seqs = [tokens(cfg, n, 10 + i) for i, n in enumerate(lengths)]
    alone = [wanted(eng, cfg, w, s, dtype) for s in seqs]
    slots = eng.open(len(seqs))
    got = [[] for _ in seqs]
    out = eng.step(slots, [s[:p] for s, p in zip(seqs, prompts)], [all_places(p) for p in prompts])
    at = 0
    for i, p in enumerate(prompts):
        got[i].append(out[at:at + p])
        at += p
    done = list(prompts)
    while True:
        live = [i for i, s in enumerate(seqs) if done[i] < len(s)]
        if not live:
            break
        out = eng.step([slots[i] for i in live], [[seqs[i][done[i]]] for i in live])
        for r, i in enumerate(live):
            got[i].append(out[r:r + 1])
            done[i] += 1
            if done[i] == len(seqs[i]):
                eng.close([slots[i]])
    eng.close([slots[0]])
    for i, s in enumerate(seqs):
        check(torch.cat(got[i]), alone[i][0], alone[i][1], f"{case}, request {i}", clear_choices(cfg, w, s) if len(s) > 1 else None)


def test_slots_and_pages_used_again(made):
    """A cache with room for little: sequences come and go, each finds the pages and the slot of one before it, with that
    one's keys in the pages and its memory (S, n and m of every pass) in the slot's row."""
    d, cfg, w = made("odd")
    eng = engine_of(d, max_tokens=256, max_slots=2)
    for round_ in range(3):
        a, b = tokens(cfg, 120 + round_, 20 + round_), tokens(cfg, 70, 30 + round_)
        sa, sb = eng.open(2)
        out = eng.step([sa, sb], [a[:100], b[:5]], [all_places(100), all_places(5)])
        rows_a, rows_b = [out[:100]], [out[100:]]
        eng.close([sa])
        rows_b.append(eng.step([sb], [b[5:]], [all_places(len(b) - 5)]))
        sc = eng.open(1)[0]
        assert sc == sa
        c = tokens(cfg, 66, 40 + round_)
        rows_c = [eng.step([sc], [c[:60]], [all_places(60)])] + [eng.step([sc], [[t]]) for t in c[60:]]
        eng.close([sb, sc])
        check(torch.cat(rows_a), plain.forward(cfg, w, a)[:100], what="first")
        check(torch.cat(rows_b), plain.forward(cfg, w, b), what="second")
        check(torch.cat(rows_c), plain.forward(cfg, w, c), what="in the first one's slot")
    assert all(v == 0 for v in eng.cache.pages_held().values())


# ---------------------------------------------------------------- one key that decides: far back, at borders, at a window's edge
def plant_token(w):
    """Channel 0 of the embedding is nonzero for token 1 only, channel 1 the same for every token, positions and step vectors
    leave both alone, and the norms pass both as they are."""
    w["embed"][:, 0] = 0.0
    w["embed"][1, 0] = 4.0
    w["embed"][:, 1] = 2.0
    w["pos"][:, :2] = 0.0
    if "loop.step" in w:
        w["loop.step"][:, :2] = 0.0
    for name in w:
        if name.endswith("norm1"):
            w[name][:2] = 1.0


def planted_attention(seed: int, window, kv_heads: int = 1, times: int = 1):
    """Attention layers whose every query looks along the last channel of a head, where only token 1 has a key that answers
    (its score is some 20 against about 1).  With ``times`` 2 the layer runs twice and adds nothing to the planted channels,
    and the first pass's result is scaled down by its output product, so that what shows is the second pass's own window."""
    D = 16
    cfg = config(32, 40, [(mixer((2, kv_heads, D, 16, window, 1.0), (1, 4, 4), 1.0, 0.0), None)],
                 loop=None if times == 1 else (0, 1, times))
    w = tensors(cfg, seed)
    plant_token(w)
    p = "l0.mix.left."
    w[p + "q"] *= 0.25
    for g in range(kv_heads):
        w[p + "k"][g * D + D - 1, :] = 0.0
        w[p + "k"][g * D + D - 1, 0] = 3.0
    for head in range(2):
        w[p + "q"][head * D + D - 1, :] = 0.0
        w[p + "q"][head * D + D - 1, 1] = 2.0
    w[p + "o"][:2, :] = 0.0
    return cfg, w


@pytest.mark.parametrize("times", [1, 2])
def test_a_key_far_back_and_at_the_borders_of_pages(tmp_path, times):
    """The one token that every later query looks for stands at the first position, at a page's last and first places, or
    300 tokens back; the rows behind it are read in a prompt and in decoding.  The plain implementation's own outputs with
    and without it differ by much, so a key that is lost or taken from a wrong place shows."""
    cfg, w = planted_attention(1, None, times=times)
    eng = engine_of(write_folder(str(tmp_path), cfg, w))
    n = 340
    base = [2 + (i * 7) % 38 for i in range(n)]
    without = plain.forward(cfg, w, base)
    for place in (0, 63, 64, 65, 127, 128, 255, 300):
        toks = list(base)
        toks[place] = 1
        want = plain.forward(cfg, w, toks)
        assert errors(want[place + 1:], without[place + 1:]).min() > 0.05, place
        for cut in (310, 62, 129) if times == 1 else (129,):
            check(prompt_then_decode(eng, toks, cut), want, what=f"the token at {place}, prompt of {cut}")


@pytest.mark.parametrize("window,kv_heads,times", [(70, 1, 1), (64, 2, 1), (65, 1, 1), (5, 1, 1), (1, 2, 1), (130, 1, 1), (40, 1, 2)])
def test_a_key_just_inside_and_just_outside_a_window(tmp_path, window, kv_heads, times):
    """A query at position i sees the planted key at p exactly if i - p < window: the plain rows with and without it differ
    by much up to p + window - 1 and not at all from the place on where neither the token nor (in a second pass) a row that
    saw it is in sight, in a prompt, in portions and in decoding, with the key at the borders of pages."""
    cfg, w = planted_attention(4, window, kv_heads=kv_heads, times=times)
    eng = engine_of(write_folder(str(tmp_path), cfg, w))
    n = 100 + times * window + 14
    base = [2 + (i * 7) % 38 for i in range(n)]
    without = plain.forward(cfg, w, base)
    for place in (0, 3, 63, 64, 100):
        toks = list(base)
        toks[place] = 1
        want = plain.forward(cfg, w, toks)
        edge, gone = place + window, place + times * (window - 1) + 1
        if window > 1:
            assert errors(want[place + 1:edge], without[place + 1:edge]).min() > 0.05, place
        assert errors(want[gone:], without[gone:]).max() < 1e-12, place
        for cut in (n - 2, edge - 1, edge, max(1, edge - 40), place + 1):       # the edge in the prompt, first decoded, decoded
            cut = max(1, min(cut, n - 1))
            check(prompt_then_decode(eng, toks, cut), want, what=f"window {window}: the token at {place}, prompt of {cut}")
        slot, rows, at = eng.open(1), [], 0                                       # and in portions that end around the edge
        for c in [place + 1, window - 2, 1, 1, 2, 7] if window > 3 else [place + 1, 2, 2, 7]:
            rows.append(eng.step(slot, [toks[at:at + c]], [all_places(c)]))
            at += c
        eng.close(slot)
        check(torch.cat(rows), want[:at], what=f"window {window}: the token at {place}, portions")


def planted_memory(seed: int, keeps: bool):
    """A memory whose every query looks along a head's first channel, where only token 1 writes, and that with an open input
    gate; ``keeps``: the forget gates stay within 1e-4 of 1, else they halve the state in a few tokens."""
    D = 8
    cfg = config(32, 40, [(mixer((1, 1, 8, 8, 4), (2, D, 16, 12.0), 0.0, 1.0), None)])
    w = tensors(cfg, seed)
    plant_token(w)
    p = "l0.mix.right."
    for n in ("i", "f"):
        w[p + n][:] *= 1.0 / 16.0      # (still bfloat16 numbers)
        w[p + n][:, :2] = 0.0
    w[p + "i"][:, 0] = 2.0
    w[p + "i.b"][:] = -2.0
    w[p + "f.b"][:] = 14.0 if keeps else 0.5
    for head in range(2):
        w[p + "k"][head * D, :] = 0.0
        w[p + "k"][head * D, 0] = 4.0
        w[p + "q"][head * D, :] = 0.0
        w[p + "q"][head * D, 1] = 8.0
    return cfg, w


def test_far_tokens_in_a_memory_that_forgets_nothing(tmp_path):
    """What the first token wrote into the memory is still read hundreds of tokens later, in a prompt and in decoding; with
    forget gates that close it is gone by then, and a token just before a row still shows."""
    for keeps in (True, False):
        cfg, w = planted_memory(3, keeps)
        eng = engine_of(write_folder(str(tmp_path / str(keeps)), cfg, w))
        base = [2 + (j * 7) % 38 for j in range(330)]
        without = plain.forward(cfg, w, base)
        for place in (0, 63, 290):
            toks = list(base)
            toks[place] = 1
            want = plain.forward(cfg, w, toks)
            gap = errors(want[300:304], without[300:304]) if not keeps and place == 290 else errors(want[300:], without[300:])
            assert gap.min() > 0.02 if keeps or place == 290 else gap.max() < 1e-3, (keeps, place, gap.min(), gap.max())
            check(prompt_then_decode(eng, toks, 295), want, what=f"keeps {keeps}, the token at {place}")
            check(prompt_then_decode(eng, toks, max(place, 1) + 4), want, what=f"keeps {keeps}, the token at {place}, decoded")


def test_queries_that_single_keys_decide(made):
    d, cfg, w = made("odd", seed=3, peaky=6.0)
    eng = engine_of(d)
    toks = tokens(cfg, 330, 9)
    want = plain.forward(cfg, w, toks)
    check(prompt_then_decode(eng, toks, 290), want, what="peaky")
    check(prompt_then_decode(eng, toks, 5), want, what="peaky, decoded")


def test_long_decoding(made):
    d, cfg, w = made("regular", seed=2)
    eng = engine_of(d)
    toks = tokens(cfg, 420, 11)
    check(prompt_then_decode(eng, toks, 3), plain.forward(cfg, w, toks), what="417 decoded tokens")


def test_a_sequence_up_to_the_last_learned_position(tmp_path):
    """A table of 70 positions: a sequence runs to the last of them, and the cache refuses one more."""
    from turboquant_cpp_amd.cache.paged import CacheError
    cfg = dict(CASES["loop_only"], max_positions=70)
    w = tensors(cfg, 8)
    eng = engine_of(write_folder(str(tmp_path), cfg, w))
    toks = tokens(cfg, 70, 3)
    slot = eng.open(1)
    rows = [eng.step(slot, [toks[:60]], [all_places(60)])] + [eng.step(slot, [[t]]) for t in toks[60:]]
    check(torch.cat(rows), plain.forward(cfg, w, toks), what="70 positions")
    with pytest.raises(CacheError):
        eng.step(slot, [[1]])


def test_values_that_a_model_may_happen_to_make_equal_or_one(tmp_path):
    """Scale 1, factors of 1 and of 0, one head, as many kv heads as heads, value widths other than key widths, one number to
    a memory's key, gate caps that bite and that never do, a loop of everything and of the last layer, one pass, one expert,
    every expert chosen, every group kept, limits that never bite and that always do, a shared expert of another limit."""
    for i, cfg in enumerate([
        config(48, 60, [(mixer((1, 1, 12, 20, None, 1.0), (1, 1, 12, 0.5)), dense(16)),
                        (mixer((1, 1, 4, 4, 200, 0.05), (4, 12, 1, 100.0), 0.0, 1.0), moe(1, 1, 8, limit=100.0, shared=(8, 0.01)))],
               loop=(0, 2, 2)),
        config(48, 60, [(mixer((3, 3, 16, 4, 2), (3, 16, 4)), moe(3, 3, 12, groups=(3, 3), limit=0.01, scale=4.0)),
                        (mixer((3, 1, 16, 33, 1), (2, 5, 9), 2.0, 0.0), moe(6, 1, 12, groups=(2, 1), shared=(7, 50.0))),
                        (mixer((8, 2, 16, 16, 64), (8, 16, 16), -1.0, 0.3), dense(7))], loop=(2, 3, 4), eps=1e-3),
        config(48, 60, [(mixer((2, 1, 16, 16, 10), (2, 16, 16)), moe(4, 2, 16, groups=(1, 1), shared=(16, 2.0)))], loop=(0, 1, 1)),
    ]):
        w = tensors(cfg, 20 + i)
        eng = engine_of(write_folder(str(tmp_path / str(i)), cfg, w))
        toks = tokens(cfg, 90, 20 + i)
        check(prompt_then_decode(eng, toks, 70), plain.forward(cfg, w, toks), what=f"configuration {i}")


# ---------------------------------------------------------------- the mechanisms' kernels, one by one
def f32(a):
    return torch.tensor(np.ascontiguousarray(a), dtype=torch.float32, device="cuda")


def memory_inputs(H, D, V, n, rng, gates: str):
    """q, k, v, g, raw gates and their biases of a run of n tokens.  ``gates``: "mixed"; "closing" (forget gates near 0: F falls by
    many units a token); "open" (forget gates near 1, input gates at both ends of the cap)."""
    P = rng.normal(size=(n, 2 * H * (D + V + 1)))
    at = 2 * H * (D + V)
    bi, bf = rng.normal(size=H), rng.normal(size=H) + 2.0
    if gates == "closing":
        bf -= 14.0
    elif gates == "open":
        P[:, at:at + H] *= 30.0
        bf += 20.0
    return P, np.concatenate([bi, bf])


def plain_memory(P, bias, H, D, V, cap, state=None):
    q, k, v, g, i, f = np.split(P, np.cumsum([H * D, H * D, H * V, H * V, H]), axis=1)
    n = len(P)
    gi = cap * np.tanh((i + bias[:H]) / cap)
    gf = plain.log_sigmoid(cap * np.tanh((f + bias[H:]) / cap))
    return plain.memory_scan(q.reshape(n, H, D) * D ** -0.5, k.reshape(n, H, D), v.reshape(n, H, V), gi, gf, state), plain.sigmoid(g)


SIZES = [(4, 16, 24), (3, 20, 12), (1, 40, 4), (3, 3, 5), (2, 128, 128), (1, 256, 40), (1, 300, 20), (1, 700, 8), (5, 2, 130)]


@pytest.mark.parametrize("gates", ["mixed", "closing", "open"])
@pytest.mark.parametrize("form", ["scan", "chunked", "decode"])
def test_the_memory_s_kernels_with_a_state_carried_over(form, gates):
    """The recurrence, its denominators and the gated, normed read-out against the plain function: several sequences side by
    side in slots in no order, the second step going on from the states that the first one left, runs of one token, of a
    chunk less one, of a chunk, of a chunk and one, of several; sizes the form does not take are left to another."""
    from turboquant_cpp_amd.csrc import ops
    cap, eps = 9.0, 1e-5
    for H, D, V in SIZES:
        if (form == "chunked" and D > 256) or (form == "decode" and V % 4):
            continue
        d = ops.MemoryDims(H, D, V, cap)
        rng = np.random.default_rng(H * 1000 + D)
        first, slots = ((130, 64, 1, 65, 63), (6, 0, 3, 1, 5)) if form == "chunked" else ((23, 1, 16), (5, 2, 0))
        second = (70,) * 5 if form == "chunked" else (17,) * 3
        if form == "decode":
            first, second = (1,) * 3, (1,) * 3
        made_ = [memory_inputs(H, D, V, a + b, rng, gates) for a, b in zip(first, second)]
        bias = made_[0][1]
        Ps = [p for p, _ in made_]
        wt = rng.normal(1.0, 0.1, H * V)
        state = torch.zeros((8, d.state_floats), dtype=torch.float32, device="cuda")
        outs = [[] for _ in Ps]
        for parts in ([P[:a] for P, a in zip(Ps, first)], [P[a:] for P, a in zip(Ps, first)]):
            x = np.concatenate(parts)
            lens = [len(q) for q in parts]
            cu = np.cumsum([0] + lens)
            runs = {"cu_seqlens": torch.tensor(cu, dtype=torch.int32, device="cuda"), "max_new": max(lens),
                    "slots": torch.tensor(slots, dtype=torch.int32, device="cuda")}
            of_token = torch.tensor(np.repeat(slots, lens), dtype=torch.int32, device="cuda")
            proj = torch.full((len(x), (x.shape[1] + 3) // 4 * 4 + 4), 9.0, dtype=torch.float32, device="cuda")   # wider than need be
            proj[:, :x.shape[1]] = f32(x)
            gate = proj[:, 2 * H * D + H * V:2 * H * D + 2 * H * V]
            if form == "scan":
                num, den, mrow = ops.mm_scan(proj, f32(bias), runs, state, d, "float32")
                y = ops.mm_out(num, den, gate, f32(wt), eps, d, "float32", mrow=mrow, slot_of_token=of_token, state=state)
            elif form == "chunked":
                num, den = ops.mm_chunked(proj, f32(bias), runs, state, d, "float32")
                y = ops.mm_out(num, den, gate, f32(wt), eps, d, "float32")
            else:
                if not ops.mm_decode_fits(proj, d):
                    continue
                y = ops.mm_decode(proj, f32(bias), runs, state, f32(wt), eps, d, "float32")
            for i in range(len(Ps)):
                outs[i].append(y.double().cpu().numpy()[cu[i]:cu[i + 1]])
        if not outs[0]:
            continue
        used = set()
        for i, P in enumerate(Ps):
            (o, (S, n, m)), g = plain_memory(P, bias, H, D, V, cap)
            want = plain.rms_norm(o, None, eps).reshape(len(P), -1) * wt * g
            got = np.concatenate(outs[i])
            # (a read-out over a denominator that nearly cancels is as exact as the cancelling sum: most tokens to 1e-5)
            err = np.abs(got - want).max(axis=1) / max(1.0, np.abs(want).max())
            assert err.max() < 2e-3 and np.quantile(err, 0.9) < 2e-5, (form, gates, (H, D, V), i, err.max(), np.quantile(err, 0.9))
            row = state[slots[i]].double().cpu().numpy()
            used.add(slots[i])
            for name, a, b in (("S", row[:H * D * V], S.ravel()), ("n", row[H * D * V:d.m_offset], n.ravel()), ("m", row[d.m_offset:d.m_offset + H], m)):
                assert np.abs(a - b).max() < 5e-5 * max(1.0, np.abs(b).max()), (form, gates, (H, D, V), i, name)
        assert float(state[[s for s in range(8) if s not in used]].abs().max()) == 0.0


def test_forms_of_the_memory_agree_where_one_hands_over_to_another():
    """A run of 200 tokens in chunks, then 5 by the scan, then 3 decoded, against the plain function over all of them."""
    from turboquant_cpp_amd.csrc import ops
    H, D, V, cap, eps = 3, 32, 48, 15.0, 1e-5
    d = ops.MemoryDims(H, D, V, cap)
    rng = np.random.default_rng(5)
    P, bias = memory_inputs(H, D, V, 208, rng, "mixed")
    wt = rng.normal(1.0, 0.1, H * V)
    state = torch.zeros((3, d.state_floats), dtype=torch.float32, device="cuda")
    slot = torch.tensor([1], dtype=torch.int32, device="cuda")
    outs, at = [], 0
    for n in (200, 5, 1, 1, 1):
        proj = torch.zeros((n, (P.shape[1] + 3) // 4 * 4), dtype=torch.float32, device="cuda")
        proj[:, :P.shape[1]] = f32(P[at:at + n])
        runs = {"cu_seqlens": torch.tensor([0, n], dtype=torch.int32, device="cuda"), "slots": slot, "max_new": n}
        gate = proj[:, 2 * H * D + H * V:2 * H * D + 2 * H * V]
        if n == 200:
            num, den = ops.mm_chunked(proj, f32(bias), runs, state, d, "float32")
            y = ops.mm_out(num, den, gate, f32(wt), eps, d, "float32")
        elif n == 5:
            num, den, mrow = ops.mm_scan(proj, f32(bias), runs, state, d, "float32")
            y = ops.mm_out(num, den, gate, f32(wt), eps, d, "float32", mrow=mrow, slot_of_token=slot.repeat(n), state=state)
        else:
            y = ops.mm_decode(proj, f32(bias), runs, state, f32(wt), eps, d, "float32")
        outs.append(y.double().cpu().numpy())
        at += n
    (o, _), g = plain_memory(P, bias, H, D, V, cap)
    want = plain.rms_norm(o, None, eps).reshape(208, -1) * wt * g
    err = np.abs(np.concatenate(outs) - want).max(axis=1)
    assert err.max() < 2e-3 and np.quantile(err, 0.9) < 2e-5 and err[200:].max() < 1e-4


def test_a_router_of_sigmoid_scores():
    """The choice within the groups with the best two scores, and its weights, against the plain function; many tokens and a
    handful, groups of one, keep of as many groups as experts are chosen (which does not make the choice free here), a bias."""
    from turboquant_cpp_amd.csrc import ops
    rng = np.random.default_rng(2)
    for T, H, E, top, groups, scale in ((1, 48, 6, 2, None, 1.0), (9, 64, 16, 4, (4, 2), 2.5), (70, 72, 8, 2, (4, 2), 0.5),
                                        (300, 50, 12, 3, (12, 5), 1.5), (40, 64, 64, 8, (8, 3), 2.0), (5, 40, 1, 1, (1, 1), 3.0),
                                        (33, 40, 9, 9, (3, 3), 1.0), (16, 64, 200, 6, (100, 7), 1.0)):
        x, wr = rng.normal(size=(T, H)), rng.normal(size=(E, H)) * 1.5 * H ** -0.5
        z = x.astype(np.float32).astype(np.float64) @ wr.astype(np.float32).astype(np.float64).T
        r = {"top": top, "scale": scale}
        if groups is not None:
            r["groups"] = {"count": groups[0], "keep": groups[1]}
        for b in (None, rng.normal(size=E)):
            s = plain.sigmoid(z if b is None else z + b)
            want_ids, want_w = plain.choose(s, r)
            kw = {} if b is None else {"bias": f32(b)}
            ids, weights, _ = ops.router_topk(f32(x), f32(wr), None, top, True, "float32", groups=groups, sigmoid=True,
                                              weight_scale=scale, pair_groups=True, **kw)
            out = ops.route(f32(x), f32(wr), None, top, True, 16, "float32", groups=groups, sigmoid=True, weight_scale=scale,
                            pair_groups=True, **kw)
            assert torch.equal(out[0], ids) and torch.equal(out[1], weights)
            same = np.array([set(a) == set(c) for a, c in zip(ids.cpu().numpy().tolist(), want_ids.tolist())])
            assert same.mean() > 0.99, (T, E, top, groups)      # (a tie to rounding may go either way)
            o1, o2 = np.argsort(ids.cpu().numpy(), axis=1), np.argsort(want_ids, axis=1)
            dw = np.abs(np.take_along_axis(weights.double().cpu().numpy(), o1, 1) - np.take_along_axis(want_w, o2, 1))
            assert dw[same].max() < 1e-5 * max(1.0, scale)


def test_two_gated_pairs_with_limits_of_their_own_in_one_launch():
    from turboquant_cpp_amd.csrc import ops
    rng = np.random.default_rng(4)
    sw = lambda g: g * plain.sigmoid(1.702 * g)
    M, K = 5, 64
    a = rng.normal(size=(M, K))
    for act, dt, tol in (("float32", torch.float32, 1e-4), ("bfloat16", torch.bfloat16, 0.03)):
        aa = f32(a).to(dt)
        probs, wants = [], []
        for N, limit in ((96, 0.6), (40, 2.0)):
            g_, u_ = (f32(rng.normal(size=(N, K)) * 2 * K ** -0.5).to(dt) for _ in range(2))
            probs.append(dict(a=aa, w=g_, w2=u_, out_act=True, activation="swish1702", pair_limit=limit))
            zg, zu = (aa.double().cpu().numpy() @ t.double().cpu().numpy().T for t in (g_, u_))
            wants.append(sw(np.minimum(zg, limit)) * (np.clip(zu, -limit, limit) + 1.0))
        for got, want in zip(ops.gemm_pair(*probs, act), wants):
            assert np.abs(got.double().cpu().numpy() - want).max() < tol * max(1.0, np.abs(want).max()), act


def test_the_sum_of_several_parts_with_a_norm_behind_it():
    """Partial sums of up to four parts with a factor each, the experts' unsummed rows and a vector for every row, added into
    the stream and normed; rows picked (then the stream stays as it is); the sum alone; the same as a tensor."""
    from turboquant_cpp_amd.csrc import ops
    rng = np.random.default_rng(6)
    for T, H, S in ((3, 64, (1, 5)), (70, 50, (2, 1, 3)), (9, 2048, (12, 1, 4, 2)), (4, 96, ()), (17, 2050, (3,))):
        x, w, vec = rng.normal(size=(T, H)), rng.normal(1.0, 0.1, H), rng.normal(size=H)
        parts = [(float(rng.normal()), rng.normal(size=(s, T, H))) for s in S]
        y, slot, wt = rng.normal(size=(3 * T, H)), rng.integers(-1, 3 * T, size=(T, 3)), rng.normal(size=(T, 3))
        for with_vec, with_y in ((True, True), (False, True), (True, False), (False, False)):
            add = sum((c * d.sum(0) for c, d in parts), np.zeros((T, H)))
            if with_vec:
                add = add + vec
            if with_y:
                add = add + np.einsum("tk,tkh->th", np.where(slot < 0, 0.0, wt), y[np.maximum(slot, 0)])
            gathered = ops.GatheredSum(f32(y), torch.tensor(slot, dtype=torch.int32, device="cuda"), f32(wt)) if with_y else None
            terms = ops.Terms([(c, f32(d)) for c, d in parts], gathered, f32(vec) if with_vec else None)
            want = x + add
            xs = f32(x)
            out, out32 = ops.add_rmsnorm(xs, terms, f32(w), 1e-5, "float32", want_f32=True)
            assert np.abs(xs.double().cpu().numpy() - want).max() < 1e-4
            for o in (out, out32):
                assert np.abs(o.double().cpu().numpy() - plain.rms_norm(want, w, 1e-5)).max() < 1e-4
            xs, rows = f32(x), [T - 1, 0, T - 1]
            out, _ = ops.add_rmsnorm(xs, terms, f32(w), 1e-5, "float32", rows=torch.tensor(rows, dtype=torch.int32, device="cuda"))
            assert np.abs(out.double().cpu().numpy() - plain.rms_norm(want[rows], w, 1e-5)).max() < 1e-4
            assert torch.equal(xs, f32(x))
            if parts or with_y or with_vec:
                assert np.abs(terms.materialize("float32")[0].double().cpu().numpy() - add).max() < 1e-4


# ---------------------------------------------------------------- the library's own entry points
def test_greedy_generation_through_the_entry_point(made):
    from turboquant_cpp_amd import Model
    d, cfg, w = made("regular", seed=5)
    prompts = [tokens(cfg, n, 50 + n) for n in (5, 70, 1, 33, 100)]
    with Model(d, dtype="float32", temperature=0.0, rep_penalty=1.0, max_tokens=24, max_batch=3, stop_tokens=()) as m:
        got = m.generate(prompts, loop_detection=False)
    for p, g in zip(prompts, got):
        assert len(g) == 24
        rows = plain.forward(cfg, w, p + g)
        for j, tok in enumerate(g):
            row = rows[len(p) - 1 + j]
            assert row[tok] >= row.max() - 1e-3, f"token {j} of a prompt of {len(p)} is not the plain model's choice"


def test_a_conversation_over_memory_and_windows(made, tmp_path):
    """``Model.chat``: a turn that goes on runs only the new tokens; a history that parts from the cached tokens starts over
    (a state has no earlier value); a saved conversation goes on in another model object with the same tokens."""
    from turboquant_cpp_amd import Model
    d, cfg, w = made("regular", seed=5)
    opts = dict(dtype="float32", temperature=0.0, rep_penalty=1.0, max_tokens=5, context_length=512)
    h1, extra, other, more = (tokens(cfg, n, 70 + n) for n in (70, 9, 150, 5))
    with Model(d, **opts) as m, Model(d, **opts) as fresh:
        brought = []
        step = m.engine.step
        m.engine.step = lambda slots, toks, *a, **k: (brought.append(len(toks[0])), step(slots, toks, *a, **k))[1]
        out1 = m.chat(h1)
        assert out1 == fresh.generate([h1])[0] and brought[0] == 70
        del brought[:]
        h2 = h1 + out1 + extra
        out2 = m.chat(h2)
        assert brought[0] == 1 + len(extra) and out2 == fresh.generate([h2])[0]
        saved = str(tmp_path / "talk.kv")
        m.save_context(saved)
        del brought[:]
        h3 = h1[:40] + other
        assert m.chat(h3) == fresh.generate([h3])[0] and brought[0] == len(h3)
        with Model(d, **opts) as later:
            later.load_context(saved)
            h4 = h2 + out2 + more
            assert later.chat(h4) == fresh.generate([h4])[0]


def test_command_line(made):
    """``bin/quant``: what it says of the folder, and greedy tokens that are the entry point's."""
    from turboquant_cpp_amd import Model
    d, cfg, w = made("regular", seed=5)
    quant = os.path.join(ROOT, "bin", "quant")
    info = subprocess.run([quant, d, "--info"], capture_output=True, text=True, timeout=300)
    assert info.returncode == 0 and "Gokezen" in info.stdout, info.stderr[-1000:]
    run = subprocess.run([quant, d, "-p", "5,17,3;8,1", "-n", "6", "-T", "0", "--rep-penalty", "1.0", "--dtype", "float32",
                          "--json", "-M"], capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    with Model(d, dtype="float32", temperature=0.0, rep_penalty=1.0, max_tokens=6) as m:
        want = m.generate([[5, 17, 3], [8, 1]])
    got = [r["tokens"] for r in json.loads(run.stdout.strip().splitlines()[-1])]
    assert got == want


def test_trace_runner_as_a_program(made, tmp_path):
    d, cfg, w = made("odd", seed=6)
    a, b = tokens(cfg, 90, 60), tokens(cfg, 41, 61)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:80], "want": [0, 41, 79]}, {"id": "b", "tokens": b[:40], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[80:81], "want": [0]}, {"id": "b", "tokens": b[40:], "want": [0]}], "end": ["b"]}]
    steps += [{"step": 2 + i, "entries": [{"id": "a", "tokens": [t], "want": [0] if i % 2 else []}], "end": ["a"] if i == 8 else []}
              for i, t in enumerate(a[81:])]
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / dtype
        run = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", dtype, "--out", str(out),
                              "--max-tokens", "256"], input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
                             capture_output=True, timeout=600)
        assert run.returncode == 0, run.stderr[-2000:]
        assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
        (wa, ca), (wb, cb) = ((plain.forward(cfg, w, t), clear_choices(cfg, w, t)) for t in (a, b))
        V = cfg["vocab"]

        def close(i, want, clear):
            got = np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, V)
            assert got.shape == want.shape
            if dtype == "float32":
                check(got, want, what=f"step {i}")
            else:       # (single rows: where a choice of experts was close, rounding may have turned it)
                assert (errors(got, want)[clear] < 0.15).all(), f"step {i}: {errors(got, want)}"
        close(0, wa[[0, 41, 79]], ca[[0, 41, 79]])
        close(1, np.stack([wa[80], wb[40]]), np.array([ca[80], cb[40]]))
        for i in range(9):
            if i % 2:
                close(2 + i, wa[81 + i:82 + i], ca[81 + i:82 + i])
            else:
                assert not (out / f"{2 + i}.f32").exists()
