"""Kiduvik on the GPU against the plain restatement of the design (tests/kiduvik_reference.py): every mechanism alone, prompts against token-by-token decoding, portions down to
two tokens, unequal batches, pages and slots that are used again, one key that stands out far back, at page borders, at the borders of the kernels' key tiles, just inside and just
outside a window and among the kept first keys, the first tokens of a sequence, long decoding, shapes of every attention kernel, and greedy generation through the engine's
scheduler."""
import copy

import numpy as np
import pytest

import nvr_import
from rugudra_util import Driver, TOL, row_errors
from kiduvik_util import as64, dense, diff, expected_logits, latent, make_config, make_key_stand_out, make_weights
import kiduvik_reference as ref

pytestmark = pytest.mark.gpu


def tokens_of(n, vocab, seed, lo=0):
    return np.random.default_rng(seed).integers(lo, vocab, n).tolist()


def check(got, want, dtype, what=""):
    e = row_errors(got, want)
    assert e.max() < TOL[dtype], f"{what}: row {int(e.argmax())} differs by {e.max():.3g} of the row's spread (limit {TOL[dtype]})"


# ------------------------------------------------------------------------------------------------ each mechanism alone
MECHANISMS = {
    "latent": make_config([latent(), latent()]),
    "latent_shared_with_the_layer_before": make_config([latent(), latent(kv_from=0)]),
    "latent_shared_by_several_of_other_sizes": make_config([latent(kv_rank=32), latent(kv_rank=16), latent(kv_from=0, kv_rank=32, heads=5, dim=8, vdim=24, scale=0.2), latent(kv_from=1, kv_rank=16, mlp=None),
                                                            latent(kv_from=0, kv_rank=32, heads=1, dim=40, vdim=8)]),
    "latent_one_head": make_config([latent(heads=1, dim=24, vdim=40, kv_rank=16, rot_dim=2)]),
    "latent_odd_sizes": make_config([latent(heads=5, dim=7, vdim=5, kv_rank=9, rot_dim=6), latent(kv_from=0, heads=3, dim=1, vdim=1, kv_rank=9, rot_dim=6)], width=60),
    "latent_rank_above_everything": make_config([latent(heads=2, dim=8, vdim=8, kv_rank=200, rot_dim=40), latent(heads=3, dim=8, vdim=8, kv_rank=208, rot_dim=48)]),
    "latent_rows_past_the_matrix_core_kernel": make_config([latent(heads=2, dim=16, vdim=16, kv_rank=264, rot_dim=16)]),
    "latent_rows_of_88": make_config([latent(heads=3, dim=16, vdim=16, kv_rank=72, rot_dim=16)]),
    "latent_fourteen_heads": make_config([latent(heads=14, dim=16, vdim=8, kv_rank=16, rot_dim=16)]),
    "latent_thirty_four_heads": make_config([latent(heads=34, dim=8, vdim=8, kv_rank=32, rot_dim=32)]),
    "latent_heads_of_64": make_config([latent(heads=3, dim=48, vdim=64, kv_rank=48, rot_dim=16), latent(heads=4, dim=56, vdim=64, kv_rank=48, rot_dim=16, kv_from=0)], width=96),
    "latent_heads_of_128": make_config([latent(heads=2, dim=64, vdim=128, kv_rank=96, rot_dim=64, base=30000.0)], width=96),
    "latent_windowed": make_config([latent(mask=(9, 2)), latent(heads=2, dim=56, vdim=64, kv_rank=48, rot_dim=8, mask=(20, 0))]),
    "differential": make_config([diff(), diff()]),
    "differential_everything_visible": make_config([diff(mask=None), diff(mask=(1000, 3))]),
    "differential_itself_only": make_config([diff(mask=(1, 0)), diff(mask=(1, 1))]),
    "differential_kept_keys_past_the_window": make_config([diff(mask=(5, 24)), diff(mask=(24, 24)), diff(mask=(2, 64))]),
    "differential_nothing_kept": make_config([diff(mask=(17, 0))]),
    "differential_nothing_rotated": make_config([diff(rot=None), diff(rot=0, scaling=None)]),
    "differential_two_numbers_rotated": make_config([diff(rot=2, scaling=None)]),
    "differential_everything_rotated": make_config([diff(rot=16), diff(dim=24, vdim=16, rot=24)]),
    "differential_frequencies_kept": make_config([diff(rot=16, scaling=(4.0, 2000, 0.01, 0.001))]),
    "differential_frequencies_divided": make_config([diff(rot=16, base=3.0, scaling=(4.0, 10, 1000.0, 500.0))]),
    "differential_frequencies_split_at_once": make_config([diff(rot=16, scaling=(5.0, 300, 3.0, 3.0))]),
    "differential_share_without_fixed_part": make_config([diff(share=0.0), diff(share=0.8)]),
    "differential_one_head": make_config([diff(heads=1, kv_heads=1, dim=8, vdim=8)]),
    "differential_odd_sizes": make_config([diff(heads=3, kv_heads=1, dim=9, vdim=5, rot=6), diff(heads=5, kv_heads=5, dim=7, vdim=1, rot=4)], width=60),
    "differential_keys_of_one_number": make_config([diff(heads=4, kv_heads=2, dim=1, vdim=16, rot=None, scale=1.0)], eps=0.2),      # (a norm over one number is a sign where eps is small)
    "differential_keys_of_24_values_of_40": make_config([diff(heads=6, kv_heads=3, dim=24, vdim=40, rot=16)]),
    "differential_keys_of_20": make_config([diff(heads=2, kv_heads=1, dim=20, vdim=40, rot=20)]),
    "differential_keys_of_128_values_of_256": make_config([diff(heads=2, kv_heads=1, dim=128, vdim=256, rot=64)]),
    "differential_keys_of_136": make_config([diff(heads=2, kv_heads=1, dim=136, vdim=24, rot=128)]),
    "differential_keys_of_32_ungrouped": make_config([diff(heads=3, kv_heads=3, dim=32, vdim=64, rot=32)], width=96),
    "differential_keys_of_32_in_twos": make_config([diff(heads=4, kv_heads=2, dim=32, vdim=64, rot=16)], width=96),
    "differential_keys_of_32_in_fours": make_config([diff(heads=8, kv_heads=2, dim=32, vdim=64, rot=12)], width=96),
    "differential_keys_of_32_in_eights": make_config([diff(heads=8, kv_heads=1, dim=32, vdim=64, rot=32)], width=96),
    "differential_keys_of_32_in_tens": make_config([diff(heads=10, kv_heads=1, dim=32, vdim=64, rot=32)], width=96),
    "differential_keys_of_64_ungrouped": make_config([diff(heads=2, kv_heads=2, dim=64, vdim=128, rot=48)], width=128),
    "differential_keys_of_64_in_fours": make_config([diff(heads=4, kv_heads=1, dim=64, vdim=128, rot=64, mask=None)], width=128),
    "feed_forward_sizes": make_config([latent(mlp=dense(1)), diff(mlp=dense(50)), latent(mlp=dense(128))], width=96),
    "no_feed_forward": make_config([latent(mlp=None), diff(mlp=None)]),
    "token_input_of_one_number": make_config([latent(), diff()], side=1, eps=0.2),
    "token_input_of_32": make_config([latent(), diff(mlp=None)], side=32),
    "no_token_input": make_config([latent(), diff(mlp=None), latent()], side=0),
    "large_eps": make_config([latent(), diff()], eps=0.05),
    "width_not_a_multiple_of_four": make_config([latent(), diff()], width=70),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_alone(name, dtype):
    cfg = MECHANISMS[name]
    w = make_weights(cfg, seed=len(name))
    toks = tokens_of(75, cfg["vocab"], 1)
    want = expected_logits(cfg, w, toks)
    check(Driver(cfg, w, dtype).run_alone(toks), want, dtype, name)
    check(Driver(cfg, w, dtype, page=8).run_alone(toks, cuts=[41, 3, 1]), want, dtype, name + ", in portions")


def test_each_part_changes_the_result():
    """A part that is left out must show: with one tensor or constant changed, the restatement's logits move by far more than the tolerance, and the engine follows."""
    cfg = make_config([latent(), diff(rot=12, mask=(20, 4)), latent(kv_from=0, heads=2)])
    w = make_weights(cfg, seed=11)
    toks = tokens_of(60, cfg["vocab"], 4)
    full = expected_logits(cfg, w, toks)
    check(Driver(cfg, w, "float32").run_alone(toks), full, "float32", "full")
    half = lambda k: np.where(np.arange(w[k].size).reshape(w[k].shape) % 2 == 0, w[k], 0.25).astype(np.float32)
    for key in ("pos", "side.embed", "l0.norm1", "l0.norm1b", "l1.norm2", "l1.norm2b", "final.norm", "l0.mix.dkv.norm", "l0.mix.sink", "l2.mix.sink", "l2.mix.uk", "l2.mix.uv", "l1.mix.q.norm", "l1.mix.k.norm",
                "l1.mix.lq1", "l1.mix.lk1", "l1.mix.lq2", "l1.mix.lk2", "l1.mix.g", "l1.mlp.up", "l2.side.gate", "l0.side.proj", "l1.side.norm"):
        w2 = dict(w); w2[key] = half(key)
        want = expected_logits(cfg, w2, toks)
        assert row_errors(want, full).max() > 20 * TOL["float32"], key
        check(Driver(cfg, w2, "float32").run_alone(toks), want, "float32", key)
    for change in (lambda c: c["layers"][0]["mixer"]["rot"].update(base=3.0), lambda c: c["layers"][0]["mixer"].update(scale=0.1), lambda c: c["layers"][2]["mixer"].update(scale=0.5),
                   lambda c: c["layers"][1]["mixer"]["rot"].update(base=40.0), lambda c: c["layers"][1]["mixer"]["rot"].update(dims=6), lambda c: c["layers"][1]["mixer"]["rot"].pop("scaling"),
                   lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=1.5), lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(original=8),
                   lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(fast=2.0), lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(slow=6.0),
                   lambda c: c["layers"][1]["mixer"].update(diff=0.6), lambda c: c["layers"][1]["mixer"].update(scale=0.1), lambda c: c["layers"][1]["mixer"]["mask"].update(size=19),
                   lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=5), lambda c: c["norm"].update(eps=0.3)):
        cfg2 = copy.deepcopy(cfg); change(cfg2)
        want = expected_logits(cfg2, w, toks)
        assert row_errors(want, full).max() > 20 * TOL["float32"]
        check(Driver(cfg2, w, "float32").run_alone(toks), want, "float32", "a constant of the configuration")


# ------------------------------------------------------------------------------------------------ a model with everything, in portions and batches
def everything(vocab=113, width=96):
    return make_config([diff(heads=6, kv_heads=3, dim=24, vdim=40, rot=16, mask=(22, 7), mlp=dense(72)), latent(heads=4, dim=24, vdim=16, kv_rank=40, rot_dim=16),
                        latent(heads=2, dim=40, vdim=24, kv_rank=40, rot_dim=16, kv_from=1, mlp=None), diff(heads=2, kv_heads=1, dim=16, vdim=16, rot=None, mask=(5, 0), share=0.55),
                        latent(heads=5, dim=8, vdim=8, kv_rank=24, rot_dim=4, base=90.0), latent(heads=3, dim=16, vdim=32, kv_rank=40, rot_dim=16, kv_from=1)], vocab=vocab, width=width, side=12)


def with_flash(vocab=97, width=128):
    return make_config([diff(heads=4, kv_heads=2, dim=32, vdim=64, rot=32, mask=(33, 6)), latent(heads=3, dim=48, vdim=64, kv_rank=48, rot_dim=16), diff(heads=2, kv_heads=2, dim=64, vdim=128, rot=32, mask=(16, 17)),
                        latent(heads=4, dim=48, vdim=64, kv_rank=48, rot_dim=16, kv_from=1, mlp=None), diff(heads=8, kv_heads=2, dim=32, vdim=64, rot=8, mask=None)], vocab=vocab, width=width, side=16)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("model", [everything, with_flash])
def test_prompt_against_token_by_token_decoding(model, dtype):
    cfg = model(); w = make_weights(cfg, seed=5)
    toks = tokens_of(60, cfg["vocab"], 3)
    want = expected_logits(cfg, w, toks)
    check(Driver(cfg, w, dtype).run_alone(toks), want, dtype, "whole prompt")
    check(Driver(cfg, w, dtype, page=8).run_alone(toks, cuts=[1]), want, dtype, "token by token")
    check(Driver(cfg, w, dtype, page=8).run_alone(toks, cuts=[37, 1]), want, dtype, "a prompt, then token by token")


@pytest.mark.parametrize("cuts", [[2], [3, 2, 17, 2, 5], [16], [15, 17], [33, 2, 1], [64, 7], [20, 1, 21, 1]])
@pytest.mark.parametrize("model, dtype", [(everything, "float32"), (everything, "bfloat16"), (with_flash, "bfloat16")])
def test_portions(model, dtype, cuts):
    cfg = model(); w = make_weights(cfg, seed=6)
    toks = tokens_of(85, cfg["vocab"], 7)
    check(Driver(cfg, w, dtype, page=16).run_alone(toks, cuts=cuts), expected_logits(cfg, w, toks), dtype, f"portions {cuts}")


def test_first_tokens():
    cfg = everything(); w = make_weights(cfg, seed=21)
    toks = tokens_of(12, cfg["vocab"], 22)
    want = expected_logits(cfg, w, toks)
    for n in (1, 2, 3):
        check(Driver(cfg, w, "float32", page=8).run_alone(toks[:n]), want[:n], "float32", f"{n} tokens")
        check(Driver(cfg, w, "float32", page=8).run_alone(toks, cuts=[n, 1, 2]), want, "float32", f"{n} tokens first")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("model", [everything, with_flash])
def test_unequal_batches_with_pages_and_slots_used_again(model, dtype):
    """Five requests of different lengths through three state slots and a pool of pages that cannot hold them all at once: portions of some beside single
    tokens of others; a finished request's pages and slot go to the next one.  Every request must come out as it does alone."""
    cfg = model(); w = make_weights(cfg, seed=8)
    reqs = {n: tokens_of(ln, cfg["vocab"], 20 + k) for k, (n, ln) in enumerate([("a", 61), ("b", 9), ("c", 34), ("d", 47), ("e", 2)])}
    want = {n: expected_logits(cfg, w, t) for n, t in reqs.items()}
    d = Driver(cfg, w, dtype, page=8, pages=20, slots=3, max_tokens=256)
    at = {n: 0 for n in reqs}
    got = {n: [] for n in reqs}
    waiting, live = ["a", "b", "c", "d", "e"], []
    sizes, k = [5, 1, 2, 11, 1, 1, 3, 8, 1, 2], 0
    while waiting or live:
        while waiting and len(live) < 3 and sum((len(reqs[n]) + 7) // 8 for n in live + waiting[:1]) <= 20:
            live.append(waiting.pop(0))
        entries = []
        for n in live:
            c = min(sizes[k % len(sizes)], len(reqs[n]) - at[n]); k += 1
            entries.append((n, reqs[n][at[n]:at[n] + c]))
            at[n] += c
        out = d.step(entries)
        for n, _ in entries:
            got[n].append(out[n])
        for n in [n for n in live if at[n] == len(reqs[n])]:
            d.end(n); live.remove(n)
    for n in reqs:
        check(np.concatenate(got[n]), want[n], dtype, f"request {n}")


@pytest.mark.parametrize("model, dtype", [(everything, "float32"), (with_flash, "bfloat16")])
def test_whole_prompts_of_a_batch(model, dtype):
    """Several whole prompts in one step (keys and values expanded for the step), of lengths around the query tiles' sizes."""
    cfg = model(); w = make_weights(cfg, seed=9)
    reqs = {"r%d" % n: tokens_of(n, cfg["vocab"], 50 + n) for n in (1, 129, 64, 17, 65)}
    d = Driver(cfg, w, dtype, page=16, pages=40, slots=5, max_tokens=512)
    out = d.step(list(reqs.items()))
    for n, t in reqs.items():
        check(out[n], expected_logits(cfg, w, t), dtype, f"prompt {n}")


def test_a_request_left_out_of_steps():
    cfg = everything(); w = make_weights(cfg, seed=31)
    a, b = tokens_of(30, cfg["vocab"], 32), tokens_of(26, cfg["vocab"], 33)
    d = Driver(cfg, w, "float32", page=8, slots=2)
    ga, gb = [], []
    out = d.step([("a", a[:7]), ("b", b[:3])]); ga.append(out["a"]); gb.append(out["b"])
    for i in range(3, 20):
        gb.append(d.step([("b", b[i:i + 1])])["b"])
    out = d.step([("a", a[7:9]), ("b", b[20:])]); ga.append(out["a"]); gb.append(out["b"])
    ga.append(d.step([("a", a[9:])])["a"])
    check(np.concatenate(ga), expected_logits(cfg, w, a), "float32", "the request that waited")
    check(np.concatenate(gb), expected_logits(cfg, w, b), "float32", "the request that went on")


# ------------------------------------------------------------------------------------------------ one key that stands out
WIN, KEEP = 100, 21
PROBE_LAYERS = {
    "differential_general": (diff(heads=2, kv_heads=1, dim=9, vdim=10, rot=6, mask=(WIN, KEEP), mlp=None), 48, 0),
    "differential_small_heads": (diff(heads=4, kv_heads=2, dim=16, vdim=24, rot=8, mask=(WIN, KEEP), mlp=None), 48, 1),
    "differential_keys_of_32": (diff(heads=4, kv_heads=2, dim=32, vdim=64, rot=16, mask=(WIN, KEEP), mlp=None), 64, 0),
    "differential_keys_of_64": (diff(heads=4, kv_heads=1, dim=64, vdim=128, rot=32, mask=(WIN, KEEP), mlp=None), 64, 0),
    "differential_keys_of_64_no_window": (diff(heads=2, kv_heads=2, dim=64, vdim=128, rot=32, mask=None, mlp=None), 64, 0),
    "latent": (latent(heads=3, dim=16, rot_dim=8, vdim=16, kv_rank=24, mlp=None), 48, 0),
    "latent_heads_of_64": (latent(heads=2, dim=48, rot_dim=16, vdim=64, kv_rank=48, mlp=None), 64, 0),
    "latent_heads_of_128": (latent(heads=2, dim=96, rot_dim=32, vdim=128, kv_rank=64, mlp=None), 64, 0),
}
PLACES = [(599, 0), (599, 1), (599, 7), (599, 8), (599, 63), (599, 64), (599, 87), (599, 88), (599, WIN - 2), (599, WIN - 1), (599, WIN), (599, WIN + 1), (599, 343), (599, 599 - KEEP), (599, 599 - KEEP + 1), (599, 598), (599, 599),
          (512, 256), (512, 512), (127, WIN - 1), (127, WIN), (128, 64), (WIN, WIN), (WIN - 1, WIN - 1), (WIN + KEEP, WIN), (WIN + KEEP - 1, WIN), (64, 64), (63, 63), (1, 1)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", sorted(PROBE_LAYERS))
@pytest.mark.parametrize("last, back", PLACES)
def test_one_key_stands_out(kind, last, back, dtype):
    """Token K occurs once, `back` positions before the last token Q (at position `last`), whose queries score far higher with K's keys than with any other: that one key decides the
    last row where it is visible, and must not be seen where it is not (8-token pages; page borders, borders of 64-key tiles, both sides of the window's edge and of the kept keys'
    end, the first position, far back).  The engine must agree with the restatement as a whole prompt, with the last token decoded alone, with the last token ending a short
    portion, and with a portion that starts at the key; a key of a DIFFERENT sequence in the same step must not be seen."""
    layer0, width, which = PROBE_LAYERS[kind]
    mask = layer0["mixer"].get("mask")
    if mask is None and back in (WIN - 2, WIN - 1, WIN, WIN + 1, 599 - KEEP, 599 - KEEP + 1) and last != back:
        pytest.skip("this layer has no window")
    if kind == "differential_general" and dtype == "bfloat16" and back not in (0, 8, WIN - 1, WIN, 599):
        pytest.skip("the general kernel is the float32 case's")
    cfg = make_config([copy.deepcopy(layer0)], vocab=31, width=width, side=0)
    Q, K, n, at = 0, 1, last + 1, last - back
    w = make_key_stand_out(cfg, make_weights(cfg, seed=9), Q, K, which=which)
    toks = tokens_of(n, cfg["vocab"], 10 + back, lo=2)
    toks[-1] = Q
    if back:
        toks[at] = K
    want = expected_logits(cfg, w, toks)
    moved = 0.0
    if back:
        seen = mask is None or back < mask["size"] or at < mask["keep_first"]
        c2 = copy.deepcopy(cfg)
        if mask is not None:                                # the restatement with this one key on the other side of the mask
            c2["layers"][0]["mixer"]["mask"] = {"size": back, "keep_first": min(mask["keep_first"], at)} if seen else {"size": back + 1, "keep_first": mask["keep_first"]}
            wrong = expected_logits(c2, w, toks)
        else:
            gone = list(toks); gone[at] = 2
            wrong = expected_logits(cfg, w, gone)
        moved = row_errors(wrong[-1:], want[-1:]).max()
        assert moved > 4 * TOL[dtype], "the key must decide the row"
    for cuts, what in (([n], "whole"), ([max(n - 1, 1), 1], "decoded"), ([max(n - 3, 1), 3], "end of a portion"), ([n - back - 1, back + 1] if 0 < back < n - 1 else [max(n - 2, 1), 2], "a portion from the key on")):
        got = Driver(cfg, w, dtype, page=8, pages=80, max_tokens=640, max_len=640).run_alone(toks, cuts=cuts)
        check(got[-4:], want[-4:], dtype, f"{what}, {back} back of {last}")
        if back:
            assert row_errors(got[-1:], want[-1:]).max() < moved / 4, f"{what}, {back} back: the last row is off by a quarter of what the key moves it"
    d = Driver(cfg, w, dtype, page=8, pages=90, slots=2, max_tokens=700, max_len=640)
    d.step([("k", [K] * 20)])
    out = d.step([("k", [K]), ("r", toks)])
    check(out["r"][-4:], want[-4:], dtype, f"beside a sequence of such keys, {back} back of {last}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", [dict(heads=3, dim=16, rot_dim=8, vdim=16, kv_rank=24), dict(heads=2, dim=48, rot_dim=16, vdim=64, kv_rank=48)])
def test_a_sink_that_takes_most(shape, dtype):
    """A sink far above the scores, alone in the first head: without it, or counted more than once over split keys, the head's share of the row would be another."""
    cfg = make_config([latent(mlp=None, **shape)], vocab=31, width=64, positions=1000, side=0)
    w = make_weights(cfg, seed=41)
    w["l0.mix.sink"] = np.array([7.0] + [-9.0] * (shape["heads"] - 1), np.float32)
    toks = tokens_of(900, 31, 42)
    want = expected_logits(cfg, w, toks)
    w2 = dict(w); w2["l0.mix.sink"] = w["l0.mix.sink"] + np.array([np.log(2.0)] + [0.0] * (shape["heads"] - 1), np.float32)
    assert np.median(row_errors(expected_logits(cfg, w2, toks), want)) > TOL[dtype]
    for cuts in ([900], [890, 1], [450, 448, 1]):
        check(Driver(cfg, w, dtype, page=16, pages=60, max_tokens=1024, max_len=1000).run_alone(toks, cuts=cuts), want, dtype, f"portions {cuts}")


# ------------------------------------------------------------------------------------------------ long sequences, many rows
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("model", [everything, with_flash])
def test_long_decoding(model, dtype):
    cfg = model(); w = make_weights(cfg, seed=34)
    toks = tokens_of(200, cfg["vocab"], 15)
    got = Driver(cfg, w, dtype, page=8, pages=32).run_alone(toks, cuts=[10, 1])
    check(got, expected_logits(cfg, w, toks), dtype, "190 decoded tokens")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [256, 1280])
def test_long_prompts_and_decoding_side_by_side(width, dtype):
    """1100 and 900 tokens: prompts cross many query and key tiles, the products take their large tiles (the GELU in the epilogue where it fits), the norm joins their wave-per-row
    form or, wider, a workgroup per row; two requests then decode side by side with their keys split over workgroups."""
    cfg = make_config([diff(heads=4, kv_heads=2, dim=64, vdim=128, rot=64, base=20000.0, scaling=(4.0, 400, 32.0, 1.0), mask=(600, 70), mlp=dense(512)),
                       latent(heads=4, dim=64, vdim=128, kv_rank=64, rot_dim=64, mlp=dense(256)), latent(heads=6, dim=24, vdim=40, kv_rank=64, rot_dim=64, kv_from=1, mlp=None),
                       diff(heads=6, kv_heads=3, dim=24, vdim=40, rot=24, mask=None, mlp=dense(256))], vocab=71, width=width, positions=1300, side=32)
    w = make_weights(cfg, seed=24)
    a, b = tokens_of(1100, 71, 25), tokens_of(900, 71, 26)
    wa, wb = expected_logits(cfg, w, a), expected_logits(cfg, w, b)
    d = Driver(cfg, w, dtype, page=64, pages=40, slots=2, max_tokens=2048, max_len=1200)
    ga, gb = [d.step([("a", a[:1080]), ("b", b[:880])])], []
    gb.append(ga[0]["b"]); ga[0] = ga[0]["a"]
    for i in range(20):
        out = d.step([("a", a[1080 + i:1081 + i]), ("b", b[880 + i:881 + i])])
        ga.append(out["a"]); gb.append(out["b"])
    check(np.concatenate(ga), wa, dtype, "first request")
    check(np.concatenate(gb), wb, dtype, "second request")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("count", [17, 70])
def test_many_sequences_decode_side_by_side(count, dtype):
    """More sequences in a decode-sized step than a tile of the products has rows, and more than the one-launch token input takes; contexts from 1 to 300 tokens."""
    cfg = make_config([diff(heads=4, kv_heads=2, dim=32, vdim=64, rot=32, mask=(40, 9)), latent(heads=20, dim=48, vdim=64, kv_rank=48, rot_dim=16, mlp=None)], vocab=97, width=96, side=16)
    w = make_weights(cfg, seed=61)
    reqs = {"s%d" % k: tokens_of(4 + (k * 37) % 300 if k % 3 == 0 else 4 + k % 7, 97, 700 + k) for k in range(count)}
    d = Driver(cfg, w, dtype, page=16, pages=count * 20, slots=count, max_tokens=8192, max_len=320)
    got = {n: [] for n in reqs}
    for cut in (slice(0, -3), slice(-3, -2), slice(-2, -1), slice(-1, None)):
        out = d.step([(n, t[cut]) for n, t in reqs.items()])
        for n in reqs:
            got[n].append(out[n])
    for n, t in reqs.items():
        check(np.concatenate(got[n]), expected_logits(cfg, w, t), dtype, f"request {n}")


def test_decode_steps_replay_a_graph():
    """Decode-sized steps are captured the second time their shape is seen and replayed from then on; every replay is compared."""
    for model, dtype in ((everything, "float32"), (with_flash, "bfloat16")):
        cfg = model(); w = make_weights(cfg, seed=16)
        toks = tokens_of(48, cfg["vocab"], 17)
        check(Driver(cfg, w, dtype, page=8).run_alone(toks, cuts=[8, 1]), expected_logits(cfg, w, toks), dtype, "replayed steps")


# ------------------------------------------------------------------------------------------------ through the engine's own entry point
@pytest.mark.parametrize("chunked", [0, 1])
def test_greedy_generation_through_the_scheduler(chunked):
    """Five requests through LLMEngine.add_request / step with three state slots and a token budget that cuts prompts (chunked) or batches them whole: every
    generated token is the arg-max of the restatement's logits for the sequence so far."""
    nvr = nvr_import.load()
    cfg = everything(); w = make_weights(cfg, seed=18)
    prompts = [tokens_of(n, cfg["vocab"], 30 + n) for n in (5, 23, 1, 40, 12)]
    new = 12
    eng = nvr.LLMEngine(nvr.Config(dtype="float32", kvcache_block_size=8, skip_block_size_check=1, num_kvcache_blocks=40, max_num_seqs=3, num_state_slots=3,
                                   max_num_batched_tokens=32 if chunked else 256, max_model_len=128, enable_chunked_prefill=chunked), nvr.ModelSpec(cfg))
    for k, v in w.items():
        eng.model_runner.load_tensor(k, np.asarray(v, dtype=np.float32))
    ids = [eng.add_request(p, nvr.SamplingParams(temperature=0.0, max_tokens=new, ignore_eos=True)) for p in prompts]
    steps = 0
    while not eng.is_finished():
        eng.step(); steps += 1
        assert steps < 400
    done = {s.seq_id: s for s in eng.take_finished()}
    assert sorted(done) == sorted(ids)
    w64 = as64(w)
    for sid, p in zip(ids, prompts):
        full = done[sid].token_ids
        assert full[:len(p)] == p and len(full) == len(p) + new
        lg = ref.forward(cfg, w64, full[:-1])[0]
        for k in range(len(p) - 1, len(full) - 1):
            row = lg[k]
            spread = np.sqrt(((row - row.mean()) ** 2).mean())
            assert row.max() - row[full[k + 1]] <= 3 * TOL["float32"] * spread, f"request {sid}: token {k + 1} is not the greedy choice"


def test_positions_end_with_the_table():
    """A sequence may use every learned position and not one more."""
    nvr = nvr_import.load()
    cfg = make_config([diff(), latent()], positions=40); w = make_weights(cfg, seed=44)
    toks = tokens_of(41, cfg["vocab"], 45)
    d = Driver(cfg, w, "float32", page=8)
    got = [d.step([("r", toks[:39])])["r"], d.step([("r", toks[39:40])])["r"]]
    check(np.concatenate(got), expected_logits(cfg, w, toks[:40]), "float32", "forty positions")
    with pytest.raises(nvr.NvrError):
        d.step([("r", toks[40:])])


def test_tensors_of_other_shapes_are_refused():
    nvr = nvr_import.load()
    cfg = make_config([latent(), diff(), latent(kv_from=0)]); w = make_weights(cfg, seed=2)
    d = Driver(cfg, w, "float32")
    for name, shape in (("pos", (3, 64)), ("l0.mix.q", (48, 64)), ("l0.mix.dkv", (24, 64)), ("l0.mix.sink", (4,)), ("l2.mix.dkv", (32, 64)), ("l1.mix.q", (64, 64)), ("l1.mix.k.norm", (32,)),
                        ("l1.mix.lq1", (8,)), ("l1.mix.g", (128, 64)), ("l1.mix.sink", (4,)), ("l0.mix.g", (36, 64)), ("l0.dwa", (2,)), ("l3.norm1", (64,)), ("lx.norm1", (64,)), ("l0.mlp.act", (4,))):
        with pytest.raises(nvr.NvrError):
            d.engine.model_runner.load_tensor(name, np.zeros(shape, np.float32))


# ------------------------------------------------------------------------------------------------ designs and schedules drawn at random
def random_design(seed):
    rng = np.random.default_rng(seed)
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers, own = [], []
    for i in range(int(rng.integers(1, 7))):
        mlp = pick([None, dense(pick([8, 24, 100, 128])), dense(64)])
        if rng.random() < 0.5:
            src = pick(own) if own and rng.random() < 0.5 else None
            m = layers[src]["mixer"] if src is not None else None
            rank, R, base = (m["kv_rank"], m["rot_dim"], m["rot"]["base"]) if m else (pick([8, 20, 32, 48, 80]), pick([2, 8, 16, 32]), pick([10.0, 500.0, 100000.0]))
            if src is None:
                own.append(i)
            D = pick([8, 12, 32, 48, 64 - R])
            layers.append(latent(heads=pick([1, 2, 3, 6]), dim=D, vdim=pick([8, 9, 24, D + R]), kv_rank=rank, rot_dim=R, base=base, kv_from=src, scale=float(rng.uniform(0.05, 0.4)), mlp=mlp))
        else:
            G, D = int(rng.integers(1, 4)), pick([8, 12, 24, 32, 32, 48])
            layers.append(diff(heads=G * pick([1, 2, 3, 4]), kv_heads=G, dim=D, vdim=pick([8, 9, 2 * D, 2 * D]), rot=pick([None, 2, D // 4 * 2, D]), base=pick([10.0, 500.0, 100000.0]), scale=float(rng.uniform(0.05, 0.6)),
                               scaling=pick([None, (4.0, 64, 8.0, 1.0), (2.0, 1000, 32.0, 0.5), (8.0, 20, 4.0, 2.0)]), mask=pick([None, (int(rng.integers(1, 60)), int(rng.integers(0, 40)))]), share=float(rng.uniform(0.0, 0.6)), mlp=mlp))
    return make_config(layers, vocab=int(rng.integers(40, 200)), width=pick([48, 64, 70, 96, 104, 128, 160]), side=pick([0, 6, 8, 32]), eps=pick([1e-6, 1e-5, 1e-3]))


@pytest.mark.parametrize("seed", range(14))
def test_random_designs_and_schedules(seed):
    """A design drawn at random (layer order, sizes, sharing, windows, rotations) runs a prompt whole, in random portions, and two requests of unequal length in
    one batch with their own portions, in both number formats."""
    cfg = random_design(100 + seed)
    w = make_weights(cfg, seed=200 + seed)
    rng = np.random.default_rng(300 + seed)
    a, b = tokens_of(int(rng.integers(20, 130)), cfg["vocab"], 400 + seed), tokens_of(int(rng.integers(2, 60)), cfg["vocab"], 500 + seed)
    wa, wb = expected_logits(cfg, w, a), expected_logits(cfg, w, b)
    for dtype in ("float32", "bfloat16"):
        check(Driver(cfg, w, dtype, page=8, pages=64).run_alone(a), wa, dtype, f"design {seed}, whole")
        cuts = [int(c) for c in rng.integers(1, 40, 12)] + [1]
        check(Driver(cfg, w, dtype, page=8, pages=64).run_alone(a, cuts=cuts), wa, dtype, f"design {seed}, portions {cuts}")
        d = Driver(cfg, w, dtype, page=8, pages=64, slots=2)
        at, got = {"a": 0, "b": 0}, {"a": [], "b": []}
        toks = {"a": a, "b": b}
        while at["a"] < len(a) or at["b"] < len(b):
            entries = []
            for n in ("a", "b"):
                if at[n] < len(toks[n]):
                    c = min(int(rng.integers(1, 24)), len(toks[n]) - at[n])
                    entries.append((n, toks[n][at[n]:at[n] + c])); at[n] += c
            out = d.step(entries)
            for n, _ in entries:
                got[n].append(out[n])
        check(np.concatenate(got["a"]), wa, dtype, f"design {seed}, batch, first request")
        check(np.concatenate(got["b"]), wb, dtype, f"design {seed}, batch, second request")
