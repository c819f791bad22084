"""Negunex on the GPU against the plain restatement of the design (tests/negunex_reference.py): every mechanism alone, prompts against token-by-token
decoding, portions down to two tokens, unequal batches, pages and state slots that are used again, one key that stands out far back, at page borders and at the
borders of the kernels' key tiles, the first tokens of a sequence, long decoding, sizes that are 1 or equal to each other, shapes of every attention kernel, the
experts' product over many rows, and greedy generation through the engine's scheduler."""
import copy

import numpy as np
import pytest

import nvr_import
from rugudra_util import Driver, TOL, row_errors
from negunex_util import as64, dense, expected_logits, layer, make_config, make_key_stand_out, make_weights, moe, settled_tokens
import negunex_reference as ref

pytestmark = pytest.mark.gpu


def tokens_of(n, vocab, seed, lo=0):
    return np.random.default_rng(seed).integers(lo, vocab, n).tolist()


def check(got, want, dtype, what=""):
    e = row_errors(got, want)
    assert e.max() < TOL[dtype], f"{what}: row {int(e.argmax())} differs by {e.max():.3g} of the row's spread (limit {TOL[dtype]})"


# ------------------------------------------------------------------------------------------------ each mechanism alone
MECHANISMS = {
    "two_streams": make_config([layer(mlp="dense"), layer(mlp="dense")]),
    "one_stream": make_config([layer(mlp="moe"), layer(mlp=None)], streams=1),
    "three_streams": make_config([layer(), layer(v_mix=False)], streams=3),
    "four_streams_odd_width": make_config([layer(), layer(mlp="moe")], streams=4, width=68),
    "seven_streams_width_not_a_multiple_of_four": make_config([layer(), layer(mlp="moe")], streams=7, width=70),
    "large_eps": make_config([layer(), layer(mlp="moe")], eps=0.05),
    "nothing_rotated": make_config([layer(rot=None), layer(rot=0)]),
    "two_numbers_rotated": make_config([layer(rot=2, scaling=None)]),
    "plain_frequencies": make_config([layer(scaling=None, base=40.0)]),
    "stretched_frequencies_all_branches": make_config([layer(dim=32, rot=32, base=3000.0, scaling=(8.0, 0.5, 2.0, 40))]),
    "stretch_without_a_blend": make_config([layer(dim=24, rot=20, base=90.0, scaling=(3.0, 2.0, 2.0, 50))]),
    "no_values_mixed": make_config([layer(v_mix=False), layer(v_mix=False)]),
    "values_mixed_from_the_second_layer_on": make_config([layer(v_mix=False), layer(), layer(v_mix=False, heads=6, kv_heads=3, dim=8, vdim=8), layer(), layer()]),
    "values_mixed_over_other_query_sizes": make_config([layer(heads=8, kv_heads=2, dim=32), layer(heads=2, kv_heads=2, dim=8, rot=4), layer(heads=4, kv_heads=2, dim=64)]),
    "one_head": make_config([layer(heads=1, kv_heads=1, dim=24, vdim=8, rot=24)]),
    "odd_heads": make_config([layer(heads=3, kv_heads=1, dim=9, vdim=5, rot=6), layer(heads=5, kv_heads=5, dim=7, vdim=1, rot=6, v_mix=False)], width=60),
    "keys_of_one_number": make_config([layer(heads=4, kv_heads=2, dim=1, vdim=16, rot=0, scale=2.0)]),
    "heads_of_64_in_groups_of_two": make_config([layer(heads=4, kv_heads=2, dim=64, vdim=64, rot=64)], width=96),
    "heads_of_64_in_groups_of_four": make_config([layer(heads=4, kv_heads=1, dim=64, vdim=64, rot=32), layer(heads=4, kv_heads=1, dim=64, vdim=64)], width=96),
    "heads_of_64_in_groups_of_eight": make_config([layer(heads=8, kv_heads=1, dim=64, vdim=64)], width=64),
    "heads_of_128_ungrouped": make_config([layer(heads=2, kv_heads=2, dim=128, vdim=128, rot=128), layer(heads=2, kv_heads=2, dim=128, vdim=128, rot=96, mlp=None)], width=128),
    "keys_of_64_values_of_32": make_config([layer(heads=6, kv_heads=2, dim=64, vdim=32, rot=40)], width=96),
    "keys_of_32_values_of_80": make_config([layer(heads=6, kv_heads=2, dim=32, vdim=80, rot=30)]),
    "keys_of_160_values_of_96": make_config([layer(heads=2, kv_heads=1, dim=160, vdim=96, rot=160), layer(heads=2, kv_heads=1, dim=256, vdim=96, rot=64)]),
    "keys_of_520": make_config([layer(heads=1, kv_heads=1, dim=520, vdim=16, rot=520)]),
    "twenty_heads_on_one": make_config([layer(heads=20, kv_heads=1, dim=32, vdim=16, rot=4)]),
    "dense_sizes": make_config([layer(mlp=dense(1)), layer(mlp=dense(50)), layer(mlp=dense(128))], width=96),
    "no_feed_forward": make_config([layer(mlp=None), layer(mlp=None)]),
    "experts_one_of_one": make_config([layer(mlp=moe(experts=1, top=1, ff=16, identity=0))]),
    "experts_without_identity": make_config([layer(mlp=moe(experts=5, top=2, ff=24, identity=None))]),
    "experts_all_chosen": make_config([layer(mlp=moe(experts=4, top=7, ff=24, identity=3))]),
    "experts_one_of_seventy": make_config([layer(mlp=moe(experts=66, top=1, ff=8, identity=4))]),
    "experts_more_identity_than_others": make_config([layer(mlp=moe(experts=2, top=3, ff=20, identity=9))], width=72),
    "experts_five_of_thirteen_odd_sizes": make_config([layer(mlp=moe(experts=9, top=5, ff=21, identity=4))], width=76),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_alone(name, dtype):
    cfg = MECHANISMS[name]
    w = make_weights(cfg, seed=len(name))
    toks = settled_tokens(cfg, w, 75, 1)
    want = expected_logits(cfg, w, toks)
    check(Driver(cfg, w, dtype).run_alone(toks), want, dtype, name)
    check(Driver(cfg, w, dtype, page=8).run_alone(toks, cuts=[41, 3, 1]), want, dtype, name + ", in portions")


def test_each_part_changes_the_result():
    """A part that is left out must show: with one tensor or constant changed, the restatement's logits move by far more than the tolerance, and the engine follows."""
    cfg = make_config([layer(rot=12), layer(mlp="moe")])
    w = make_weights(cfg, seed=11)
    toks = settled_tokens(cfg, w, 60, 4)
    full = expected_logits(cfg, w, toks)
    check(Driver(cfg, w, "float32").run_alone(toks), full, "float32", "full")
    for key, val in (("l0.hc2.in", 0.1), ("l0.hc1.out", 0.0), ("l0.hc2.mix", 0.5), ("l1.hc2.out", 1.0), ("l1.hc1.in", 0.2), ("l0.norm1", 0.3), ("l1.norm2", 2.0), ("l0.mix.q.b", 0.0), ("l0.mix.k.b", 0.0),
                     ("l1.mix.v.b", 0.0), ("l1.mix.vmix", 0.0), ("l1.mix.vmix", 1.0), ("l0.mix.g", 0.0), ("l1.mlp.correction", 0.0), ("l1.mlp.router", 0.0), ("final.norm", 0.5)):
        w2 = dict(w); w2[key] = np.full_like(w[key], val)
        if key == "l1.mlp.correction":
            w2[key] = bf16_ramp(len(w[key]))
        if key == "l0.hc2.mix":
            w2[key] = np.ascontiguousarray(w[key].T)         # (the matrix is indexed [from, to])
        if key in ("l0.norm1", "final.norm"):
            w2[key] = np.where(np.arange(len(w[key])) % 2 == 0, w[key], val).astype(np.float32)
        want = expected_logits(cfg, w2, toks)
        assert row_errors(want, full).max() > 20 * TOL["float32"], key
        check(Driver(cfg, w2, "float32").run_alone(toks), want, "float32", key)
    w2 = dict(w); w2["l0.mix.vmix"] = np.full_like(w["l0.mix.vmix"], 0.9)      # (the first layer's share is not used)
    assert np.array_equal(expected_logits(cfg, w2, toks), full)
    check(Driver(cfg, w2, "float32").run_alone(toks), full, "float32", "the first layer's share")
    for change in (lambda c: c["layers"][0]["mixer"]["rot"].update(base=3.0), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6), lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0.5),
                   lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(original=8), lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(high=30.0),
                   lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=3.0), lambda c: c["layers"][1]["mixer"].update(scale=0.1), lambda c: c["layers"][1]["mixer"].update(v_mix=False),
                   lambda c: c["norm"].update(eps=0.3)):
        cfg2 = copy.deepcopy(cfg); change(cfg2)
        want = expected_logits(cfg2, w, toks)
        assert row_errors(want, full).max() > 20 * TOL["float32"]
        check(Driver(cfg2, w, "float32").run_alone(toks), want, "float32", "a constant of the configuration")


def bf16_ramp(n):
    return (np.arange(n) * 0.5).astype(np.float32)


# ------------------------------------------------------------------------------------------------ a model with everything, in portions and batches
def everything(vocab=113, width=96, streams=3):
    return make_config([layer(heads=4, kv_heads=2, dim=32, vdim=32, rot=16, v_mix=False, mlp="dense"),
                        layer(heads=6, kv_heads=1, dim=16, vdim=80, mlp=moe(experts=5, top=3, ff=40, identity=2)),
                        layer(heads=3, kv_heads=1, dim=24, vdim=80, rot=24, mlp=None),
                        layer(heads=5, kv_heads=1, dim=64, vdim=80, base=9000.0, scaling=(8.0, 1.0, 3.0, 100), mlp=moe(experts=3, top=1, ff=56, identity=1)),
                        layer(heads=2, kv_heads=1, dim=64, vdim=80, rot=None, scale=0.2, mlp=dense(72))],
                       vocab=vocab, width=width, streams=streams)


def with_flash(vocab=97, width=128):
    return make_config([layer(heads=4, kv_heads=2, dim=64, vdim=64, rot=64), layer(heads=8, kv_heads=2, dim=64, vdim=64, rot=48, mlp=moe(experts=6, top=3, ff=64, identity=3)),
                        layer(heads=2, kv_heads=2, dim=64, vdim=64, rot=16, v_mix=True, mlp=None)], vocab=vocab, width=width)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("model", [everything, with_flash])
def test_prompt_against_token_by_token_decoding(model, dtype):
    cfg = model(); w = make_weights(cfg, seed=5)
    toks = settled_tokens(cfg, w, 60, 3)
    want = expected_logits(cfg, w, toks)
    check(Driver(cfg, w, dtype).run_alone(toks), want, dtype, "whole prompt")
    check(Driver(cfg, w, dtype, page=8).run_alone(toks, cuts=[1]), want, dtype, "token by token")
    check(Driver(cfg, w, dtype, page=8).run_alone(toks, cuts=[37, 1]), want, dtype, "a prompt, then token by token")


@pytest.mark.parametrize("cuts", [[2], [3, 2, 17, 2, 5], [16], [15, 17], [33, 2, 1], [64, 7], [20, 1, 21, 1]])
@pytest.mark.parametrize("model, dtype", [(everything, "float32"), (with_flash, "bfloat16")])
def test_portions(model, dtype, cuts):
    cfg = model(); w = make_weights(cfg, seed=6)
    toks = settled_tokens(cfg, w, 85, 7)
    check(Driver(cfg, w, dtype, page=16).run_alone(toks, cuts=cuts), expected_logits(cfg, w, toks), dtype, f"portions {cuts}")


def test_first_tokens():
    cfg = everything(); w = make_weights(cfg, seed=21)
    toks = settled_tokens(cfg, w, 12, 22)
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
    reqs = {n: settled_tokens(cfg, w, ln, 20 + k) for k, (n, ln) in enumerate([("a", 61), ("b", 9), ("c", 34), ("d", 47), ("e", 2)])}
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


def test_a_request_left_out_of_steps():
    cfg = everything(); w = make_weights(cfg, seed=31)
    a, b = settled_tokens(cfg, w, 30, 32), settled_tokens(cfg, w, 26, 33)
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
PROBE_LAYERS = {
    "small_heads": (dict(heads=4, kv_heads=2, dim=16, vdim=16, rot=8), 48),
    "heads_of_64": (dict(heads=4, kv_heads=2, dim=64, vdim=64, rot=32), 96),
    "heads_of_128": (dict(heads=2, kv_heads=2, dim=128, vdim=128, rot=64), 96),
    "keys_of_64_values_of_80": (dict(heads=3, kv_heads=1, dim=64, vdim=80, rot=4), 64),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", sorted(PROBE_LAYERS))
@pytest.mark.parametrize("last, back", [(599, 0), (599, 1), (599, 7), (599, 8), (599, 23), (599, 63), (599, 64), (599, 87), (599, 88), (599, 343), (599, 598), (599, 599), (512, 1), (512, 256),
                                        (512, 512), (511, 511), (128, 64), (64, 64), (63, 63), (1, 1)])
def test_one_key_stands_out(kind, last, back, dtype):
    """Token K occurs once, `back` positions before the last token Q (at position `last`), whose queries lie along K's keys while every other key lies across: that one key
    decides the last row (8-token pages; the key at the first position, at page borders, at the borders of 64-key tiles and far back).  The engine must agree with the
    restatement as a whole prompt, with the last token decoded alone, with the last token ending a short portion, and with a portion that starts at the key; a key of a
    DIFFERENT sequence in the same step (its neighbour in the pool) must not be seen."""
    shape, width = PROBE_LAYERS[kind]
    if kind == "small_heads" and dtype == "bfloat16" and back not in (0, 8, 64, 599):
        pytest.skip("the general kernel is the float32 case's")
    cfg = make_config([layer(v_mix=False, mlp=None, **shape), layer(v_mix=False, mlp=None)], vocab=31, width=width)
    Q, K, n = 0, 1, last + 1
    w = make_key_stand_out(cfg, make_weights(cfg, seed=9), Q, K, 14.0)
    toks = tokens_of(n, cfg["vocab"], 10 + back, lo=2)
    toks[-1] = Q
    if back:
        toks[n - 1 - back] = K
    want = expected_logits(cfg, w, toks)
    gone = list(toks); gone[n - 1 - back] = 2
    moved = row_errors(expected_logits(cfg, w, gone)[-1:], want[-1:]).max() if back else 0.0
    if back:
        assert moved > 4 * TOL[dtype], "the key must decide the row"
    for cuts, what in (([n], "whole"), ([max(n - 1, 1), 1], "decoded"), ([max(n - 3, 1), 3], "end of a portion"), ([n - back - 1, back + 1] if 0 < back < n - 1 else [max(n - 2, 1), 2], "a portion from the key on")):
        got = Driver(cfg, w, dtype, page=8, pages=80, max_tokens=640, max_len=640).run_alone(toks, cuts=cuts)
        check(got[-4:], want[-4:], dtype, f"{what}, {back} back of {last}")
        if back:
            assert row_errors(got[-1:], want[-1:]).max() < moved / 4, f"{what}, {back} back: the last row is off by a quarter of what the key moves it"
    other = [K] * 20
    d = Driver(cfg, w, dtype, page=8, pages=90, slots=2, max_tokens=700, max_len=640)
    d.step([("k", other)])
    out = d.step([("k", [K]), ("r", toks)])
    check(out["r"][-4:], want[-4:], dtype, f"beside a sequence of such keys, {back} back of {last}")


# ------------------------------------------------------------------------------------------------ long sequences, many rows
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("model", [everything, with_flash])
def test_long_decoding(model, dtype):
    cfg = model(); w = make_weights(cfg, seed=14)
    toks = settled_tokens(cfg, w, 200, 15)
    got = Driver(cfg, w, dtype, page=8, pages=32).run_alone(toks, cuts=[10, 1])
    check(got, expected_logits(cfg, w, toks), dtype, "190 decoded tokens")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_and_decoding_side_by_side(dtype):
    """Heads of 64 over 1100 tokens, fourteen experts of which four return their input: prompts cross many 64-key tiles, the streams take the wave-per-row form, the
    experts' rows take the padded blocks of 256 (and the blocks behind the last used one are left out); two requests then decode side by side through the split
    decode attention."""
    cfg = make_config([layer(heads=4, kv_heads=2, dim=64, vdim=64, rot=64, base=20000.0, scaling=(4.0, 1.0, 4.0, 400), mlp=moe(experts=10, top=3, ff=128, identity=4)),
                       layer(heads=4, kv_heads=2, dim=64, vdim=64, rot=32, mlp=dense(256))], vocab=71, width=256)
    w = make_weights(cfg, seed=24)
    a, b = settled_tokens(cfg, w, 1100, 25), settled_tokens(cfg, w, 900, 26)
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
@pytest.mark.parametrize("streams, width", [(2, 256), (4, 512), (1, 1024), (3, 1536), (5, 256)])
def test_streams_over_many_rows(streams, width, dtype):
    """Every form of the streams' kernel (a wave per row, a workgroup per row, the general one), and the experts' rows summed up inside it, over 1300 rows and over a few."""
    cfg = make_config([layer(heads=2, kv_heads=1, dim=64, vdim=64, mlp=moe(experts=4, top=5, ff=128, identity=3)), layer(heads=2, kv_heads=1, dim=64, vdim=64, mlp=dense(64))],
                      vocab=61, width=width, streams=streams)
    w = make_weights(cfg, seed=40 + streams)
    toks = settled_tokens(cfg, w, 1310, 41)
    want = expected_logits(cfg, w, toks)
    got = Driver(cfg, w, dtype, page=64, pages=24, max_tokens=1536, max_len=1400).run_alone(toks, cuts=[1300, 5, 1])
    check(got, want, dtype, f"{streams} streams of {width}")


def test_decode_steps_replay_a_graph():
    """Decode-sized steps are captured the second time their shape is seen and replayed from then on; every replay is compared."""
    for model, dtype in ((everything, "float32"), (with_flash, "bfloat16")):
        cfg = model(); w = make_weights(cfg, seed=16)
        toks = settled_tokens(cfg, w, 48, 17)
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
        m = []
        lg = ref.forward(cfg, w64, full[:-1], margins=m)[0]
        for k in range(len(p) - 1, len(full) - 1):
            row = lg[k]
            spread = np.sqrt(((row - row.mean()) ** 2).mean())
            assert row.max() - row[full[k + 1]] <= 3 * TOL["float32"] * spread or min(m) < 1e-4, f"request {sid}: token {k + 1} is not the greedy choice"


def test_tensors_of_other_shapes_are_refused():
    nvr = nvr_import.load()
    cfg = make_config([layer(), layer(mlp="moe")]); w = make_weights(cfg, seed=2)
    d = Driver(cfg, w, "float32")
    for name, shape in (("l0.hc1.mix", (3, 3)), ("l0.mix.q.b", (7,)), ("l0.mix.vmix", (2,)), ("l1.mlp.correction", (6,)), ("l1.mlp.e6.gate", (24, 64)), ("l0.mlp.router", (8, 64)), ("l2.norm1", (64,)),
                        ("l0.mix.sink", (4,)), ("lx.norm1", (64,)), ("l0.hc3.in", (2,))):
        with pytest.raises(nvr.NvrError):
            d.engine.model_runner.load_tensor(name, np.zeros(shape, np.float32))


# ------------------------------------------------------------------------------------------------ designs and schedules drawn at random
def random_design(seed):
    rng = np.random.default_rng(seed)
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    width = pick([48, 64, 72, 96, 104, 128, 160])
    G, vd, layers = int(rng.integers(1, 4)), pick([8, 16, 24, 48, 64]), []
    for i in range(int(rng.integers(1, 6))):
        mlp = pick([None, dense(pick([8, 24, 100, 128])), "moe", "moe"])
        if mlp == "moe":
            E, I = int(rng.integers(1, 12)), int(rng.integers(0, 6))
            mlp = moe(experts=E, top=int(rng.integers(1, E + I + 1)), ff=pick([8, 24, 40, 100]), identity=I)
        mixes = bool(rng.random() < 0.6)
        g, dv = (G, vd) if mixes else (int(rng.integers(1, 4)), pick([8, 16, 33, 64]))
        dim = pick([8, 16, 32, dv, 64, 96])
        rot = pick([None, 2, 4, dim // 2 * 2])
        layers.append(layer(heads=g * pick([1, 2, 4, 5]), kv_heads=g, dim=dim, vdim=dv, scale=float(rng.uniform(0.05, 0.4)), rot=rot, base=pick([10.0, 500.0, 100000.0]),
                            scaling=pick([None, (4.0, 1.0, 4.0, 64), (2.0, 0.5, 8.0, 1000), (8.0, 1.0, 2.0, 20)]), v_mix=mixes, mlp=mlp))
    return make_config(layers, vocab=int(rng.integers(40, 200)), width=width, streams=pick([1, 2, 2, 3, 4, 6]), eps=pick([1e-6, 1e-5, 1e-3]))


@pytest.mark.parametrize("seed", range(14))
def test_random_designs_and_schedules(seed):
    """A design drawn at random (layer order, sizes, streams, rotations, feed-forwards) runs a prompt whole, in random portions, and two requests of unequal length in
    one batch with their own portions, in both number formats."""
    cfg = random_design(100 + seed)
    w = make_weights(cfg, seed=200 + seed)
    rng = np.random.default_rng(300 + seed)
    a, b = settled_tokens(cfg, w, int(rng.integers(20, 130)), 400 + seed), settled_tokens(cfg, w, int(rng.integers(2, 60)), 500 + seed)
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
