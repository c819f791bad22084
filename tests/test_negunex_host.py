"""Host side of the Negunex design, no GPU: the model registry's reading of a configuration and its refusals, and the plain restatement's own consistency
(keys and values carried over a cut give the rows of the whole prompt; one stream with unit weights is the plain residual sum; the stretched frequencies' branches; the
probe the GPU tests rely on does decide its row)."""
import copy

import numpy as np
import pytest

import nvr_import
import negunex_reference as ref
from negunex_util import as64, dense, expected_logits, layer, make_config, make_key_stand_out, make_weights, moe, settled_tokens

nvr = nvr_import.load()


def small():
    return make_config([layer(), layer(mlp="moe"), layer(v_mix=False, mlp=None), layer(rot=8, mlp=moe(experts=3, top=1, ff=8, identity=None))], vocab=53, width=48)


def test_registry_reads_the_design():
    assert "Negunex" in nvr.registered_architectures()
    s = nvr.ModelSpec(small())
    assert (s.architecture, s.family, s.vocab_size, s.num_layer_runs) == ("Negunex", 1, 53, 4)
    cfg = small()
    cfg["layers"][0]["mixer"]["rot"] = None; cfg["layers"][1]["mixer"]["rot"]["scaling"] = None; cfg["layers"][1]["mixer"].pop("v_mix"); cfg["layers"][2].pop("mlp")
    cfg["layers"][3]["mlp"]["router"].update(identity=5, top=8)
    assert nvr.ModelSpec(cfg).num_layer_runs == 4


@pytest.mark.parametrize("breakage, message", [
    (lambda c: c.pop("width"), "'width' is missing"),
    (lambda c: c.pop("streams"), "'streams' is missing"),
    (lambda c: c.update(streams=0), "streams must be positive"),
    (lambda c: c.update(streams=1.5), "'streams' is not an integer"),
    (lambda c: c.pop("norm"), "'norm' is missing"),
    (lambda c: c["norm"].pop("eps"), "'norm.eps' is missing"),
    (lambda c: c.update(layers=[]), "'layers' is not a list"),
    (lambda c: c["layers"][0].update(type="retention"), "layer type 'retention'"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "mixer.scale' is missing"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "4 heads over 3 key/value heads"),
    (lambda c: c["layers"][0]["mixer"].update(v_mix="yes"), "v_mix' is not true or false"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=8), "mixes values of other sizes than layer 0's"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "an even rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "rot.dims <= dim"),
    (lambda c: c["layers"][0]["mixer"]["rot"].pop("base"), "rot.base' is missing"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("original"), "scaling.original' is missing"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=5.0), "high at least low"),
    (lambda c: c["layers"][0]["mlp"].update(kind="poly"), "mlp.kind' (dense or moe)"),
    (lambda c: c["layers"][0]["mlp"].update(ff=0), "mlp.ff' must be positive"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "1 <= top <= experts + identity"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(identity=-1), "identity >= 0"),
    (lambda c: c["layers"][1]["mlp"]["router"].pop("experts"), "router.experts' is missing"),
])
def test_registry_refuses(breakage, message):
    cfg = small()
    breakage(cfg)
    with pytest.raises(nvr.NvrError) as e:
        nvr.ModelSpec(cfg)
    assert message in str(e.value)


def test_cached_keys_and_values_give_the_rows_of_the_whole_prompt():
    cfg = small(); w = as64(make_weights(cfg, seed=3))
    toks = np.random.default_rng(4).integers(0, cfg["vocab"], 31).tolist()
    whole, _ = ref.forward(cfg, w, toks)
    for cuts in ([1] * 31, [2, 9, 20], [30, 1]):
        at, states, rows = 0, None, []
        for c in cuts:
            lg, states = ref.forward(cfg, w, toks[at:at + c], pos0=at, states=states)
            rows.append(lg); at += c
        assert np.abs(np.concatenate(rows) - whole).max() < 1e-9


def test_one_stream_with_unit_weights_is_the_residual_sum():
    cfg = make_config([layer(), layer(v_mix=False)], streams=1); w = as64(make_weights(cfg, seed=5))
    for i in (0, 1):
        for q in "12":
            w["l%d.hc%s.in" % (i, q)], w["l%d.hc%s.out" % (i, q)], w["l%d.hc%s.mix" % (i, q)] = np.ones(1), np.ones(1), np.ones((1, 1))
    toks = np.random.default_rng(6).integers(0, cfg["vocab"], 9)
    eps, x = cfg["norm"]["eps"], w["embed"][toks]
    for i in (0, 1):
        p = "l%d." % i
        x = x + ref.attention(ref.layer_norm(x, w[p + "norm1"], eps), cfg["layers"][i]["mixer"], w, p + "mix.", eps)[0]
        x = x + ref.dense_ff(ref.layer_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
    want = ref.layer_norm(x, w["final.norm"], eps) @ w["head"].T
    assert np.abs(ref.forward(cfg, w, toks)[0] - want).max() < 1e-9


def test_stretched_frequencies():
    rot = {"dims": 16, "base": 500.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}}
    f, plain = ref.frequencies(rot), ref.frequencies({"dims": 16, "base": 500.0})
    wave = 2 * np.pi / plain
    assert f[0] == plain[0] and abs(f[-1] * 4.0 - plain[-1]) < 1e-15                 # short wavelengths stay, long ones are stretched
    between = (wave > 16) & (wave < 64)
    assert between.any() and np.all(f[between] < plain[between]) and np.all(f[between] > plain[between] / 4.0)
    assert np.all(np.diff(f) < 0)


def test_identity_experts_return_their_input():
    cfg = make_config([layer(mlp=moe(experts=2, top=3, ff=8, identity=1))]); w = as64(make_weights(cfg, seed=7))
    h = np.random.default_rng(8).standard_normal((5, cfg["width"]))
    for e in (0, 1):
        w["l0.mlp.e%d.down" % e] *= 0.0                     # (every router output is chosen: only the identity expert's share is left)
    chosen, s = ref.route(h, w, "l0.mlp.", 3)
    share = np.take_along_axis(s, np.argsort(chosen, axis=1)[:, 2:3], axis=1)
    assert np.abs(ref.expert_ff(h, cfg["layers"][0]["mlp"], w, "l0.mlp.") - share * h).max() < 1e-12
    assert np.abs(s.sum(axis=1) - 1.0).max() < 1e-12


def test_the_correction_moves_the_choice_and_not_the_weights():
    cfg = make_config([layer(mlp=moe(experts=4, top=1, ff=8, identity=2))]); w = as64(make_weights(cfg, seed=9))
    h = np.random.default_rng(10).standard_normal((7, cfg["width"]))
    w["l0.mlp.correction"] = np.array([0.0, 0.0, 0.0, 0.0, 0.0, 5.0])
    chosen, s = ref.route(h, w, "l0.mlp.", 2)
    assert np.all(chosen[:, 0] == 5)
    z = h @ w["l0.mlp.router"].T
    p = np.exp(z) / np.exp(z).sum(axis=1, keepdims=True)
    c = np.take_along_axis(p, chosen, axis=1)
    assert np.abs(s - c / c.sum(axis=1, keepdims=True)).max() < 1e-12


def test_the_probe_key_decides_its_row():
    cfg = make_config([layer(dim=16, vdim=16, rot=8, v_mix=False, mlp=None)], vocab=31, width=48)
    w = make_key_stand_out(cfg, make_weights(cfg, seed=9), 0, 1, 14.0)
    toks = np.random.default_rng(11).integers(2, 31, 300).tolist()
    toks[-1], toks[57] = 0, 1
    gone = list(toks); gone[57] = 2
    a, b = expected_logits(cfg, w, toks)[-1], expected_logits(cfg, w, gone)[-1]
    assert np.sqrt(((a - b) ** 2).mean()) > 0.2 * a.std()


def test_settled_tokens_have_no_close_calls():
    cfg = small(); w = make_weights(cfg, seed=12)
    m = []
    ref.forward(cfg, as64(w), settled_tokens(cfg, w, 60, 13), margins=m)
    assert len(m) == 120 and min(m) > 0.01


def test_configurations_are_not_shared_between_tests():
    a, b = small(), small()
    assert a == b and a is not b and copy.deepcopy(a) == b and dense() == {"kind": "dense", "ff": 48}
