"""Host side of the Kiduvik design, no GPU: the model registry's reading of a configuration and its refusals, and the plain restatement's own consistency (cached rows, keys and
values carried over a cut give the rows of the whole prompt; the absorbed form of latent attention; the stretched frequencies' branches; sinks, windows and kept keys; the probe
the GPU tests rely on does decide its row)."""
import copy

import numpy as np
import pytest

import nvr_import
import kiduvik_reference as ref
from kiduvik_util import as64, dense, diff, expected_logits, latent, make_config, make_key_stand_out, make_weights
from rugudra_util import row_errors

nvr = nvr_import.load()


def small():
    return make_config([latent(), diff(mask=(7, 3)), latent(kv_from=0, heads=2, dim=8, vdim=20, mlp=None), diff(heads=3, kv_heads=1, dim=6, vdim=10, rot=4, scaling=None, mask=(4, 0))], vocab=53, width=48)


def test_registry_reads_the_design():
    assert "Kiduvik" in nvr.registered_architectures()
    s = nvr.ModelSpec(small())
    assert (s.architecture, s.family, s.vocab_size, s.num_layer_runs) == ("Kiduvik", 1, 53, 4)
    cfg = small()
    cfg["token_side"] = None
    cfg["layers"][0].pop("mlp"); cfg["layers"][1]["mixer"].update(rot=None, mask=None); cfg["layers"][3]["mixer"]["mask"].pop("keep_first"); cfg["layers"][3]["mixer"]["rot"]["scaling"] = None
    cfg["layers"][0]["mixer"]["kv_from"] = None
    assert nvr.ModelSpec(cfg).num_layer_runs == 4


@pytest.mark.parametrize("breakage, message", [
    (lambda c: c.pop("width"), "'width' is missing"),
    (lambda c: c.pop("max_positions"), "'max_positions' is missing"),
    (lambda c: c.update(max_positions=0), "max_positions must be positive"),
    (lambda c: c.update(vocab=3.5), "'vocab' is not an integer"),
    (lambda c: c["norm"].pop("eps"), "'norm.eps' is missing"),
    (lambda c: c["token_side"].pop("dim"), "'token_side.dim' is missing"),
    (lambda c: c.update(layers=[]), "'layers' is not a list"),
    (lambda c: c["layers"][0].update(type="gla"), "layer type 'gla'"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "mixer.scale' is missing"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "mixer.kv_rank' is missing"),
    (lambda c: c["layers"][0]["mixer"].update(kv_rank=0), "positive kv_rank"),
    (lambda c: c["layers"][0]["mixer"].update(rot_dim=6), "rot.dims = rot_dim"),
    (lambda c: c["layers"][0]["mixer"].update(rot_dim=7, rot={"dims": 7, "base": 10.0}), "an even number"),
    (lambda c: c["layers"][0]["mixer"]["rot"].pop("base"), "rot.base' is missing"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "must name an earlier layer"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "a latent of its own"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=32), "the same kv_rank and rot_dim"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "4 heads over 3 key/value heads"),
    (lambda c: c["layers"][1]["mixer"].pop("diff"), "mixer.diff' is missing"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=18), "rot.dims <= dim"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("fast"), "scaling.fast' is missing"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0), "must be positive"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "a positive size"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1), "keep_first >= 0"),
    (lambda c: c["layers"][1]["mlp"].update(kind="moe"), "mlp.kind' (dense)"),
    (lambda c: c["layers"][1]["mlp"].update(ff=0), "mlp.ff' must be positive"),
])
def test_registry_refuses(breakage, message):
    cfg = small()
    breakage(cfg)
    with pytest.raises(nvr.NvrError) as e:
        nvr.ModelSpec(cfg)
    assert message in str(e.value)


def test_what_is_cached_gives_the_rows_of_the_whole_prompt():
    cfg = small(); w = as64(make_weights(cfg, seed=3))
    toks = np.random.default_rng(4).integers(0, cfg["vocab"], 31).tolist()
    whole, _ = ref.forward(cfg, w, toks)
    for cuts in ([1] * 31, [2, 9, 20], [30, 1]):
        at, states, rows = 0, None, []
        for c in cuts:
            lg, states = ref.forward(cfg, w, toks[at:at + c], pos0=at, states=states)
            rows.append(lg); at += c
        assert np.abs(np.concatenate(rows) - whole).max() < 1e-9


def test_absorbed_latent_attention():
    """The key expansion folded into the queries, the value expansion behind the sum: the same output from the cached rows alone."""
    cfg = small(); w = as64(make_weights(cfg, seed=5)); m = cfg["layers"][0]["mixer"]
    eps, p, pos = cfg["norm"]["eps"], "l0.mix.", np.arange(11)
    h = np.random.default_rng(6).standard_normal((11, cfg["width"]))
    rows = ref.latent_rows(h, m, w, p, eps, pos)
    H, D, R, Dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w[p + "q"].T).reshape(11, H, D + R)
    qr = ref.rotate_halves(q[..., D:], pos, m["rot"])
    uk, uv = w[p + "uk"].reshape(H, D, r), w[p + "uv"].reshape(H, Dv, r)
    o = np.empty((11, H, Dv))
    for a in range(H):
        qa = np.concatenate([q[:, a, :D] @ uk[a], qr[:, a]], axis=1)
        o[:, a] = ref.softmax(qa @ rows.T * m["scale"], ref.visible(pos, 11, None), w[p + "sink"][a]) @ rows[:, :r] @ uv[a].T
    assert np.abs(o.reshape(11, -1) @ w[p + "o"].T - ref.latent_attention(h, m, w, p, pos, rows)).max() < 1e-12


def test_a_shared_latent_follows_its_source():
    cfg = small(); w = as64(make_weights(cfg, seed=7))
    toks = np.random.default_rng(8).integers(0, cfg["vocab"], 12)
    full, _ = ref.forward(cfg, w, toks)
    w2 = dict(w); w2["l0.mix.uk"], w2["l0.mix.uv"] = 0 * w["l0.mix.uk"], 0 * w["l0.mix.uv"]      # (layer 2 expands the rows with matrices of its own)
    a = []; ref.forward(cfg, w, toks, a)
    h = ref.rms(w["embed"][toks] + w["pos"][:12], cfg["norm"]["eps"]) * w["l0.norm1"]
    rows = ref.latent_rows(h, cfg["layers"][0]["mixer"], w, "l0.mix.", cfg["norm"]["eps"], np.arange(12))
    _, states = ref.forward(cfg, w, toks)
    assert states[2] is states[0] and np.abs(states[0] - rows).max() < 1e-12
    assert row_errors(ref.forward(cfg, w2, toks)[0], full).max() > 0.05


def test_stretched_frequencies():
    rot = {"dims": 16, "base": 500.0, "scaling": {"factor": 6.0, "original": 64, "fast": 8.0, "slow": 1.0}}
    f, gain = ref.stretch(rot)
    plain, one = ref.stretch({"dims": 16, "base": 500.0})
    assert one == 1.0 and abs(gain - (0.1 * np.log(6.0) + 1.0)) < 1e-15
    turns = 64 * plain / (2 * np.pi)                       # how often a wavelength fits the original length
    assert np.allclose(f[turns >= 8.0], plain[turns >= 8.0]) and f[0] == plain[0]
    assert np.allclose(f[-1] * 6.0, plain[-1])
    between = (f < plain * (1 - 1e-12)) & (f > plain / 6.0 * (1 + 1e-12))
    assert between.any()
    # both ends clipped: everything stays (fast and slow below any wavelength's turns), everything is divided (far above)
    rot["scaling"].update(fast=1e-9, slow=1e-12)
    assert np.allclose(ref.stretch(rot)[0][:-1], plain[:-1])
    rot["scaling"].update(fast=1e9, slow=1e8)
    assert np.allclose(ref.stretch(rot)[0][1:], plain[1:] / 6.0)


def test_window_and_kept_keys():
    see = ref.visible(np.arange(10), 10, {"size": 3, "keep_first": 2})
    assert see[9].tolist() == [True, True, False, False, False, False, False, True, True, True]
    assert see[2].tolist() == [True] * 3 + [False] * 7 and see[4].tolist() == [True, True, True, True, True] + [False] * 5
    assert see[5].tolist() == [True, True, False, True, True, True] + [False] * 4
    assert np.array_equal(ref.visible(np.arange(4), 4, {"size": 9}), np.tril(np.ones((4, 4), bool)))


def test_a_sink_only_dilutes():
    s, see = np.random.default_rng(9).standard_normal((5, 5)), np.tril(np.ones((5, 5), bool))
    a, b = ref.softmax(s, see), ref.softmax(s, see, 1.3)
    z = np.where(see, np.exp(s), 0).sum(axis=1, keepdims=True)
    assert np.abs(b - a * z / (z + np.exp(1.3))).max() < 1e-12


def test_two_equal_maps_cancel():
    """With the same queries and keys in both maps the difference is (1 - lambda) times one attention: only its sign and direction are left behind the norm."""
    cfg = small(); w = as64(make_weights(cfg, seed=10)); m = cfg["layers"][1]["mixer"]
    p, eps = "l1.mix.", 0.0
    for n, heads in (("q", m["heads"]), ("k", m["kv_heads"])):
        v = w[p + n].reshape(heads, 2, m["dim"], -1)
        w[p + n] = np.repeat(v[:, :1], 2, axis=1).reshape(w[p + n].shape)
    h = np.random.default_rng(11).standard_normal((9, cfg["width"]))
    a, _ = ref.differential_attention(h, m, w, p, eps, np.arange(9))
    w2 = dict(w); w2[p + "lq1"] = 0 * w[p + "lq1"]; w2[p + "lq2"] = 0 * w[p + "lq2"]
    b, _ = ref.differential_attention(h, m, w2, p, eps, np.arange(9))
    sign = np.sign((1 - ref.share(m, w, p)) * (1 - ref.share(m, w2, p)))
    assert np.abs(a - sign * b).max() < 1e-9


@pytest.mark.parametrize("layer0", [diff(mask=(100, 9)), latent(heads=2)])
@pytest.mark.parametrize("which", [0, 1])
def test_the_probe_key_decides_its_row(layer0, which):
    layer0 = copy.deepcopy(layer0); layer0["mlp"] = None
    cfg = make_config([layer0], vocab=31, width=48)
    w = make_key_stand_out(cfg, make_weights(cfg, seed=9), 0, 1, which=which)
    for at in (57, 3, 119):
        toks = np.random.default_rng(11).integers(2, 31, 120).tolist()
        toks[-1] = 0
        if at < 119:
            toks[at] = 1
        gone = list(toks); gone[at] = 2
        a, b = expected_logits(cfg, w, toks)[-1:], expected_logits(cfg, w, gone)[-1:]
        assert row_errors(b, a).max() > 0.2
    assert dense() == {"kind": "dense", "ff": 40}
