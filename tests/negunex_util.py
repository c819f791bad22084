"""Helpers of the Negunex tests: small configurations, random tensors by the checkpoint's names (float32 on the bfloat16 grid), token sequences whose
router decisions are no close calls, and weights turned so that one key decides a row.  The expected values come from tests/negunex_reference.py."""
import numpy as np

import negunex_reference as ref
from rugudra_util import bf16_round


def dense(ff=48):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24, identity=2):
    r = {"experts": experts, "top": top}
    if identity is not None:
        r["identity"] = identity
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def layer(heads=4, kv_heads=2, dim=16, vdim=24, scale=None, rot="default", base=500.0, scaling=(4.0, 1.0, 4.0, 64), v_mix=True, mlp="dense"):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else 1.5 * dim ** -0.5, "v_mix": v_mix}
    if rot == "default":
        rot = min(16, dim // 2 * 2)
    if rot is not None:
        m["rot"] = {"dims": rot, "base": base}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "attention", "mixer": m, "mlp": dense() if mlp == "dense" else moe() if mlp == "moe" else mlp}


def make_config(layers, vocab=83, width=64, streams=2, eps=1e-5):
    return {"architecture": "Negunex", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "layers": layers}


ROUTED = 8      # the routers read the first channels only, where the embeddings are large: see make_weights


def make_weights(cfg, seed=0):
    """Random tensors.  The first ROUTED channels of the embeddings are large, everything that writes into the streams writes little into them, and the routers read only
    these channels: a router's decision is then (nearly) a property of the token, 16-bit noise hardly reaches it, and tokens can be drawn so that no decision is a
    close call (settled_tokens)."""
    rng = np.random.default_rng(seed)
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    quiet = np.ones(W); quiet[:ROUTED] = 0.02

    def lin(o, i, g=1.0):
        return bf16_round(rng.standard_normal((o, i)) * (g / np.sqrt(i)))

    def out(i):                                             # a projection into the streams
        return bf16_round(rng.standard_normal((W, i)) * (1.0 / np.sqrt(i)) * quiet[:, None])

    def gains(n, spread=0.2):
        return bf16_round(1.0 + spread * rng.standard_normal(n))
    emb = rng.standard_normal((V, W)); emb[:, :ROUTED] *= 4.0
    w = {"embed": bf16_round(emb), "head": lin(V, W), "final.norm": gains(W)}
    for i, L in enumerate(cfg["layers"]):
        p, m, mlp = "l%d." % i, L["mixer"], L.get("mlp")
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for q in (1, 2)[:2 if mlp else 1]:
            w[p + "norm%d" % q] = gains(W)
            w[p + "hc%d.in" % q] = bf16_round((1.0 + 0.4 * rng.standard_normal(S)) / S)
            w[p + "hc%d.out" % q] = bf16_round(1.0 + 0.4 * rng.standard_normal(S))
            w[p + "hc%d.mix" % q] = bf16_round(np.eye(S) + 0.2 * rng.standard_normal((S, S)) / np.sqrt(S))
        w[p + "mix.q"], w[p + "mix.k"], w[p + "mix.v"], w[p + "mix.g"], w[p + "mix.o"] = lin(H * D, W), lin(G * D, W), lin(G * Dv, W), lin(H * Dv, W), out(H * Dv)
        w[p + "mix.q.b"], w[p + "mix.k.b"], w[p + "mix.v.b"] = (bf16_round(0.5 * rng.standard_normal(n)) for n in (H * D, G * D, G * Dv))
        w[p + "mix.vmix"] = bf16_round(np.float32(rng.uniform(0.2, 0.7)))
        if mlp and mlp["kind"] == "dense":
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = lin(mlp["ff"], W, 2.0), lin(mlp["ff"], W, 2.0), out(mlp["ff"])
        elif mlp:
            E, n = mlp["router"]["experts"], mlp["router"]["experts"] + (mlp["router"].get("identity") or 0)
            rt = np.zeros((n, W)); rt[:, :ROUTED] = rng.standard_normal((n, ROUTED)) * 0.4
            w[p + "mlp.router"], w[p + "mlp.correction"] = bf16_round(rt), bf16_round(0.2 * rng.standard_normal(n))
            fe = mlp["expert"]["ff"]
            for e in range(E):
                w[p + "mlp.e%d.gate" % e], w[p + "mlp.e%d.up" % e], w[p + "mlp.e%d.down" % e] = lin(fe, W, 2.0), lin(fe, W, 2.0), out(fe)
    return w


def as64(weights):
    return {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}


def expected_logits(cfg, weights, tokens):
    return ref.forward(cfg, as64(weights), list(tokens))[0]


def settled_tokens(cfg, w, n, seed, gap=0.01, lo=0):
    """n random tokens for which every router decision of the restatement has a gap of at least `gap` between the last chosen and the first rejected choice score (a
    bfloat16 engine may otherwise choose another expert than the float64 restatement: no comparison should rest on such a call)."""
    V, w64 = cfg["vocab"], as64(w)
    good = list(range(lo, V))
    for k in range(60):
        toks, m = [good[j] for j in np.random.default_rng(seed + 1000 * k).integers(0, len(good), n)], []
        ref.forward(cfg, w64, toks, margins=m)
        if not m or min(m) > gap:
            return toks
        per = np.asarray(m).reshape(-1, n).min(axis=0)      # drop the tokens whose own decisions are close and draw again among the rest
        bad = {t for t, g in zip(toks, per) if g <= gap}
        if len(good) - len(bad) >= max(4, V // 8):
            good = [t for t in good if t not in bad]
    raise AssertionError("no token sequence with settled router decisions")


def make_key_stand_out(cfg, w, qtok, ktok, amount, seed=77):
    """Layer 0 (a vocabulary no larger than the width, so that the layer's input tells the tokens apart): the query and key projections are replaced so that token
    qtok's queries and token ktok's keys lie along one unrotated direction per key/value head while every other token's queries and keys lie across it — behind the unit
    norms the score of that pair is the largest there is, `amount` above everything else.  Values are scaled up so that the row follows the key."""
    m, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    H, G, D, R = m["heads"], m["kv_heads"], m["dim"], (m.get("rot") or {"dims": 0})["dims"]
    assert cfg["vocab"] + 1 <= cfg["width"] and D - R >= 2
    m["scale"] = amount / D                                  # (unit norms make q.k = D for equal directions)
    out, w64 = dict(w), as64(w)
    u = w64["embed"] * w64["l0.hc1.in"].sum()
    h = ref.layer_norm(u, w64["l0.norm1"], eps)
    pick = np.linalg.pinv(h)                                # [W, vocab]: column t is 1 on token t's input and 0 on the others'
    rng = np.random.default_rng(seed)
    away = rng.standard_normal((G, 2, D)); away[:, :, :R] = 0.0
    along, across = away[:, 0], away[:, 1]
    across = across - along * (along * across).sum(-1, keepdims=True) / (along * along).sum(-1, keepdims=True)
    rest = np.ones(cfg["vocab"])

    def proj(n, tok):                                       # rows: `along` on tok's input, `across` on the others'
        sel = rest.copy(); sel[tok] = 0.0
        a = np.concatenate([along[hd // (n // G)] for hd in range(n)]); c = np.concatenate([across[hd // (n // G)] for hd in range(n)])
        return bf16_round(4.0 * np.outer(a, pick[:, tok]) + 4.0 * np.outer(c, pick @ sel))
    out["l0.mix.q"], out["l0.mix.k"] = proj(H, qtok), proj(G, ktok)
    out["l0.mix.q.b"], out["l0.mix.k.b"] = np.zeros_like(w["l0.mix.q.b"]), np.zeros_like(w["l0.mix.k.b"])
    return out
