"""Helpers of the Kiduvik tests: small configurations, random tensors by the checkpoint's names (float32 on the bfloat16 grid) and weights turned so that one key decides a
row.  The expected values come from tests/kiduvik_reference.py; the engine is driven by rugudra_util.Driver."""
import numpy as np

import kiduvik_reference as ref
from rugudra_util import bf16_round


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def latent(heads=3, dim=16, rot_dim=8, vdim=12, kv_rank=24, kv_from=None, base=700.0, scale=None, mlp="dense", mask=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale if scale is not None else 1.5 * (dim + rot_dim) ** -0.5,
         "rot": {"dims": rot_dim, "base": base}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    if mask is not None:
        m["mask"] = dict(zip(("size", "keep_first"), mask))
    return {"type": "latent_attention", "mixer": m, "mlp": dense() if mlp == "dense" else mlp}


def diff(heads=4, kv_heads=2, dim=16, vdim=32, rot=8, base=500.0, scaling=(6.0, 64, 8.0, 1.0), scale=None, mask=(30, 5), share=0.35, mlp="dense"):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else 1.5 * dim ** -0.5, "diff": share}
    if rot is not None:
        m["rot"] = {"dims": rot, "base": base}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if mask is not None:
        m["mask"] = dict(zip(("size", "keep_first"), mask))
    return {"type": "attention", "mixer": m, "mlp": dense() if mlp == "dense" else mlp}


def make_config(layers, vocab=83, width=64, positions=700, side=8, eps=1e-5):
    cfg = {"architecture": "Kiduvik", "vocab": vocab, "width": width, "max_positions": positions, "norm": {"eps": eps}, "layers": layers}
    if side:
        cfg["token_side"] = {"dim": side}
    return cfg


def make_weights(cfg, seed=0, pos_gain=0.5):
    rng = np.random.default_rng(seed)
    W, V, nL = cfg["width"], cfg["vocab"], len(cfg["layers"])
    side = (cfg.get("token_side") or {}).get("dim", 0)

    def lin(o, i, g=1.0):
        return bf16_round(rng.standard_normal((o, i)) * (g / np.sqrt(i)))

    def gains(n, mean=1.0):
        return bf16_round(mean * (1.0 + 0.2 * rng.standard_normal(n)))
    w = {"embed": bf16_round(rng.standard_normal((V, W))), "pos": bf16_round(pos_gain * rng.standard_normal((cfg["max_positions"], W))), "head": lin(V, W), "final.norm": gains(W)}
    if side:
        w["side.embed"] = bf16_round(rng.standard_normal((V, nL * side)))
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        q = p + "mix."
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        w[p + "norm1"], w[p + "norm1b"] = gains(W), gains(W, 0.7)
        if L["type"] == "latent_attention":
            r, R = m["kv_rank"], m["rot_dim"]
            w[q + "q"], w[q + "uk"], w[q + "uv"] = lin(H * (D + R), W), lin(H * D, r), lin(H * Dv, r)
            w[q + "sink"] = bf16_round(1.0 + rng.standard_normal(H))
            if m.get("kv_from") is None:
                w[q + "dkv"], w[q + "dkv.norm"] = lin(r + R, W), gains(r)
        else:
            G = m["kv_heads"]
            w[q + "q"], w[q + "k"], w[q + "v"], w[q + "g"] = lin(H * 2 * D, W), lin(G * 2 * D, W), lin(G * Dv, W), lin(H, W)
            w[q + "q.norm"], w[q + "k.norm"] = gains(D), gains(D)
            for n in ("lq1", "lk1", "lq2", "lk2"):         # (shares well below 1: two maps that see the same then leave no difference of roundings behind the norm)
                w[q + n] = bf16_round(0.5 * D ** -0.5 * rng.standard_normal(D))
        w[q + "o"] = lin(W, H * Dv)
        if L.get("mlp"):
            F = L["mlp"]["ff"]
            w[p + "norm2"], w[p + "norm2b"], w[p + "mlp.up"], w[p + "mlp.down"] = gains(W), gains(W, 0.7), lin(F, W, 1.5), lin(W, F)
        if side:
            w[p + "side.gate"], w[p + "side.proj"], w[p + "side.norm"] = lin(side, W), lin(W, side), gains(W, 0.4)
    return w


def as64(weights):
    return {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}


def expected_logits(cfg, weights, tokens):
    return ref.forward(cfg, as64(weights), list(tokens))[0]


def make_key_stand_out(cfg, w, qtok, ktok, amount=14.0, which=0, seed=77):
    """Layer 0 (a vocabulary smaller than the width, so that the layer's input tells the tokens apart, and faint positions): token qtok's queries meet token ktok's keys with a score
    `amount` above every other key's.  Differential attention: in map `which` the pair lies along one unrotated direction and every other query and key across it; the other map
    sees the keys alike.  Latent attention: the queries of qtok are turned towards the unrotated keys of ktok."""
    L, eps = cfg["layers"][0], cfg["norm"]["eps"]
    m, p = L["mixer"], "l0.mix."
    H, D = m["heads"], m["dim"]
    assert cfg["vocab"] < cfg["width"]
    out, rng = dict(w), np.random.default_rng(seed)
    out["pos"] = bf16_round(0.01 * np.asarray(w["pos"]))
    w64 = as64(out)
    h = ref.rms(w64["embed"], eps) * w64["l0.norm1"]
    pick = np.linalg.pinv(h)                                # [W, vocab]: column t is 1 on token t's input and 0 on the others'
    if L["type"] == "latent_attention":
        c = ref.rms((h[[ktok]] @ w64[p + "dkv"].T)[:, :m["kv_rank"]], eps) * w64[p + "dkv.norm"]
        k = (c @ w64[p + "uk"].T).reshape(H, D)
        wq = w64[p + "q"].reshape(H, D + m["rot_dim"], -1).copy()
        for a in range(H):
            wq[a, :D] += amount / (m["scale"] * (k[a] @ k[a])) * np.outer(k[a], pick[:, qtok])
        out[p + "q"] = bf16_round(wq.reshape(w64[p + "q"].shape))
        out[p + "sink"] = bf16_round(0.0 * w64[p + "sink"])
        return out
    R = (m.get("rot") or {"dims": 0})["dims"]
    assert D - R >= 2
    m["scale"] = amount / D                                 # (normed heads: q.k = D for equal directions)
    along, across = np.zeros(D), np.zeros(D)
    a = rng.standard_normal((2, D - R))
    along[R:], across[R:] = a[0], a[1] - a[0] * (a[0] @ a[1]) / (a[0] @ a[0])
    rest = np.ones(cfg["vocab"])

    def proj(n, tok):                                       # [n, 2, D, W]: map `which` tells tok from the others, the other map does not
        sel = rest.copy(); sel[tok] = 0.0
        tells = 4.0 * np.outer(along, pick[:, tok]) + 4.0 * np.outer(across, pick @ sel)
        alike = 4.0 * np.outer(across if tok == ktok else along, pick @ rest)
        maps = [alike, alike]; maps[which] = tells
        return bf16_round(np.concatenate([np.concatenate(maps)] * n))
    out[p + "q"], out[p + "k"] = proj(H, qtok), proj(m["kv_heads"], ktok)
    out[p + "q.norm"], out[p + "k.norm"] = np.ones(D, np.float32), np.ones(D, np.float32)
    return out
