"""A plain restatement of the Kiduvik design in numpy float64, one function per mechanism, written from the design's equations.  It shares no
code with the library: the GPU tests compare the engine against it.

Notation.  x [T, W] is the residual stream of ONE sequence, `cfg` the configuration (the dict of config.json), `wt` a dict name -> array with the
checkpoint's tensor names.  Linear weights are [out, in]; rms(v) = v / sqrt(mean(v^2) + eps).

  x       =  embed[token] + pos[position]
  layer i:   x <- x + rms(mixer(rms(x) w1)) w1b;   x <- x + rms(ff(rms(x) w2)) w2b   (no feed-forward: this step is left out)
             x <- x + rms(side_i(x, token)) ws
  logits  =  head (rms(x) wf)
"""
import numpy as np
from scipy.special import erf


def rms(v, eps):
    return v / np.sqrt((v * v).mean(axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def gelu(z):
    return 0.5 * z * (1.0 + erf(z / np.sqrt(2.0)))


def stretch(rot):
    """Rotation frequencies [dims / 2] and the factor on cosines and sines.  With a scaling: a frequency whose wavelength fits the original length `fast` times or
    more stays, one that fits it `slow` times or less is divided by `factor`, in between (by the index of the frequency) a blend."""
    dims = rot["dims"]
    f = rot["base"] ** (-2.0 * np.arange(dims // 2) / dims)
    sc = rot.get("scaling")
    if sc is None:
        return f, 1.0
    index = lambda turns: dims * np.log(sc["original"] / (2.0 * np.pi * turns)) / (2.0 * np.log(rot["base"]))      # where a wavelength fits `turns` times
    lo, hi = max(np.floor(index(sc["fast"])), 0.0), min(np.ceil(index(sc["slow"])), dims - 1.0)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f * ((1.0 - ramp) + ramp / sc["factor"]), 0.1 * np.log(sc["factor"]) + 1.0


def rotate_halves(v, pos, rot):
    """v [T, ..., D]: of the first dims numbers, number i pairs with i + dims/2; the pair is turned by pos * f_i (and scaled)."""
    if rot is None or rot["dims"] == 0:
        return v.copy()
    half = rot["dims"] // 2
    f, gain = stretch(rot)
    ang = (pos[:, None] * f).reshape(len(pos), *([1] * (v.ndim - 2)), half)
    c, s = gain * np.cos(ang), gain * np.sin(ang)
    out = v.copy()
    a, b = v[..., :half], v[..., half:2 * half]
    out[..., :half] = a * c - b * s
    out[..., half:2 * half] = b * c + a * s
    return out


def visible(pos, n, mask):
    """[T, n]: whether the query at pos[t] sees key j: causal, inside the window or among the kept first keys."""
    i, j = pos[:, None], np.arange(n)[None, :]
    see = j <= i
    if mask is not None:
        see &= (i - j < mask["size"]) | (j < (mask.get("keep_first") or 0))
    return see


def softmax(s, see, sink=None):
    """Rows of scores [T, n]; exp(sink) joins the denominator only."""
    s = np.where(see, s, -np.inf)
    top = s.max(axis=1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink)
    e = np.exp(s - top)
    return e / (e.sum(axis=1, keepdims=True) + (np.exp(sink - top) if sink is not None else 0.0))


def latent_rows(h, m, wt, p, eps, pos):
    """What latent attention caches per token: kv_rank normed numbers, then rot_dim rotated ones."""
    z = h @ wt[p + "dkv"].T
    r = m["kv_rank"]
    return np.concatenate([rms(z[:, :r], eps) * wt[p + "dkv.norm"], rotate_halves(z[:, r:], pos, {"dims": m["rot_dim"], "base": m["rot"]["base"]} if m["rot_dim"] else None)], axis=1)


def latent_attention(h, m, wt, p, pos, rows):
    """rows: the cached rows of all positions up to the last of `pos` (this layer's, or those of the layer it shares them with)."""
    T = h.shape[0]
    H, D, R, Dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ wt[p + "q"].T).reshape(T, H, D + R)
    qr = rotate_halves(q[..., D:], pos, {"dims": R, "base": m["rot"]["base"]} if R else None)
    n = rows.shape[0]
    k, v = (rows[:, :r] @ wt[p + "uk"].T).reshape(n, H, D), (rows[:, :r] @ wt[p + "uv"].T).reshape(n, H, Dv)
    see = visible(pos, n, m.get("mask"))
    o = np.empty((T, H, Dv))
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + qr[:, a] @ rows[:, r:].T) * m["scale"]
        o[:, a] = softmax(s, see, wt[p + "sink"][a]) @ v[:, a]
    return o.reshape(T, H * Dv) @ wt[p + "o"].T


def share(m, wt, p):
    """The number the second map is weighted with."""
    return np.exp((wt[p + "lq1"] * wt[p + "lk1"]).sum()) - np.exp((wt[p + "lq2"] * wt[p + "lk2"]).sum()) + m["diff"]


def differential_attention(h, m, wt, p, eps, pos, past=None):
    """past: (k [n, G, 2, D], v [n, G, Dv]) of the positions before pos[0].  Returns (result, (k, v) of all positions)."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ wt[p + "q"].T).reshape(T, H, 2, D), eps) * wt[p + "q.norm"]
    k = rms((h @ wt[p + "k"].T).reshape(T, G, 2, D), eps) * wt[p + "k.norm"]
    v = (h @ wt[p + "v"].T).reshape(T, G, Dv)
    q, k = rotate_halves(q, pos, m.get("rot")), rotate_halves(k, pos, m.get("rot"))
    if past is not None:
        k, v = np.concatenate([past[0], k]), np.concatenate([past[1], v])
    see = visible(pos, k.shape[0], m.get("mask"))
    lam, gate = share(m, wt, p), sigmoid(h @ wt[p + "g"].T)
    o = np.empty((T, H, Dv))
    for a in range(H):
        g = a // (H // G)
        a1, a2 = (softmax(q[:, a, i] @ k[:, g, i].T * m["scale"], see) @ v[:, g] for i in (0, 1))
        o[:, a] = rms(a1 - lam * a2, eps) * (1.0 - m["diff"]) * gate[:, a:a + 1]
    return o.reshape(T, H * Dv) @ wt[p + "o"].T, (k, v)


def dense_ff(h, wt, p):
    return gelu(h @ wt[p + "up"].T) @ wt[p + "down"].T


def token_input(x, tokens, wt, p, i, dim):
    e = wt["side.embed"][tokens][:, i * dim:(i + 1) * dim]
    return (gelu_tanh(x @ wt[p + "side.gate"].T) * e) @ wt[p + "side.proj"].T


def forward(cfg, wt, tokens, layer_outputs=None, pos0=0, states=None):
    """Logits [T, vocab] of one sequence's tokens at positions pos0 ..; states: the list forward returned for the tokens before (None: a new
    sequence).  Returns (logits, states)."""
    eps = cfg["norm"]["eps"]
    tokens = np.asarray(tokens)
    pos = pos0 + np.arange(len(tokens))
    x = wt["embed"][tokens] + wt["pos"][pos]
    new = []
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        h = rms(x, eps) * wt[p + "norm1"]
        old = states[i] if states is not None else None
        if L["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                rows = latent_rows(h, m, wt, p + "mix.", eps, pos)
                st = rows if old is None else np.concatenate([old, rows])
            else:
                st = new[src]
            y = latent_attention(h, m, wt, p + "mix.", pos, st)
        else:
            y, st = differential_attention(h, m, wt, p + "mix.", eps, pos, old)
        new.append(st)
        x = x + rms(y, eps) * wt[p + "norm1b"]
        if L.get("mlp") is not None:
            x = x + rms(dense_ff(rms(x, eps) * wt[p + "norm2"], wt, p + "mlp."), eps) * wt[p + "norm2b"]
        if cfg.get("token_side") is not None:
            x = x + rms(token_input(x, tokens, wt, p, i, cfg["token_side"]["dim"]), eps) * wt[p + "side.norm"]
        if layer_outputs is not None:
            layer_outputs.append(x)
    return (rms(x, eps) * wt["final.norm"]) @ wt["head"].T, new
