"""A plain restatement of the Negunex design in numpy float64, one function per mechanism, written from the design's equations.  It shares no
code with the library: the GPU tests compare the engine against it.

Notation.  X [S, T, W] are the S parallel residual streams of ONE sequence, `cfg` the configuration (the dict of config.json), `wt` a dict
name -> array with the checkpoint's tensor names.  Linear weights are [out, in].

  X_s      =  embed[token]   for every stream s
  sublayer:   u = sum_s a_s X_s;   y = f(LN(u));   X_t <- sum_s M_st X_s + b_t y     (a = hc.in, M = hc.mix [from, to], b = hc.out)
              with f the mixer (hc1, norm1), then the feed-forward (hc2, norm2) where the layer has one
  logits   =  head LN_final(sum_s X_s)
"""
import numpy as np


def layer_norm(v, w, eps):
    """(v - mean) / sqrt(variance + eps) * w; no bias."""
    d = v - v.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w


def unit_rms(v, eps):
    return v / np.sqrt((v * v).mean(axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def frequencies(rot):
    """base^(-2i/dims), the long wavelengths stretched by `factor` and the ones between original/high and original/low blended."""
    dims = rot["dims"]
    f = rot["base"] ** (-2.0 * np.arange(dims // 2) / dims)
    sc = rot.get("scaling")
    if sc is None:
        return f
    out = np.empty_like(f)
    for i, fi in enumerate(f):
        wave = 2.0 * np.pi / fi
        if wave < sc["original"] / sc["high"]:
            out[i] = fi
        elif wave > sc["original"] / sc["low"]:
            out[i] = fi / sc["factor"]
        else:
            s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
            out[i] = (1.0 - s) * fi / sc["factor"] + s * fi
    return out


def rotate_pairs(v, pos, rot):
    """v [T, heads, D]: the numbers (2i, 2i+1) of the first rot.dims are turned by pos * f_i."""
    if rot is None or rot["dims"] == 0:
        return v.copy()
    dims = rot["dims"]
    ang = pos[:, None] * frequencies(rot)[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = v.copy()
    a, b = v[..., 0:dims:2], v[..., 1:dims:2]
    out[..., 0:dims:2] = a * c - b * s
    out[..., 1:dims:2] = b * c + a * s
    return out


def attention(h, m, wt, p, eps, pos0=0, past=None, v_first=None):
    """Grouped heads; q, k, v with biases; q and k rotated, then divided by their root mean square over the head; causal softmax of
    (q.k) scale; heads times sigmoid(W_g h); W_o.  v_first (rows of this call's tokens, or None: this layer does not mix): the values become
    (1 - lambda) v + lambda v_first.  past: (k, v) of the positions before pos0 or None.
    Returns (result, (k, v) of all positions, this call's values before the mixing)."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = pos0 + np.arange(T)
    q = (h @ wt[p + "q"].T + wt[p + "q.b"]).reshape(T, H, D)
    k = (h @ wt[p + "k"].T + wt[p + "k.b"]).reshape(T, G, D)
    v = (h @ wt[p + "v"].T + wt[p + "v.b"]).reshape(T, G, Dv)
    own = v
    q = unit_rms(rotate_pairs(q, pos, m.get("rot")), eps)
    k = unit_rms(rotate_pairs(k, pos, m.get("rot")), eps)
    if v_first is not None:
        lam = float(wt[p + "vmix"])
        v = (1.0 - lam) * v + lam * v_first
    if past is not None:
        k, v = np.concatenate([past[0], k]), np.concatenate([past[1], v])
    o = np.zeros((T, H, Dv))
    for t in range(T):
        n = pos0 + t + 1
        for a in range(H):
            g = a // (H // G)
            s = k[:n, g] @ q[t, a] * m["scale"]
            e = np.exp(s - s.max())
            o[t, a] = (e / e.sum()) @ v[:n, g]
    o = o.reshape(T, H * Dv) * sigmoid(h @ wt[p + "g"].T)
    return o @ wt[p + "o"].T, (k, v), own


def dense_ff(h, wt, p):
    return (gelu_tanh(h @ wt[p + "gate"].T) * (h @ wt[p + "up"].T)) @ wt[p + "down"].T


def expert(h, wt, p):
    return (silu(h @ wt[p + "gate"].T) * (h @ wt[p + "up"].T)) @ wt[p + "down"].T


def route(h, wt, p, top, margins=None):
    """Scores s = softmax over all router rows; chosen by s + correction; weights s / (sum of the chosen s + 1e-20).  margins (a list) collects, per
    token, the gap between the last chosen and the first rejected choice score."""
    z = h @ wt[p + "router"].T
    s = np.exp(z - z.max(axis=-1, keepdims=True))
    s /= s.sum(axis=-1, keepdims=True)
    c = s + wt[p + "correction"]
    if margins is not None and top < c.shape[1]:
        cs = np.sort(c, axis=-1)[:, ::-1]
        margins.extend((cs[:, top - 1] - cs[:, top]).tolist())
    chosen = np.argsort(-c, axis=-1, kind="stable")[:, :top]
    w = np.take_along_axis(s, chosen, axis=-1)
    return chosen, w / (w.sum(axis=-1, keepdims=True) + 1e-20)


def expert_ff(h, f, wt, p, margins=None):
    """Router outputs `experts` and up are identity experts: their output is h itself."""
    chosen, w = route(h, wt, p, f["router"]["top"], margins)
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for c, wc in zip(chosen[t], w[t]):
            y[t] += wc * (expert(h[t:t + 1], wt, p + "e%d." % c)[0] if c < f["router"]["experts"] else h[t])
    return y


def read_streams(X, wt, p):
    return np.einsum("s,stw->tw", wt[p + "in"], X)


def write_streams(X, y, wt, p):
    return np.einsum("sq,stw->qtw", wt[p + "mix"], X) + wt[p + "out"][:, None, None] * y[None]


def forward(cfg, wt, tokens, layer_outputs=None, pos0=0, states=None, margins=None):
    """Logits [T, vocab] of one sequence's tokens at positions pos0 ..; states: the list forward returned for the tokens before (None: a new
    sequence).  Returns (logits, states)."""
    eps = cfg["norm"]["eps"]
    e = wt["embed"][np.asarray(tokens)].astype(np.float64)
    X = np.stack([e] * cfg["streams"])
    v_first, new_states = None, []
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        h = layer_norm(read_streams(X, wt, p + "hc1."), wt[p + "norm1"], eps)
        mixes = bool(m.get("v_mix"))
        y, st, own = attention(h, m, wt, p + "mix.", eps, pos0, states[i] if states is not None else None, v_first if mixes else None)
        if mixes and v_first is None:
            v_first = own
        new_states.append(st)
        X = write_streams(X, y, wt, p + "hc1.")
        f = L.get("mlp")
        if f is not None:
            h = layer_norm(read_streams(X, wt, p + "hc2."), wt[p + "norm2"], eps)
            y = dense_ff(h, wt, p + "mlp.") if f["kind"] == "dense" else expert_ff(h, f, wt, p + "mlp.", margins)
            X = write_streams(X, y, wt, p + "hc2.")
        if layer_outputs is not None:
            layer_outputs.append(X.sum(axis=0))
    return layer_norm(X.sum(axis=0), wt["final.norm"], eps) @ wt["head"].T, new_states
