"""Plain, slow numpy statement (float64) of the layered decoder: a stack whose layers each name a mixer
(attention with rotary positions and value mixing, or a selective scan) and a feed-forward block (none, dense or
mixture of experts), with a norm before and after each.  TEST INFRASTRUCTURE: one function a mechanism, loops
where a loop says it best, no code shared with the library.

Tensors are a dict name -> array; the configuration is the parsed config.json.
"""
from __future__ import annotations

import math

import numpy as np

f64 = np.float64


def layer_norm(x, w, b, eps):
    mu = x.mean(axis=-1, keepdims=True)
    var = ((x - mu) ** 2).mean(axis=-1, keepdims=True)
    return (x - mu) / np.sqrt(var + eps) * w + b


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def clamped_swiglu(g, u, limit):
    """min(g, L) sigmoid(1.702 min(g, L)) (clip(u, -L, L) + 1)"""
    g, u = np.minimum(g, limit), np.clip(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


# ---- rotary positions ---------------------------------------------------------------------------

def rotary_frequencies(rot):
    """(frequency of each pair, factor on cos and sin)."""
    d, base = rot["dims"], float(rot["base"])
    f = np.array([base ** (-2.0 * i / d) for i in range(d // 2)], f64)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor = float(sc["factor"])

    def turns(t):  # the dimension whose pair turns t times over the original context
        return d * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(turns(sc["fast"])), 0)
    hi = min(math.ceil(turns(sc["slow"])), d - 1)
    ramp = np.array([min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(d // 2)], f64)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_interleaved(v, pos0, rot):
    """v [T, heads, dim]: pairs (2i, 2i + 1) of the first rot.dims dimensions turn by (pos0 + t) f_i."""
    freq, mag = rotary_frequencies(rot)
    out = v.copy()
    for t in range(v.shape[0]):
        a = (pos0 + t) * freq
        c, s = mag * np.cos(a), mag * np.sin(a)
        x, y = v[t, :, 0:rot["dims"]:2], v[t, :, 1:rot["dims"]:2]
        out[t, :, 0:rot["dims"]:2] = x * c - y * s
        out[t, :, 1:rot["dims"]:2] = y * c + x * s
    return out


# ---- mixers ---------------------------------------------------------------------------------------

def attend(q, K, V, pos0, scale):
    """q [T, H, d] at positions pos0 + t over K [n, G, d], V [n, G, dv]: causal softmax attention."""
    T, H, _ = q.shape
    G = K.shape[1]
    out = np.zeros((T, H, V.shape[2]), f64)
    for t in range(T):
        n = pos0 + t + 1
        for h in range(H):
            g = h // (H // G)
            s = K[:n, g] @ q[t, h] * scale
            e = np.exp(s - s.max())
            out[t, h] = (e / e.sum()) @ V[:n, g]
    return out


def attention(h, w, m, cache, pos0, v_first):
    """Mixer `attention`; cache {"k", "v"} is appended to.  v_first: the values of the first value-mixing layer for
    these tokens, or None in that layer and where the layer does not mix.  Returns (output, the layer's own v)."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_interleaved((h @ w["q"].T).reshape(T, H, d), pos0, m["rot"])
    k = rotate_interleaved((h @ w["k"].T).reshape(T, G, d), pos0, m["rot"])
    v = (h @ w["v"].T).reshape(T, G, dv)
    own = v
    if v_first is not None:
        lam = float(w["vmix"])
        v = (1.0 - lam) * v + lam * v_first.reshape(v.shape)
    cache["k"] = np.concatenate([cache.get("k", np.zeros((0, G, d))), k])
    cache["v"] = np.concatenate([cache.get("v", np.zeros((0, G, dv))), v])
    o = attend(q, cache["k"], cache["v"], pos0, m["scale"])
    return o.reshape(T, H * dv) @ w["o"].T, own


def causal_conv_silu(x, w, b, tail):
    """Per channel: sum_j w[c, j] x[t - (taps - 1) + j, c] + b[c], then silu.  tail [taps - 1, C]: the inputs in
    front of x.  Returns (result, the new tail)."""
    taps = w.shape[1]
    full = np.concatenate([tail, x])
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        y[t] = (full[t:t + taps] * w.T).sum(axis=0) + b
    return silu(y), full[full.shape[0] - (taps - 1):]


def selective_scan(x, dt, A, B, C, D, S):
    """S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;  y_c = sum_n S[c, n] C_n + D_c x_c."""
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        S = np.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba1(h, w, m, state):
    """Mixer `mamba1`; state {"conv", "S"} is carried over."""
    inner, N, R, taps = m["inner"], m["state"], m["dt_rank"], m["conv"]
    xz = h @ w["in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x, state["conv"] = causal_conv_silu(x, w["conv"], w["conv.b"], state.get("conv", np.zeros((taps - 1, inner))))
    p = x @ w["x"].T
    dt = softplus(p[:, :R] @ w["dt"].T + w["dt.b"])
    y, state["S"] = selective_scan(x, dt, -np.exp(w["A_log"]), p[:, R:R + N], p[:, R + N:], w["D"],
                                   state.get("S", np.zeros((inner, N))))
    return (y * silu(z)) @ w["o"].T


# ---- feed-forward blocks ---------------------------------------------------------------------------

def dense_mlp(h, w, limit):
    return clamped_swiglu(h @ w["gate"].T, h @ w["up"].T, limit) @ w["down"].T


def route(h, router, bias, top):
    """ids [T, top] by descending logit, and the softmax over the chosen logits."""
    z = h @ router.T + bias
    ids = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    zs = np.take_along_axis(z, ids, axis=-1)
    e = np.exp(zs - zs.max(axis=-1, keepdims=True))
    return ids, e / e.sum(axis=-1, keepdims=True)


def route_margin(h, router, bias, top):
    """Per token, how far the last chosen logit lies above the first one left out (inf where all are chosen)."""
    z = np.sort(h @ router.T + bias, axis=-1)[:, ::-1]
    return z[:, top - 1] - z[:, top] if top < z.shape[1] else np.full(len(z), np.inf)


def moe_mlp(h, w, mlp):
    ids, wts = route(h, w["router"], w["router.b"], mlp["router"]["top"])
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(ids[t], wts[t]):
            ew = {k: w[f"e{e}.{k}"] for k in ("gate", "up", "down")}
            y[t] += p * dense_mlp(h[t:t + 1], ew, mlp["expert"]["limit"])[0]
    return y


# ---- the model ---------------------------------------------------------------------------------------

class LayeredOracle:
    def __init__(self, config, tensors):
        self.cfg = config
        self.w = {k: np.asarray(v, f64) for k, v in tensors.items()}
        self.reset()

    def reset(self):
        self.n_past = 0
        self.margin = np.zeros(0)   # per token, the smallest route_margin of its layers
        self.state = [{} for _ in self.cfg["layers"]]

    def part(self, prefix):
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def norm(self, x, name):
        return layer_norm(x, self.w[name], self.w[name + ".b"], self.cfg["norm"]["eps"])

    def forward(self, tokens, layers=None):
        """Appends the tokens, returns the logits of all of them; `layers` collects the residual stream."""
        mult, pos0 = self.cfg["residual_mult"], self.n_past
        x = self.w["embed"][np.asarray(tokens)] * self.cfg["embedding"]["scale"]
        v_first = None
        margin = np.full(len(tokens), np.inf)
        for i, layer in enumerate(self.cfg["layers"]):
            p, m = f"l{i}.", layer["mixer"]
            h = self.norm(x, p + "norm1")
            w = self.part(p + "mix.")
            if layer["type"] == "attention":
                mixes = m.get("v_mix", False)
                y, own = attention(h, w, m, self.state[i], pos0, v_first if mixes else None)
                if mixes and v_first is None:
                    v_first = own
            else:
                y = mamba1(h, w, m, self.state[i])
            x = x + mult * self.norm(y, p + "norm1b")
            mlp = layer.get("mlp")
            if mlp:
                h = self.norm(x, p + "norm2")
                w = self.part(p + "mlp.")
                y = dense_mlp(h, w, mlp["limit"]) if mlp["kind"] == "dense" else moe_mlp(h, w, mlp)
                if mlp["kind"] == "moe":
                    margin = np.minimum(margin, route_margin(h, w["router"], w["router.b"], mlp["router"]["top"]))
                x = x + mult * self.norm(y, p + "norm2b")
            if layers is not None:
                layers.append(x.copy())
        self.n_past += len(tokens)
        self.margin = np.concatenate([self.margin, margin])
        return self.norm(x, "final.norm") @ self.w["head"].T
