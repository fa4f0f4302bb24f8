"""Plain, slow numpy statement (float64) of the layered decoders: a stack whose layers each name a mixer (attention
with rotary positions and value mixing, a selective scan, latent attention with sinks, a matrix memory, linear
attention with a constant decay) and a feed-forward block (none, dense or mixture of experts).  `LayeredOracle` (Bozosun)
puts a norm before and after each, `FasesunOracle` runs mixer and feed-forward block side by side on one norm.
TEST INFRASTRUCTURE: one function a mechanism, loops where a loop says it best, no code shared with the library.

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


def rms_norm(x, eps):
    return x / np.sqrt((x ** 2).mean(axis=-1, keepdims=True) + eps)


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


def decayed_memory_step(S, k, v, q, decay):
    """One head, one token: S <- decay S + k v^T, S^T q.  S [dim, vdim]."""
    S = decay * S + np.outer(k, v)
    return S, S.T @ q


def lightning(h, w, m, state, eps):
    """Mixer `lightning`; state {"S"} [heads, dim, vdim] is carried over."""
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = silu(h @ w["q"].T).reshape(T, H, d), silu(h @ w["k"].T).reshape(T, H, d)
    v = silu(h @ w["v"].T).reshape(T, H, dv)
    S = state.get("S", np.zeros((H, d, dv))).copy()
    o = np.zeros((T, H, dv))
    for t in range(T):
        for a in range(H):
            S[a], o[t, a] = decayed_memory_step(S[a], k[t, a], v[t, a], q[t, a], m["decay"][a])
    state["S"] = S
    return (rms_norm(o.reshape(T, H * dv), eps) * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T


def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def matrix_memory_step(S, n, mx, q, k, v, log_i, log_f):
    """One head, one token of a matrix memory with exponential gates, held relative to exp(mx)."""
    new = max(log_f + mx, log_i)
    keep, write = np.exp(log_f + mx - new), np.exp(log_i - new)
    S, n = keep * S + write * np.outer(k, v), keep * n + write * k
    return S, n, new, S.T @ q / (max(abs(n @ q), np.exp(-new)) + 1e-6)


def mlstm(h, w, m, state, eps):
    """Mixer `mlstm`; state {"S", "n", "m"} is carried over, all of it zero in front of the first token."""
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = (h @ w["q"].T).reshape(T, H, d) * d ** -0.5, (h @ w["k"].T).reshape(T, H, d)
    v = (h @ w["v"].T).reshape(T, H, dv)
    log_i = soft_cap(h @ w["i"].T + w["i.b"], m["gate_cap"])
    log_f = -softplus(-soft_cap(h @ w["f"].T + w["f.b"], m["gate_cap"]))
    S, n, mx = (state.get(x, z).copy() for x, z in (("S", np.zeros((H, d, dv))), ("n", np.zeros((H, d))), ("m", np.zeros(H))))
    o = np.zeros((T, H, dv))
    for t in range(T):
        for a in range(H):
            S[a], n[a], mx[a], o[t, a] = matrix_memory_step(S[a], n[a], mx[a], q[t, a], k[t, a], v[t, a], log_i[t, a], log_f[t, a])
    state.update(S=S, n=n, m=mx)
    return (rms_norm(o, eps).reshape(T, H * dv) * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T


def softmax_with_sink(s, sink):
    """Weights over the scores s whose denominator also counts exp(sink)."""
    top = max(s.max(), sink)
    e = np.exp(s - top)
    return e / (e.sum() + np.exp(sink - top))


def latent_attention(h, w, m, cache, pos0, eps):
    """Mixer `latent_attention`; cache {"c", "r"}, the latents and the rotated shared keys, is appended to."""
    T, H, d, rd, dv, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = ((rms_norm(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T).reshape(T, H, d + rd)
    down = h @ w["dkv"].T
    qr = rotate_interleaved(q[:, :, d:], pos0, m["rot"])
    cache["c"] = np.concatenate([cache.get("c", np.zeros((0, R))), rms_norm(down[:, :R], eps) * w["dkv.norm"]])
    cache["r"] = np.concatenate([cache.get("r", np.zeros((0, rd))), rotate_interleaved(down[:, None, R:], pos0, m["rot"])[:, 0]])
    k = (cache["c"] @ w["uk"].T).reshape(-1, H, d)
    v = (cache["c"] @ w["uv"].T).reshape(-1, H, dv)
    o = np.zeros((T, H, dv))
    for t in range(T):
        n = pos0 + t + 1
        for a in range(H):
            s = (k[:n, a] @ q[t, a, :d] + cache["r"][:n] @ qr[t, a]) * m["scale"]
            o[t, a] = softmax_with_sink(s, w["sink"][a]) @ v[:n, a]
    return (o.reshape(T, H * dv) * sigmoid(h @ w["g"].T)) @ w["o"].T


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


def swiglu_mlp(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def route_sigmoid(h, router, correction, top):
    """ids [T, top] by descending score + correction, and the chosen experts' scores, as they are."""
    s = sigmoid(h @ router.T)
    ids = np.argsort(-(s + correction), axis=-1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, axis=-1)


def shared_moe_mlp(h, w, mlp):
    """Sigmoid-routed experts, and a shared one that every token runs behind a gate of its own."""
    ids, wts = route_sigmoid(h, w["router"], w["correction"], mlp["router"]["top"])
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(ids[t], wts[t]):
            y[t] += p * swiglu_mlp(h[t:t + 1], {k: w[f"e{e}.{k}"] for k in ("gate", "up", "down")})[0]
    if mlp.get("shared"):
        y += sigmoid(h @ w["shared.sg"].T) * swiglu_mlp(h, {k: w[f"shared.{k}"] for k in ("gate", "up", "down")})
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


class FasesunOracle(LayeredOracle):
    def runs(self):
        """The layers in the order in which they run."""
        n, loop = len(self.cfg["layers"]), self.cfg.get("loop")
        if not loop:
            return list(range(n))
        a, b = loop["start"], loop["stop"]
        return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))

    def reset(self):
        super().reset()
        self.state = [{} for _ in self.runs()]

    def forward(self, tokens, layers=None):
        eps, pos0 = self.cfg["norm"]["eps"], self.n_past
        x = self.w["embed"][np.asarray(tokens)]
        margin = np.full(len(tokens), np.inf)
        for r, i in enumerate(self.runs()):
            layer, p = self.cfg["layers"][i], f"l{i}."
            m, mlp = layer["mixer"], layer.get("mlp")
            h = rms_norm(x, eps) * self.w[p + "norm1"]
            w = self.part(p + "mix.")
            if layer["type"] == "latent_attention":
                y = latent_attention(h, w, m, self.state[r], pos0, eps)
            else:
                y = {"mlstm": mlstm, "lightning": lightning}[layer["type"]](h, w, m, self.state[r], eps)
            if mlp:
                w = self.part(p + "mlp.")
                y = y + shared_moe_mlp(h, w, mlp)
                z = np.sort(sigmoid(h @ w["router"].T) + w["correction"], axis=-1)[:, ::-1]
                top = mlp["router"]["top"]
                if top < z.shape[1]:
                    margin = np.minimum(margin, z[:, top - 1] - z[:, top])
            x = x + y
            if layers is not None:
                layers.append(x.copy())
        self.n_past += len(tokens)
        self.margin = np.concatenate([self.margin, margin])
        return (rms_norm(x, eps) * self.w["final.norm"]) @ self.w["embed"].T
