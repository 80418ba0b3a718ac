"""A plain float64 restatement of the Kemuzen design, one function per mechanism, written from its equations
with loops over tokens and heads.  It shares no code with the library and is slow on purpose.

A model is (config, tensors): the parsed config.json and a dict name -> float64 array.  `state` objects are
explicit, so a sequence can be continued from where an earlier call left it."""
import math

import numpy as np


# ---- pieces ------------------------------------------------------------------------------------
def rms(x, eps):
    """x over its root mean square"""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softcap(z, cap):
    return z if not cap else cap * np.tanh(z / cap)


def sinusoid(position, width):
    """sin and cos of position * 10000^(-2i/width) in turn"""
    out = np.zeros(width)
    for e in range(width):
        a = position * 10000.0 ** (-(e - e % 2) / width)
        out[e] = math.cos(a) if e % 2 else math.sin(a)
    return out


def visible(position, mask):
    """Positions that a token at `position` looks at: its window and the sequence's first tokens."""
    size, keep = (mask["size"], mask.get("keep_first", 0)) if mask else (None, 0)
    return [j for j in range(position + 1) if size is None or position - j < size or j < keep]


def slope(head, heads):
    """what a distance of one costs this head's score"""
    return 2.0 ** (-8.0 * (head + 1) / heads)


def short_conv(history, now, weight, bias=None):
    """A causal filter per channel and silu.  history: the inputs before `now`, oldest first (fewer than taps - 1 of
    them at the start of a sequence, where zeros stand in); weight's last column meets `now`."""
    taps = weight.shape[1]
    z = weight[:, taps - 1] * now
    for back in range(1, taps):
        if back <= len(history):
            z = z + weight[:, taps - 1 - back] * history[-back]
    history.append(now)
    return silu(z if bias is None else z + bias)


def unit(x):
    return x / math.sqrt(float(x @ x) + 1e-6)


def softmax(s):
    w = np.exp(s - s.max())
    return w / w.sum()


def delta_step(S, q, k, v, beta, g):
    """One token of the gated delta rule for one head; S [dim, vdim] -> (S, o)"""
    S = g * S
    u = beta * (v - S.T @ k)
    S = S + np.outer(k, u)
    return S, S.T @ q


def ssd_step(S, x, B, C, dt, a, D):
    """One token of the state-space recurrence for one head; S [state, vdim] -> (S, y); a = exp(A_log)"""
    S = math.exp(-a * dt) * S + dt * np.outer(B, x)
    return S, S.T @ C + D * x


# ---- mixers: (tensors with the layer's prefix removed, sizes, eps, rows h, first position, state) -> rows --------
def attention_rows(t, m, eps, h, position, state, bias=False, alibi=False):
    """Heads' outputs before the output projection.  state: {"k": [kv_heads, dim] per position, "v": ..}.  A layer without
    projections of keys and values finds its positions already there."""
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    b = lambda n: t[n + ".b"] if bias else 0.0
    out = []
    if "k" in t:
        for x in h:
            state["k"].append(rms((t["k"] @ x + b("k")).reshape(G, dim), eps) * t["k.norm"])
            state["v"].append((t["v"] @ x + b("v")).reshape(G, vdim))
    for r, x in enumerate(h):
        p = position + r
        q = rms((t["q"] @ x + b("q")).reshape(H, dim), eps) * t["q.norm"]
        keys = visible(p, m.get("mask"))
        heads = []
        for head in range(H):
            g = head // (H // G)
            k = np.stack([state["k"][j][g] for j in keys])
            v = np.stack([state["v"][j][g] for j in keys])
            s = softcap((k @ q[head]) * m["scale"], m.get("softcap"))
            if alibi:
                s = s - slope(head, H) * (p - np.array(keys, np.float64))
            heads.append(softmax(s) @ v)
        if "g" in t:
            heads = [o * z for o, z in zip(heads, sigmoid(t["g"] @ x))]
        out.append(np.concatenate(heads))
    return np.stack(out)


def attention(t, m, eps, h, position, state):
    return attention_rows(t, m, eps, h, position, state, bias=True) @ t["o"].T + t["o.b"]


def delta(t, m, eps, h, position, state):
    """state: {"S": [heads, dim, vdim], "q", "k", "v": inputs of the three filters}"""
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    out = []
    for x in h:
        q, k, v = (short_conv(state[n], t[n] @ x, t[n + ".conv"]) for n in "qkv")
        q, k, v = q.reshape(G, dim), k.reshape(G, dim), v.reshape(H, vdim)
        beta = sigmoid(t["b"] @ x)
        g = np.exp(-np.exp(t["A_log"]) * softplus(t["a"] @ x + t["dt_bias"]))
        rows = []
        for head in range(H):
            j = head // (H // G)
            state["S"][head], o = delta_step(state["S"][head], unit(q[j]) * dim ** -0.5, unit(k[j]), v[head], beta[head], g[head])
            rows.append(rms(o, eps) * t["norm"])
        out.append(t["o"] @ (np.concatenate(rows) * silu(t["g"] @ x)))
    return np.stack(out)


def ssd(t, m, eps, h, position, state):
    """state: {"S": [heads, state, vdim], "in": inputs of the filter}"""
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    out = []
    for row in h:
        z, xbc, dt = np.split(t["in"] @ row, [inner, 2 * inner + 2 * G * N])
        x, B, C = np.split(short_conv(state["in"], xbc, t["conv"], t["conv.b"]), [inner, inner + G * N])
        dt = softplus(dt + t["dt_bias"])
        y = np.zeros((H, P))
        for head in range(H):
            j = head // (H // G)
            state["S"][head], y[head] = ssd_step(state["S"][head], x.reshape(H, P)[head], B.reshape(G, N)[j], C.reshape(G, N)[j],
                                                 dt[head], math.exp(t["A_log"][head]), t["D"][head])
        y = y.reshape(-1) * silu(z)
        y = rms(y.reshape(m["norm_groups"], -1), eps).reshape(-1) * t["norm"]
        out.append(t["o"] @ y)
    return np.stack(out)


def sub(t, prefix):
    return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}


def parallel(t, m, eps, h, position, state):
    lt = sub(t, "left.")
    left = attention_rows(lt, m["left"], eps, h, position, state["left"], alibi=True) @ lt["o"].T
    right = ssd(sub(t, "right."), m["right"], eps, h, position, state["right"])
    return m["left_scale"] * left + m["right_scale"] * right


def swiglu(t, h):
    return np.stack([t["down"] @ (silu(t["gate"] @ x) * (t["up"] @ x)) for x in h])


def token_side(t, e, x, eps):
    """What a layer takes from its part e of the tokens' own vectors"""
    return np.stack([rms(t["proj"] @ (gelu_tanh(t["gate"] @ r) * v), eps) * t["norm"] for r, v in zip(x, e)])


MIXERS = {"attention": attention, "delta": delta, "parallel": parallel}


def new_state(layer):
    m = layer["mixer"]
    if layer["type"] == "delta":
        return {"S": np.zeros((m["heads"], m["dim"], m["vdim"])), "q": [], "k": [], "v": []}
    if layer["type"] == "parallel":
        r = m["right"]
        return {"left": {"k": [], "v": []}, "right": {"S": np.zeros((r["heads"], r["state"], r["vdim"])), "in": []}}
    return {"k": [], "v": []}


# ---- the model -----------------------------------------------------------------------------------
class Oracle:
    def __init__(self, config, tensors):
        self.cfg, self.t = config, {k: np.asarray(v, np.float64) for k, v in tensors.items()}

    def new_states(self):
        out = []
        for layer in self.cfg["layers"]:
            source = layer["mixer"].get("kv_from") if layer["type"] == "attention" else None
            out.append(new_state(layer) if source is None else out[source])
        return out

    def _norm(self, name, x):
        return rms(x, self.cfg["norm"]["eps"]) * (1.0 + self.t[name])

    def forward(self, tokens, position=0, states=None, residuals=None):
        """Logits of `tokens`, the first of them at `position`; residuals (a list) receives x after every layer."""
        states = self.new_states() if states is None else states
        cfg, eps, ids = self.cfg, self.cfg["norm"]["eps"], np.asarray(tokens)
        x = self.t["embed"][ids] * cfg["embedding"]["scale"]
        x = x + np.stack([sinusoid(position + r, cfg["width"]) for r in range(len(ids))])
        for i, layer in enumerate(cfg["layers"]):
            p = "l%d." % i
            x = x + self._norm(p + "norm1", MIXERS[layer["type"]](sub(self.t, p + "mix."), layer["mixer"], eps, x, position, states[i]))
            if layer.get("mlp") is not None:
                x = x + self._norm(p + "norm2", swiglu(sub(self.t, p + "mlp."), x))
            if cfg.get("token_side"):
                d = cfg["token_side"]["dim"]
                x = x + token_side(sub(self.t, p + "side."), self.t["side.embed"][ids, i * d:(i + 1) * d], x, eps)
            if residuals is not None:
                residuals.append(x.copy())
        return softcap(self._norm("final.norm", x) @ self.t["embed"].T, cfg.get("logit_softcap"))

    def greedy(self, tokens, n):
        states, out = self.new_states(), []
        logits = self.forward(tokens, 0, states)[-1]
        position = len(tokens)
        for _ in range(n):
            out.append(int(np.argmax(logits)))
            if len(out) == n:
                break
            logits = self.forward(out[-1:], position, states)[-1]
            position += 1
        return out
