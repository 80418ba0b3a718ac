"""A plain float64 restatement of the Pakirax design, one function per mechanism, written from its equations
with loops over tokens and heads.  It shares no code with the library and is slow on purpose.

A model is (config, tensors): the parsed config.json and a dict name -> float64 array.  `state` objects are
explicit, so a sequence can be continued from where an earlier call left it."""
import math

import numpy as np

_erf = np.vectorize(math.erf, otypes=[np.float64])


# ---- pieces ------------------------------------------------------------------------------------
def layer_norm(x, w, b, eps):
    mean = x.mean(-1, keepdims=True)
    var = ((x - mean) ** 2).mean(-1, keepdims=True)
    return (x - mean) / np.sqrt(var + eps) * w + b


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def gelu_erf(z):
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def rotate_half(x, position, base, dims):
    """The first `dims` entries of x (last axis) turned in pairs (i, i + dims / 2) by position * base^(-2i/dims)."""
    out = np.array(x)
    half = dims // 2
    for i in range(half):
        a = position * base ** (-2.0 * i / dims)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * math.cos(a) - v * math.sin(a)
        out[..., i + half] = v * math.cos(a) + u * math.sin(a)
    return out


def window_keys(position, size):
    """Positions a token may look at: itself and the size - 1 before it (size None: every one before it)."""
    return range(0 if size is None else max(0, position - size + 1), position + 1)


def decay(z, tau):
    """sigmoid(z)^(1 / tau)"""
    return np.exp(np.where(z >= 0, -np.log1p(np.exp(-np.abs(z))), z - np.log1p(np.exp(-np.abs(z)))) / tau)


# ---- mixers: (tensors with the layer's prefix removed, sizes, rows h, first position, state) -> rows ------------
def latent_attention(t, m, eps, h, position, state):
    """state: {"c": [latent per position], "k": [rotated key part per position]}"""
    H, dim, rot, vdim, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    size = m["mask"]["size"] if m.get("mask") else None
    out = []
    for r, x in enumerate(h):
        p = position + r
        cq = rms_norm(t["dq"] @ x, t["dq.norm"], eps)
        q = (t["uq"] @ cq).reshape(H, dim + rot)
        ckv = t["dkv"] @ x
        state["c"].append(rms_norm(ckv[:rank], t["dkv.norm"], eps))
        state["k"].append(rotate_half(ckv[rank:], p, m["rot"]["base"], m["rot"]["dims"]))
        gate = sigmoid(t["g"] @ x)
        heads = []
        for head in range(H):
            uk = t["uk"][head * dim:(head + 1) * dim]
            uv = t["uv"][head * vdim:(head + 1) * vdim]
            qn, qr = q[head, :dim], rotate_half(q[head, dim:], p, m["rot"]["base"], m["rot"]["dims"])
            keys = list(window_keys(p, size))
            c = np.stack([state["c"][j] for j in keys])
            k = np.stack([state["k"][j] for j in keys])
            s = ((c @ uk.T) @ qn + k @ qr) * m["scale"]
            w = np.exp(s - s.max())
            w /= w.sum()
            heads.append(w @ (c @ uv.T) * gate[head])
        out.append(t["o"] @ np.concatenate(heads))
    return np.stack(out)


def gla(t, m, eps, h, position, state):
    """state: {"S": [heads, dim, vdim]}"""
    H, dk, dv, tau = m["heads"], m["dim"], m["vdim"], m["tau"]
    out = []
    for x in h:
        q = (t["q"] @ x).reshape(H, dk) * dk ** -0.5
        k = (t["k"] @ x).reshape(H, dk)
        v = (t["v"] @ x).reshape(H, dv)
        alpha = decay(t["a2"] @ (t["a1"] @ x) + t["a2.b"], tau).reshape(H, dk)
        rows = []
        for head in range(H):
            S = alpha[head][:, None] * state["S"][head] + np.outer(k[head], v[head])
            state["S"][head] = S
            rows.append(rms_norm(S.T @ q[head], t["norm"], eps))
        out.append(t["o"] @ (np.concatenate(rows) * silu(t["g"] @ x)))
    return np.stack(out)


def dense_ff(t, h):
    return np.stack([t["down"] @ gelu_erf(t["up"] @ x) for x in h])


MIXERS = {"latent_attention": latent_attention, "gla": gla}


def new_state(layer):
    if layer["type"] == "gla":
        m = layer["mixer"]
        return {"S": np.zeros((m["heads"], m["dim"], m["vdim"]))}
    return {"c": [], "k": []}


# ---- the model -----------------------------------------------------------------------------------
class Oracle:
    def __init__(self, config, tensors):
        self.cfg, self.t = config, {k: np.asarray(v, np.float64) for k, v in tensors.items()}

    def new_states(self):
        return [new_state(layer) for layer in self.cfg["layers"]]

    def _sub(self, prefix):
        return {k[len(prefix):]: v for k, v in self.t.items() if k.startswith(prefix)}

    def _norm(self, name, x):
        return layer_norm(x, self.t[name], self.t[name + ".b"], self.cfg["norm"]["eps"])

    def forward(self, tokens, position=0, states=None, residuals=None):
        """Logits of `tokens`, the first of them at `position`; residuals (a list) receives x after every layer."""
        states = self.new_states() if states is None else states
        eps, mult = self.cfg["norm"]["eps"], self.cfg["residual_mult"]
        x = self.t["embed"][np.asarray(tokens)]
        for i, layer in enumerate(self.cfg["layers"]):
            p = "l%d." % i
            y = MIXERS[layer["type"]](self._sub(p + "mix."), layer["mixer"], eps, self._norm(p + "norm1", x), position, states[i])
            x = x + mult * self._norm(p + "norm1b", y)
            if layer["mlp"] is not None:
                y = dense_ff(self._sub(p + "mlp."), self._norm(p + "norm2", x))
                x = x + mult * self._norm(p + "norm2b", y)
            if residuals is not None:
                residuals.append(x.copy())
        return self._norm("final.norm", x) @ self.t["embed"].T

    def greedy(self, tokens, n):
        states, position, out = self.new_states(), 0, []
        logits = self.forward(tokens, 0, states)[-1]
        position = len(tokens)
        for _ in range(n):
            out.append(int(np.argmax(logits)))
            if len(out) == n:
                break
            logits = self.forward(out[-1:], position, states)[-1]
            position += 1
        return out
