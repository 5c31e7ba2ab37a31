"""Plain restatement of layered decoders in numpy: Suripel (attention with pooled blocks, gated delta rule, retention) and
Lesarax (attention with sinks whose values are its keys, latent attention, mixture of experts, looped layers).

Test infrastructure only: one function per mechanism, whole sequences at once or token by token from the
equations, in float64, sharing nothing with the product path. A model is (config, weights): the dictionary of
config.json and a dictionary of arrays under the tensor names of model.safetensors. Shapes: rows are tokens, [T][channels].
"""
import json

import numpy as np

F = np.float64


def load_safetensors(path):
    """name -> float64 (or int32) array. Little-endian; the elements of a bfloat16 are the upper halves of float32."""
    raw = open(path, "rb").read()
    n = int.from_bytes(raw[:8], "little")
    out = {}
    for name, d in json.loads(raw[8:8 + n]).items():
        if name == "__metadata__":
            continue
        lo, hi = d["data_offsets"]
        body = raw[8 + n + lo:8 + n + hi]
        if d["dtype"] == "BF16":
            a = (np.frombuffer(body, "<u2").astype(np.uint32) << 16).view(np.float32).astype(F)
        elif d["dtype"] == "F32":
            a = np.frombuffer(body, "<f4").astype(F)
        elif d["dtype"] == "I32":
            a = np.frombuffer(body, "<i4")
        else:
            raise ValueError(d["dtype"])
        out[name] = a.reshape(d["shape"])
    return out


def bf16_bits(x):
    """float array -> uint16 bit patterns, round to nearest even."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32).astype(np.uint64)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_round(x):
    return (bf16_bits(x).astype(np.uint32) << 16).view(np.float32).astype(F)


def save_safetensors(path, tensors):
    """Writes every array as bfloat16 (rounded to nearest even)."""
    head, blobs, at = {}, [], 0
    for name, a in tensors.items():
        b = bf16_bits(a).tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    text = json.dumps(head).encode()
    with open(path, "wb") as f:
        f.write(len(text).to_bytes(8, "little") + text + b"".join(blobs))


# ---------------------------------------------------------------------------------------------- small pieces
def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(0.0, x)


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w


def over_rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return over_rms(x, eps) * w


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def causal_conv(x, w):
    """y[t][c] = sum_j w[c][j] x[t - taps + 1 + j][c], zeros in front of the sequence."""
    T, taps = x.shape[0], w.shape[1]
    y = np.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * x[s]
    return y


def rotate_half(x, pos, dims, base):
    """x [..., dim] at position pos: dimension i turns with dimension i + dims / 2; what lies past dims stays."""
    y = np.array(x, dtype=F)
    half = dims // 2
    for i in range(half):
        a = pos * float(base) ** (-2.0 * i / dims)
        u, v = x[..., i], x[..., i + half]
        y[..., i] = u * np.cos(a) - v * np.sin(a)
        y[..., i + half] = v * np.cos(a) + u * np.sin(a)
    return y


def polynorm(z, abce, eps):
    a, b, c, e = abce
    return a * over_rms(z, eps) + b * over_rms(z ** 2, eps) + c * over_rms(z ** 3, eps) + e


# ---------------------------------------------------------------------------------------------- mixers
def pooled_window_attention(q, k, v, scale, size, pool, lead=None):
    """q [T][H][d], k [T][G][d], v [T][G][dv] -> [T][H][dv]. Query i attends to tokens (i - size, i] and to the mean key /
    value of each block of `pool` tokens that ends at i - lead or earlier (lead: size), under a common softmax."""
    lead = size if lead is None else lead
    T, H = q.shape[:2]
    rep = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]), dtype=F)
    for i in range(T):
        lo = max(0, i - size + 1)
        nb = max(0, (i - lead + 1) // pool)           # blocks b with b * pool + pool - 1 <= i - lead
        for h in range(H):
            kk, vv = k[:, h // rep], v[:, h // rep]
            keys = [kk[b * pool:(b + 1) * pool].mean(0) for b in range(nb)] + [kk[j] for j in range(lo, i + 1)]
            vals = [vv[b * pool:(b + 1) * pool].mean(0) for b in range(nb)] + [vv[j] for j in range(lo, i + 1)]
            s = np.array([q[i, h] @ key for key in keys]) * scale
            p = np.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ np.array(vals)
    return out


def delta_rule(q, k, v, g, beta, state=None):
    """q, k [T][H][d], v [T][H][dv], g, beta [T][H]; state [H][d][dv]. Decay, erase and write, then read."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), dtype=F) if state is None else state
    out = np.zeros((T, H, v.shape[2]), dtype=F)
    for t in range(T):
        for h in range(H):
            S[h] = g[t, h] * S[h]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] = S[h] + np.outer(k[t, h], u)
            out[t, h] = S[h].T @ q[t, h]
    return out


def retention(q, k, v, decay, state=None):
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), dtype=F) if state is None else state
    out = np.zeros((T, H, v.shape[2]), dtype=F)
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ q[t, h]
    return out


# ---------------------------------------------------------------------------------------------- layers
def mixer_attention(cfg, w, p, mx, h, kv_of):
    T = h.shape[0]
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = causal_conv(h @ w[p + "q"].T, w[p + "q.conv"]).reshape(T, H, d)
    if mx.get("kv_from") is None:
        k = causal_conv(h @ w[p + "k"].T, w[p + "k.conv"]).reshape(T, G, d)
        v = causal_conv(h @ w[p + "v"].T, w[p + "v.conv"]).reshape(T, G, dv)
    else:
        k, v = kv_of[mx["kv_from"]]
    o = pooled_window_attention(q, k, v, mx["scale"], mx["mask"]["size"], mx["mask"]["pool"])
    return o.reshape(T, H * dv) @ w[p + "o"].T, (k, v)


def mixer_delta(cfg, w, p, mx, h):
    T = h.shape[0]
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    eps = cfg["norm"]["eps"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    rep = H // G
    q = np.repeat(unit(q.reshape(T, G, d)), rep, axis=1) * d ** -0.5
    k = np.repeat(unit(k.reshape(T, G, d)), rep, axis=1)
    beta = sigmoid(h @ w[p + "b"].T)
    g = np.exp(-np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o = delta_rule(q, k, v.reshape(T, H, dv), g, beta)
    o = over_rms(o, eps) * w[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def mixer_retention(cfg, w, p, mx, h):
    T = h.shape[0]
    H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
    q, k = ((h @ w[p + n].T).reshape(T, H, d) for n in "qk")
    v = (h @ w[p + "v"].T).reshape(T, H, dv)
    for t in range(T):
        q[t] = rotate_half(q[t], t, mx["rot"]["dims"], mx["rot"]["base"])
        k[t] = rotate_half(k[t], t, mx["rot"]["dims"], mx["rot"]["base"])
    o = retention(q, k * d ** -0.5, v, mx["decay"])
    o = over_rms(o, cfg["norm"]["eps"])
    return (o.reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def feed_forward(cfg, w, p, h):
    return polynorm(h @ w[p + "up"].T, w[p + "act"], cfg["norm"]["eps"]) @ w[p + "down"].T


# ---------------------------------------------------------------------------------------------- Lesarax
def sink_attention(q, k, v, scale, sinks, size=None):
    """q [T][H][d], k [T][G][d], v [T][G][dv] -> [T][H][dv]: causal, over the last `size` tokens (None: all of them), with
    exp(sink of the head) as one more term of the softmax's denominator."""
    T, H = q.shape[:2]
    rep = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]), dtype=F)
    for i in range(T):
        lo = 0 if size is None else max(0, i - size + 1)
        for h in range(H):
            s = k[lo:i + 1, h // rep] @ q[i, h] * scale
            top = max(s.max(), sinks[h])
            p = np.exp(s - top)
            out[i, h] = p @ v[lo:i + 1, h // rep] / (p.sum() + np.exp(sinks[h] - top))
    return out


def rotate_rows(x, rot):
    """x [T][heads][dim], row t at position t."""
    return np.stack([rotate_half(x[t], t, rot["dims"], rot["base"]) for t in range(x.shape[0])])


def mixer_tied_attention(cfg, w, p, mx, h):
    """Rotary attention with sinks; the values are the keys before their rotation."""
    T, H, G, d = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"]
    q = (h @ w[p + "q"].T).reshape(T, H, d)
    k = (h @ w[p + "k"].T).reshape(T, G, d)
    o = sink_attention(rotate_rows(q, mx["rot"]), rotate_rows(k, mx["rot"]), k, mx["scale"], w[p + "sink"])
    return o.reshape(T, H * d) @ w[p + "o"].T


def mixer_latent_attention(cfg, w, p, mx, h):
    """Queries from a normed latent, keys and values from another one, one rotated key part for all heads, sinks, a window
    and a gate per head."""
    T, H, d, r, dv = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    eps, rank = cfg["norm"]["eps"], mx["kv_rank"]
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(T, H, d + r)
    ckv = h @ w[p + "dkv"].T
    c = rms_norm(ckv[:, :rank], w[p + "dkv.norm"], eps)
    k_rot = rotate_rows(ckv[:, None, rank:], mx["rot"])
    q = np.concatenate([q[..., :d], rotate_rows(q[..., d:], mx["rot"])], -1)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, d), np.repeat(k_rot, H, 1)], -1)
    v = (c @ w[p + "uv"].T).reshape(T, H, dv)
    o = sink_attention(q, k, v, mx["scale"], w[p + "sink"], mx["mask"]["size"])
    o = o * sigmoid(h @ w[p + "g"].T)[..., None]
    return o.reshape(T, H * dv) @ w[p + "o"].T


def clamped_expert(h, gate, up, down, limit):
    g = np.minimum(gate @ h, limit)
    u = np.clip(up @ h, -limit, limit)
    return down @ (g * sigmoid(1.702 * g) * (u + 1))


def route(logits, top):
    """(indices of the `top` largest, softmax over them)"""
    pick = np.argsort(-logits, kind="stable")[:top]
    e = np.exp(logits[pick] - logits[pick].max())
    return pick, e / e.sum()


def mixture_of_experts(w, p, mlp, h):
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(*route(w[p + "router"] @ h[t], mlp["router"]["top"])):
            q = p + f"e{e}."
            out[t] += a * clamped_expert(h[t], w[q + "gate"], w[q + "up"], w[q + "down"], mlp["expert"]["limit"])
    return out


def layer_runs(cfg):
    """[(layer, whether it is the first one of a pass through the looped part)] in the order they run."""
    lp = cfg["loop"]
    runs = [(i, False) for i in range(lp["start"])]
    for _ in range(lp["times"]):
        runs += [(i, i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, False) for i in range(lp["stop"], len(cfg["layers"]))]


def lesarax_forward(cfg, w, tokens, layers_out=None):
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x0 = np.array(w["embed"][np.asarray(tokens)], dtype=F)
    x = x0
    for i, pass_starts in layer_runs(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        if pass_starts:
            x = np.concatenate([x, x0], -1) @ w["loop.in"].T
        mixer = {"attention": mixer_tied_attention, "latent_attention": mixer_latent_attention}[layer["type"]]
        x = x + m * mixer(cfg, w, p + "mix.", layer["mixer"], rms_norm(x, w[p + "norm1"], eps))
        if layer.get("mlp") is not None:
            x = x + m * mixture_of_experts(w, p + "mlp.", layer["mlp"], rms_norm(x, w[p + "norm2"], eps))
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T][vocab] of a whole sequence; appends the residual stream after every layer to layers_out."""
    if cfg["architecture"] == "Lesarax":
        return lesarax_forward(cfg, w, tokens, layers_out)
    eps = cfg["norm"]["eps"]
    x = np.array(w["embed"][np.asarray(tokens)], dtype=F)
    kv = {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = layer_norm(x, w[p + "norm1"], eps)
        h = h + causal_conv(h, w[p + "canon1"])
        mx, m = layer["mixer"], p + "mix."
        if layer["type"] == "attention":
            y, kv[i] = mixer_attention(cfg, w, m, mx, h, kv)
        elif layer["type"] == "delta":
            y = mixer_delta(cfg, w, m, mx, h)
        elif layer["type"] == "retention":
            y = mixer_retention(cfg, w, m, mx, h)
        else:
            raise ValueError(layer["type"])
        x = x + y
        if layer.get("mlp") is not None:
            h = layer_norm(x, w[p + "norm2"], eps)
            h = h + causal_conv(h, w[p + "canon2"])
            x = x + feed_forward(cfg, w, p + "mlp.", h)
        if layers_out is not None:
            layers_out.append(x.copy())
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T
