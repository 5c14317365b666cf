"""A plain, slow float64 implementation of the Vuladra design, one function per mechanism, written
from the design's equations and sharing no code with the package: whole sequences at once, dense
score matrices, explicit masks, explicit token loops, no cache. Tests build configurations and
random weights here."""
import math

import torch

F64 = torch.float64
ALPHA = 1.702          # slope of the routed experts' gate


# ---- configuration builders ----------------------------------------------------------------
def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit, shared=None):
    """shared: (ff, limit) of the expert that every token uses, or None."""
    f = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        f["shared"] = {"ff": shared[0], "limit": shared[1]}
    return f


def pooled_layer(heads, kv_heads, dim, vdim, scale, window, pool, mlp):
    """Sigmoid attention over a sliding window and pooled blocks before it (pool None: window only)."""
    mask = {"size": window}
    if pool:
        mask["pool"] = pool
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": mask}}


def side_layer(left, right, left_scale, right_scale, mlp):
    """left: (heads, kv_heads, dim, vdim, scale, window), right: (dim, vdim, decays)."""
    h, g, d, dv, sc, win = left
    rd, rdv, decay = right
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": {"heads": h, "kv_heads": g, "dim": d, "vdim": dv, "scale": sc, "mask": {"size": win}},
                      "left_scale": left_scale,
                      "right": {"heads": len(decay), "dim": rd, "vdim": rdv, "decay": list(decay)},
                      "right_scale": right_scale}}


def mamba_layer(inner, state, dt_rank, taps, mlp):
    return {"type": "mamba1", "mlp": mlp, "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": taps}}


def config(layers, width, vocab, eps):
    return {"architecture": "Vuladra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def random_weights(cfg, seed):
    """name -> bf16 tensor, under the names a model folder uses."""
    g = torch.Generator().manual_seed(seed)
    W, out = cfg["width"], {}

    def mat(name, rows, cols, std=None):
        out[name] = (torch.randn(rows, cols, generator=g) * (std or 1.0 / math.sqrt(cols))).to(torch.bfloat16)

    def vec(name, n, mean, std):
        out[name] = (mean + std * torch.randn(n, generator=g)).to(torch.bfloat16)

    def glu(p, ff):
        mat(p + "gate", ff, W, 1.5 / math.sqrt(W))
        mat(p + "up", ff, W, 1.5 / math.sqrt(W))
        mat(p + "down", W, ff)

    mat("embed", cfg["vocab"], W, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if L["mlp"] else ()):
            vec(p + n, W, 1.0, 0.2)
        x = p + "mix."
        if L["type"] == "attention":
            H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            mat(x + "q", H * D, W)
            mat(x + "k", G * D, W)
            mat(x + "v", G * Dv, W)
            vec(x + "q.norm", H * D, 1.0, 0.2)
            vec(x + "k.norm", G * D, 1.0, 0.2)
            vec(x + "pb", H, -1.0, 1.0)
            mat(x + "g", H * Dv, W)
            mat(x + "o", W, H * Dv)
        elif L["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            mat(x + "left.q", H * D, W)
            mat(x + "left.k", G * D, W)
            mat(x + "left.v", G * Dv, W)
            mat(x + "left.o", W, H * Dv)
            H, D, Dv = r["heads"], r["dim"], r["vdim"]
            mat(x + "right.q", H * D, W)
            mat(x + "right.k", H * D, W)
            mat(x + "right.v", H * Dv, W)
            mat(x + "right.g", H * Dv, W)
            mat(x + "right.o", W, H * Dv)
            vec(x + "right.norm", H * Dv, 1.0, 0.2)
        else:
            C, N, R, taps = m["inner"], m["state"], m["dt_rank"], m["conv"]
            mat(x + "in", 2 * C, W)
            mat(x + "conv", C, taps, 0.6)
            vec(x + "conv.b", C, 0.0, 0.3)
            mat(x + "x", R + 2 * N, C)
            mat(x + "dt", C, R)
            vec(x + "dt.b", C, -1.5, 1.0)
            out[x + "A_log"] = (torch.log(torch.arange(1, N + 1).float())[None] - 1.0 +
                                0.3 * torch.randn(C, N, generator=g)).to(torch.bfloat16)
            vec(x + "D", C, 1.0, 0.3)
            mat(x + "o", W, C)
        f = L["mlp"]
        if f and f["kind"] == "dense":
            glu(p + "mlp.", f["ff"])
        elif f:
            mat(p + "mlp.router", f["router"]["experts"], W)
            for e in range(f["router"]["experts"]):
                glu(p + f"mlp.e{e}.", f["expert"]["ff"])
            if f.get("shared"):
                glu(p + "mlp.shared.", f["shared"]["ff"])
    vec("final.norm", W, 1.0, 0.2)
    return out


# ---- mechanisms ------------------------------------------------------------------------------
def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(x):
    return x * torch.sigmoid(x)


def visible(T, window):
    """[T, T] bool: row i sees column j when 0 <= i - j < window."""
    dist = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (dist >= 0) & (dist < window)


def pooled_rows(x, pool):
    """x [T, ...] -> the means of rows 0 .. pool - 1, pool .. 2 pool - 1, ... (whole blocks only)."""
    n = x.shape[0] // pool
    return torch.stack([x[b * pool:(b + 1) * pool].mean(0) for b in range(n)]) if n else x[:0]


def pooled_sigmoid_attention(q, k, v, scale, bias, window, pool):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]. Position i weighs every token of its window and every
    block of `pool` tokens that ends at or before i - window by sigmoid(score + bias[h]); the weights
    are not normalised."""
    T, H, _ = q.shape
    G = k.shape[1]
    keys, vals, seen = k, v, visible(T, window)
    if pool:
        keys, vals = torch.cat([k, pooled_rows(k, pool)]), torch.cat([v, pooled_rows(v, pool)])
        n = keys.shape[0] - T
        last = torch.arange(n) * pool + pool - 1                      # a block's last position
        seen = torch.cat([seen, last[None, :] <= (torch.arange(T)[:, None] - window)], 1)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        wt = torch.sigmoid((q[:, h] @ keys[:, g].T) * scale + bias[h]) * seen.to(F64)
        out[:, h] = wt @ vals[:, g]
    return out


def pooled_attention(h, m, w, p, eps):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    # the norm runs over the whole projection, all heads together
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).view(T, H, D)
    k = rms_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps).view(T, G, D)
    v = (h @ w[p + "v"].T).view(T, G, Dv)
    o = pooled_sigmoid_attention(q, k, v, m["scale"], w[p + "pb"], m["mask"]["size"], m["mask"].get("pool"))
    o = o.reshape(T, H * Dv) * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def window_softmax_attention(q, k, v, scale, window):
    T, H, _ = q.shape
    G = k.shape[1]
    seen = visible(T, window)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(~seen, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def decayed_linear_attention(q, k, v, decay):
    """q, k [T, H, D], v [T, H, Dv]: S <- decay[h] S + k v^T, o = S^T q, S = 0 at the start."""
    T, H, D = q.shape
    o = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        S = torch.zeros(D, v.shape[2], dtype=F64)
        for t in range(T):
            S = decay[h] * S + torch.outer(k[t, h], v[t, h])
            o[t, h] = q[t, h] @ S
    return o


def side_by_side(h, m, w, p, eps):
    T = h.shape[0]
    a, r = m["left"], m["right"]
    H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
    l = p + "left."
    o = window_softmax_attention((h @ w[l + "q"].T).view(T, H, D), (h @ w[l + "k"].T).view(T, G, D),
                                 (h @ w[l + "v"].T).view(T, G, Dv), a["scale"], a["mask"]["size"])
    left = o.reshape(T, H * Dv) @ w[l + "o"].T
    H, D, Dv = r["heads"], r["dim"], r["vdim"]
    l = p + "right."
    o = decayed_linear_attention(silu(h @ w[l + "q"].T).view(T, H, D), silu(h @ w[l + "k"].T).view(T, H, D),
                                 silu(h @ w[l + "v"].T).view(T, H, Dv), r["decay"])
    o = rms_norm(o.reshape(T, H * Dv), w[l + "norm"], eps) * torch.sigmoid(h @ w[l + "g"].T)
    right = o @ w[l + "o"].T
    return m["left_scale"] * left + m["right_scale"] * right


def causal_conv(x, taps_w, bias):
    """x [T, C], taps_w [C, taps]: y_t = sum_j taps_w[:, j] x_(t - taps + 1 + j) + bias."""
    T, C = x.shape
    n = taps_w.shape[1]
    y = torch.zeros(T, C, dtype=F64)
    for t in range(T):
        y[t] = bias
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                y[t] += taps_w[:, j] * x[s]
    return y


def selective_scan(x, dt, A, B, C, D):
    """x, dt [T, c], A [c, n], B, C [T, n], D [c]: S <- exp(dt A) S + dt x B, y = S C + D x."""
    T, c = x.shape
    S = torch.zeros(c, A.shape[1], dtype=F64)
    y = torch.zeros(T, c, dtype=F64)
    for t in range(T):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba_mixer(h, m, w, p, eps):
    C, N, R = m["inner"], m["state"], m["dt_rank"]
    u = h @ w[p + "in"].T
    x, z = u[:, :C], u[:, C:]
    x = silu(causal_conv(x, w[p + "conv"], w[p + "conv.b"]))
    s = x @ w[p + "x"].T
    dt = torch.nn.functional.softplus(s[:, :R] @ w[p + "dt"].T + w[p + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(w[p + "A_log"]), s[:, R:R + N], s[:, R + N:], w[p + "D"])
    return (y * silu(z)) @ w[p + "o"].T


def clamped_glu(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(ALPHA * g) * (u + 1.0)) @ w[p + "down"].T


def silu_glu(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def routed_experts(h, f, w, p, choice=None):
    """The top experts by router logit, weighed by the softmax over the chosen logits, plus the
    shared expert. `choice` (a list) collects the logits for tests that avoid close calls."""
    top = f["router"]["top"]
    z = h @ w[p + "router"].T
    if choice is not None:
        choice.append(z)
    val, idx = z.topk(top, -1)
    wt = torch.softmax(val, -1)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for n, e in enumerate(idx[t].tolist()):
            y[t] += wt[t, n] * clamped_glu(h[t:t + 1], w, p + f"e{e}.", f["expert"]["limit"])[0]
    if f.get("shared"):
        y = y + clamped_glu(h, w, p + "shared.", f["shared"]["limit"])
    return y


MIXERS = {"attention": pooled_attention, "parallel": side_by_side, "mamba1": mamba_mixer}


def forward(cfg, weights, tokens, layers_out=None, choice=None):
    """logits [T, vocab] of one sequence; layers_out (a list) collects the residual after every layer."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[L["type"]](rms_norm(x, w[p + "norm1"], eps), L["mixer"], w, p + "mix.", eps)
        x = x + rms_norm(y, w[p + "norm1b"], eps)
        f = L["mlp"]
        if f:
            h = rms_norm(x, w[p + "norm2"], eps)
            y = silu_glu(h, w, p + "mlp.") if f["kind"] == "dense" else routed_experts(h, f, w, p + "mlp.", choice)
            x = x + rms_norm(y, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T


def greedy(cfg, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, weights, toks)[-1].argmax()))
    return toks[len(prompt):]
