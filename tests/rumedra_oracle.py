"""A plain, slow float64 implementation of the Rumedra design, one function per mechanism, written
from the design's equations and sharing no code with the package: whole sequences at once, dense
score matrices, explicit masks, explicit token loops, no cache. Tests build configurations and
random weights here."""
import math

import torch

F64 = torch.float64


# ---- configuration builders ----------------------------------------------------------------
def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, groups=(1, 1), identity=0, scale=1.0, shared=None):
    """groups: (count, kept) over experts and identity experts; shared: the shared expert's width."""
    f = {"kind": "moe", "expert": {"ff": ff},
         "router": {"experts": experts, "top": top, "groups": {"count": groups[0], "keep": groups[1]},
                    "identity": identity, "scale": scale}}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def parallel_layer(left, right, left_scale, right_scale, mlp):
    """left: (heads, kv_heads, dim, vdim, scale, window, rot), right: (dim, vdim, decays, rot) with rot =
    (dims, base[, (factor, low, high, original)])."""
    def rotation(r):
        d = {"dims": r[0], "base": r[1]}
        if len(r) > 2:
            d["scaling"] = dict(zip(("factor", "low", "high", "original"), r[2]))
        return d

    h, g, d, dv, sc, win, rot = left
    rd, rdv, decay, rrot = right
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": {"heads": h, "kv_heads": g, "dim": d, "vdim": dv, "scale": sc, "mask": {"size": win},
                               "rot": rotation(rot)},
                      "left_scale": left_scale,
                      "right": {"heads": len(decay), "dim": rd, "vdim": rdv, "decay": list(decay), "rot": rotation(rrot)},
                      "right_scale": right_scale}}


def hgrn_layer(heads, dim, vdim, mlp):
    return {"type": "hgrn2", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def config(layers, width, vocab, eps, scale):
    return {"architecture": "Rumedra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


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
        mat(p + "down", W, ff, 1.5 / math.sqrt(ff))

    mat("embed", cfg["vocab"], W, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        for n in ("norm1",) + (("norm2",) if L["mlp"] else ()):
            vec(p + n, W, 1.0, 0.2)
        x = p + "mix."
        if L["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                mat(x + "left." + n, rows, W)
                vec(x + f"left.{n}.b", rows, 0.0, 0.5)
            mat(x + "left.g", H * Dv, W)
            mat(x + "left.o", W, H * Dv, 1.5 / math.sqrt(H * Dv))
            H, D, Dv = r["heads"], r["dim"], r["vdim"]
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * Dv), ("g", H * Dv)):
                mat(x + "right." + n, rows, W)
            mat(x + "right.o", W, H * Dv, 1.5 / math.sqrt(H * Dv))
        else:
            H, D, Dv = m["heads"], m["dim"], m["vdim"]
            mat(x + "q", H * D, W)
            mat(x + "f", H * D, W)
            vec(x + "f.b", H * D, 1.0, 1.0)
            out[x + "lower"] = (torch.rand(H * D, generator=g) * 0.9).to(torch.bfloat16)
            mat(x + "v", H * Dv, W)
            vec(x + "norm", Dv, 1.0, 0.2)
            mat(x + "o", W, H * Dv, 1.5 / math.sqrt(H * Dv))
        f = L["mlp"]
        if f and f["kind"] == "dense":
            glu(p + "mlp.", f["ff"])
        elif f:
            n = f["router"]["experts"] + f["router"].get("identity", 0)
            mat(p + "mlp.router", n, W)
            vec(p + "mlp.correction", n, -0.05, 0.2)
            for e in range(f["router"]["experts"]):
                glu(p + f"mlp.e{e}.", f["expert"]["ff"])
            if f.get("shared"):
                glu(p + "mlp.shared.", f["shared"]["ff"])
    vec("final.norm", W, 1.0, 0.2)
    return out


# ---- mechanisms ------------------------------------------------------------------------------
def rms_norm(x, w, eps):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def silu(x):
    return x * torch.sigmoid(x)


def frequencies(rot):
    """Angular frequencies of the rotated pairs; with rot.scaling, long wavelengths are stretched by
    `factor`, short ones are kept, and between the two bounds the two are blended."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        s = rot.get("scaling")
        if s:
            wave = 2.0 * math.pi / f
            if wave > s["original"] / s["low"]:
                f = f / s["factor"]
            elif wave >= s["original"] / s["high"]:
                mix = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
                f = (1.0 - mix) * f / s["factor"] + mix * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate_half(x, rot, first=0):
    """x [T, H, D] at positions first .. first + T - 1: dimension i turns with dimension i + dims / 2."""
    n = rot["dims"] // 2
    y = x.clone()
    ang = (first + torch.arange(x.shape[0], dtype=F64))[:, None, None] * frequencies(rot)
    u, v = x[..., :n], x[..., n:2 * n]
    y[..., :n] = u * torch.cos(ang) - v * torch.sin(ang)
    y[..., n:2 * n] = v * torch.cos(ang) + u * torch.sin(ang)
    return y


def visible(T, window):
    """[T, T] bool: row i sees column j when 0 <= i - j < window."""
    dist = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (dist >= 0) & (dist < window)


def window_softmax_attention(q, k, v, scale, window):
    """q [T, H, D], k [T, G, D], v [T, G, Dv] -> [T, H, Dv]."""
    T, H, _ = q.shape
    G = k.shape[1]
    seen = visible(T, window)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(~seen, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def rotated_window_attention(h, a, w, p):
    T, H, G, D, Dv = h.shape[0], a["heads"], a["kv_heads"], a["dim"], a["vdim"]
    q = rotate_half((h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, D), a["rot"])
    k = rotate_half((h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, D), a["rot"])
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, Dv)
    o = window_softmax_attention(q, k, v, a["scale"], a["mask"]["size"]).reshape(T, H * Dv)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


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


def retention(h, r, w, p, eps):
    T, H, D, Dv = h.shape[0], r["heads"], r["dim"], r["vdim"]
    q = rotate_half((h @ w[p + "q"].T).view(T, H, D), r["rot"])
    k = rotate_half((h @ w[p + "k"].T).view(T, H, D), r["rot"]) * D ** -0.5
    o = decayed_linear_attention(q, k, (h @ w[p + "v"].T).view(T, H, Dv), r["decay"])
    o = rms_norm(o, None, eps).reshape(T, H * Dv)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel_mixer(h, m, w, p, eps):
    left = rotated_window_attention(h, m["left"], w, p + "left.")
    right = retention(h, m["right"], w, p + "right.", eps)
    return m["left_scale"] * left + m["right_scale"] * right


def gated_linear_attention(q, f, v):
    """q, f [T, H, D], v [T, H, Dv]: S <- diag(f) S + (1 - f) v^T, o = S^T q, S = 0 at the start."""
    T, H, D = q.shape
    o = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        S = torch.zeros(D, v.shape[2], dtype=F64)
        for t in range(T):
            S = f[t, h][:, None] * S + torch.outer(1.0 - f[t, h], v[t, h])
            o[t, h] = q[t, h] @ S
    return o


def forget_gate(z, bias, lower):
    return lower + (1.0 - lower) * torch.sigmoid(z + bias)


def hgrn_mixer(h, m, w, p, eps):
    T, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    f = forget_gate(h @ w[p + "f"].T, w[p + "f.b"], w[p + "lower"])
    o = gated_linear_attention(silu(h @ w[p + "q"].T).view(T, H, D), f.view(T, H, D), (h @ w[p + "v"].T).view(T, H, Dv))
    return rms_norm(o, w[p + "norm"], eps).reshape(T, H * Dv) @ w[p + "o"].T


def glu(h, w, p, act):
    return (act(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def group_mask(c, count, keep):
    """c [n] choice scores -> bool [n]: the members of the `keep` groups with the largest best score."""
    n = c.shape[0]
    size = n // count
    best = torch.stack([c[g * size:(g + 1) * size].max() for g in range(count)])
    ok = torch.zeros(n, dtype=torch.bool)
    for g in best.topk(keep).indices.tolist():
        ok[g * size:(g + 1) * size] = True
    return ok


def router(h, f, w, p, choice=None):
    """-> per token the chosen indices [T, top] and their weights. `choice` (a list) collects, per token, how
    close the choice was (the smallest gap between what was taken and what was left, groups included)."""
    r = f["router"]
    top, grp = r["top"], r.get("groups") or {"count": 1, "keep": 1}
    s = torch.softmax(h @ w[p + "router"].T, -1)
    c = s + w[p + "correction"]
    T, n = s.shape
    ids = torch.zeros(T, top, dtype=torch.long)
    wt = torch.zeros(T, top, dtype=F64)
    margin = torch.full((T,), math.inf, dtype=F64)
    for t in range(T):
        ok = group_mask(c[t], grp["count"], grp["keep"])
        order = c[t].masked_fill(~ok, -math.inf).sort(descending=True)
        ids[t] = order.indices[:top]
        if top < int(ok.sum()):
            margin[t] = order.values[top - 1] - order.values[top]
        if grp["keep"] < grp["count"]:
            best = c[t].view(grp["count"], -1).max(-1).values.sort(descending=True).values
            margin[t] = min(margin[t], best[grp["keep"] - 1] - best[grp["keep"]])
        pick = s[t][ids[t]]
        wt[t] = pick / (pick.sum() + 1e-20) * r.get("scale", 1.0)
    if choice is not None:
        choice.append(margin)
    return ids, wt


def routed_experts(h, f, w, p, choice=None):
    """Outputs past the last expert's index are the input itself."""
    ids, wt = router(h, f, w, p, choice)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for n, e in enumerate(ids[t].tolist()):
            one = h[t] if e >= f["router"]["experts"] else glu(h[t:t + 1], w, p + f"e{e}.", silu)[0]
            y[t] += wt[t, n] * one
    if f.get("shared"):
        y = y + glu(h, w, p + "shared.", silu)
    return y


MIXERS = {"parallel": parallel_mixer, "hgrn2": hgrn_mixer}


def forward(cfg, weights, tokens, layers_out=None, choice=None):
    """logits [T, vocab] of one sequence; layers_out (a list) collects the residual after every layer."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + MIXERS[L["type"]](rms_norm(x, w[p + "norm1"], eps), L["mixer"], w, p + "mix.", eps)
        f = L["mlp"]
        if f:
            h = rms_norm(x, w[p + "norm2"], eps)
            x = x + (glu(h, w, p + "mlp.", torch.relu) if f["kind"] == "dense" else
                     routed_experts(h, f, w, p + "mlp.", choice))
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T


def greedy(cfg, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, weights, toks)[-1].argmax()))
    return toks[len(prompt):]
