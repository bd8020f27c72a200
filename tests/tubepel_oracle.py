"""A plain, slow float64 implementation of the Tubepel equations, one function
per mechanism, sharing no code with the package. It works on whole sequences
(no cache, no batching, no portions) and is the yardstick for the engine in
tests/test_tubepel.py. It also makes small configurations and random
checkpoints.

Notation: h [T, W] is a sublayer's input, weights are [out, in], `w` maps
checkpoint tensor names to float64 tensors (already rounded to bf16, which is
how they are stored).

The design: the residual is a bundle of S streams X [S, T, W], all equal to
embed[token] at first. A sublayer (a mixer or a feed-forward) reads a weighted
sum of the streams and its result is written back to all of them while they
are mixed:
    y = sub(n(sum_s a_s X_s));    X'_t = sum_s M_st X_s + b_t y,
n an RMS norm with a plain weight. The mixer is one of
  * latent attention: normed query latent, keys and values from one normed
    latent, one rotated key part shared by all heads; the rotation pairs
    neighbours (2i, 2i+1) in one kind of layer and (i, i + d/2) in the other;
  * windowed grouped-query attention with kept first tokens, a learned sink
    per head in the softmax denominator and an elementwise sigmoid gate.
The feed-forward is down(relu(up h)^2), or routed SwiGLU experts: sigmoid
scores, the best `top`, each expert reads score * h; plus a shared expert. A
run of layers may be passed several times with the same weights. Logits =
head . n_final(sum of the streams).
"""

import json
import math
import os

import torch

F64 = torch.float64


# ---------------------------------------------------------------- pieces ----

def rms(x, w, eps):
    return x / ((x * x).mean(-1, keepdim=True) + eps).sqrt() * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def relu_squared(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def bundle_read(X, a):
    """X [S, T, W], a [S]: what a sublayer reads."""
    return torch.einsum("s,stw->tw", a, X)


def bundle_write(X, M, b, y):
    """M [from, to], b [to]: the bundle after a sublayer whose result is y."""
    return torch.einsum("so,stw->otw", M, X) + b[:, None, None] * y


def turn(x, rot, neighbours):
    """x [T, n] at positions 0..T-1; the first rot.dims dimensions turn in
    pairs, (2i, 2i+1) with `neighbours`, else (i, i + dims/2)."""
    d = int((rot or {}).get("dims", 0))
    if not d:
        return x
    out = x.clone()
    for i in range(d // 2):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + d // 2)
        ang = torch.arange(x.shape[0], dtype=F64) \
            * float(rot["base"]) ** (-2.0 * i / d)
        c, s = ang.cos(), ang.sin()
        out[:, a] = x[:, a] * c - x[:, b] * s
        out[:, b] = x[:, b] * c + x[:, a] * s
    return out


def sees(T, window=0, keep=0):
    """[T, T] bool: query row i sees key column j."""
    i, j = torch.arange(T).unsqueeze(1), torch.arange(T).unsqueeze(0)
    ok = j <= i
    if window:
        ok = ok & ((i - j < window) | (j < keep))
    return ok


def attend(q, k, v, scale, mask, sink=None):
    """Softmax attention of one head; `sink` is a score without key or value."""
    s = ((q @ k.T) * scale).masked_fill(~mask, -math.inf)
    top = s.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, torch.as_tensor(float(sink), dtype=F64))
    e = torch.exp(s - top)
    z = e.sum(-1, keepdim=True)
    if sink is not None:
        z = z + torch.exp(float(sink) - top)
    return (e / z) @ v


# ---------------------------------------------------------------- mixers ----

def latent_mixer(h, w, p, mc, eps, neighbours):
    H, dk, dr, dv, R = (mc[n] for n in ("heads", "dim", "rot_dim", "vdim",
                                        "kv_rank"))
    cq = rms(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).view(-1, H, dk + dr)
    both = h @ w[p + "dkv"].T
    c = rms(both[:, :R], w[p + "dkv.norm"], eps)
    shared = turn(both[:, R:], mc["rot"], neighbours)
    k = (c @ w[p + "uk"].T).view(-1, H, dk)
    v = (c @ w[p + "uv"].T).view(-1, H, dv)
    mask = sees(h.shape[0])
    heads = [attend(torch.cat([q[:, a, :dk],
                               turn(q[:, a, dk:], mc["rot"], neighbours)], 1),
                    torch.cat([k[:, a], shared], 1), v[:, a],
                    float(mc["scale"]), mask) for a in range(H)]
    return torch.cat(heads, 1) @ w[p + "o"].T


def window_mixer(h, w, p, mc):
    H, G, dk, dv = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    q, k, v = (h @ w[p + n].T for n in "qkv")
    m = mc.get("mask") or {}
    mask = sees(h.shape[0], m.get("size", 0), m.get("keep_first", 0))
    heads = []
    for a in range(H):
        g = a * G // H
        heads.append(attend(
            turn(q[:, a * dk:(a + 1) * dk], mc.get("rot"), False),
            turn(k[:, g * dk:(g + 1) * dk], mc.get("rot"), False),
            v[:, g * dv:(g + 1) * dv], float(mc["scale"]), mask,
            sink=w[p + "sink"][a]))
    return (torch.cat(heads, 1) * torch.sigmoid(h @ w[p + "g"].T)) \
        @ w[p + "o"].T


def mixer(kind, h, w, p, mc, eps):
    if kind == "attention":
        return window_mixer(h, w, p, mc)
    return latent_mixer(h, w, p, mc, eps, {"latent_attention": True,
                                           "latent_attention_2": False}[kind])


# ----------------------------------------------------------- feed-forwards ---

def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def routed(h, w, p, fc):
    """Each token's best experts read score * h; results are summed."""
    score = torch.sigmoid(h @ w[p + "router"].T)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in score[t].argsort(descending=True, stable=True)[
                :fc["router"]["top"]].tolist():
            out[t] += expert(score[t, e] * h[t:t + 1], w, f"{p}e{e}.")[0]
    if fc.get("shared"):
        out = out + expert(h, w, p + "shared.")
    return out


def feed_forward(h, w, p, fc):
    if fc["kind"] == "dense":
        return relu_squared(h @ w[p + "up"].T) @ w[p + "down"].T
    return routed(h, w, p, fc)


# ----------------------------------------------------------------- model ----

def layer_order(config):
    """Layer indices in the order they run."""
    n, lp = len(config["layers"]), config.get("loop")
    if not lp:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def forward(config, w, tokens, streams=None):
    """Logits [T, vocab] of one whole sequence. `streams`, when a list,
    receives the sum of the bundle after every layer run."""
    eps = float(config["norm"]["eps"])
    X = w["embed"][torch.as_tensor(tokens, dtype=torch.long)].expand(
        config["streams"], -1, -1)
    for i in layer_order(config):
        lc, lp = config["layers"][i], f"l{i}."
        subs = [("hc1.", "norm1", lambda h: mixer(
            lc["type"], h, w, lp + "mix.", lc["mixer"], eps))]
        if lc.get("mlp"):
            subs.append(("hc2.", "norm2", lambda h: feed_forward(
                h, w, lp + "mlp.", lc["mlp"])))
        for hc, norm, fn in subs:
            y = fn(rms(bundle_read(X, w[lp + hc + "in"]), w[lp + norm], eps))
            X = bundle_write(X, w[lp + hc + "mix"], w[lp + hc + "out"], y)
        if streams is not None:
            streams.append(X.sum(0))
    return rms(X.sum(0), w["final.norm"], eps) @ w["head"].T


# ------------------------------------------------- configs and checkpoints ----

def latent_cfg(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale=None,
               base=10000.0):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
            "q_rank": q_rank, "kv_rank": kv_rank,
            "scale": (dim + rot_dim) ** -0.5 if scale is None else scale,
            "rot": {"dims": rot_dim, "base": base}}


def attn_cfg(heads, kv_heads, dim, vdim, window, keep, rot_dims, scale=None,
             base=10000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": dim ** -0.5 if scale is None else scale,
            "rot": {"dims": rot_dims, "base": base},
            "mask": {"size": window, "keep_first": keep}}


def dense_cfg(ff):
    return {"kind": "dense", "ff": ff}


def moe_cfg(ff, experts, top, shared_ff=0):
    m = {"kind": "moe", "expert": {"ff": ff},
         "router": {"experts": experts, "top": top}}
    if shared_ff:
        m["shared"] = {"ff": shared_ff}
    return m


def layer(kind, mixer_cfg, mlp=None):
    return json.loads(json.dumps({"type": kind, "mixer": mixer_cfg,
                                  "mlp": mlp}))


def make_config(width, vocab, layers, streams=2, loop=None, eps=1e-5):
    cfg = {"architecture": "Tubepel", "width": width, "vocab": vocab,
           "streams": streams, "norm": {"eps": eps}, "layers": layers}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def make_weights(config, seed=0):
    """Random weights (already rounded to bf16) under checkpoint names.

    Which experts a token uses must not hang on rounding, or bf16 runs could
    not be compared: the first columns (one per expert) are written by no
    sublayer, every token's embedding holds well separated numbers there in an
    order of its own, and router row e looks at column e alone. The scores
    still depend on everything that scales the normed input."""
    g = torch.Generator().manual_seed(seed)
    W, S = config["width"], config["streams"]
    w = {}

    def rnd(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=g) * std + mean

    def lin(out, inn, gain=1.0):
        return rnd(out, inn, std=gain * inn ** -0.5)

    def swi(p, ff):
        w[p + "gate"], w[p + "up"] = lin(ff, W), lin(ff, W)
        w[p + "down"] = lin(W, ff)

    w["embed"], w["head"] = rnd(config["vocab"], W), lin(config["vocab"], W)
    E = max([(lc.get("mlp") or {}).get("router", {}).get("experts", 0)
             for lc in config["layers"]])
    if E:
        levels = torch.linspace(-1.5, 1.5, E)
        for t in range(config["vocab"]):
            w["embed"][t, :E] = levels[torch.randperm(E, generator=g)]
    w["final.norm"] = rnd(W, std=0.2, mean=1.0)
    for i, lc in enumerate(config["layers"]):
        lp, mc, fc = f"l{i}.", lc["mixer"], lc.get("mlp")
        p = lp + "mix."
        for q in ("1", "2") if fc else ("1",):
            w[lp + "norm" + q] = rnd(W, std=0.2, mean=1.0)
            hc = lp + f"hc{q}."
            w[hc + "in"] = rnd(S, std=0.3, mean=1.0 / S)
            w[hc + "out"] = rnd(S, std=0.4, mean=0.7)
            # far from symmetric, so that [from, to] and [to, from] differ
            w[hc + "mix"] = 0.75 * torch.eye(S) + rnd(S, S, std=0.3)
        H, dk, dv = mc["heads"], mc["dim"], mc["vdim"]
        if lc["type"] == "attention":
            G = mc["kv_heads"]
            w[p + "q"], w[p + "k"] = lin(H * dk, W), lin(G * dk, W)
            w[p + "v"], w[p + "g"] = lin(G * dv, W), lin(H * dv, W, 2.0)
            w[p + "sink"] = rnd(H, std=1.0, mean=1.0)
        else:
            R, Q, dr = mc["kv_rank"], mc["q_rank"], mc["rot_dim"]
            w[p + "dq"], w[p + "dq.norm"] = lin(Q, W), rnd(Q, std=0.2, mean=1.0)
            w[p + "uq"] = lin(H * (dk + dr), Q)
            w[p + "dkv"] = lin(R + dr, W)
            w[p + "dkv.norm"] = rnd(R, std=0.2, mean=1.0)
            w[p + "uk"], w[p + "uv"] = lin(H * dk, R), lin(H * dv, R)
        w[p + "o"] = lin(W, H * dv)
        if fc is None:
            continue
        m = lp + "mlp."
        if fc["kind"] == "dense":
            w[m + "up"], w[m + "down"] = lin(fc["ff"], W), lin(W, fc["ff"])
            continue
        n = fc["router"]["experts"]
        w[lp + "norm2"][:E] = 1.0
        w[m + "router"] = torch.zeros(n, W)
        w[m + "router"][:, :n] = 1.5 * torch.eye(n)
        for e in range(fc["router"]["experts"]):
            swi(f"{m}e{e}.", fc["expert"]["ff"])
        if fc.get("shared"):
            swi(m + "shared.", fc["shared"]["ff"])
    for k, v in w.items():
        if k.endswith((".o", ".down")):
            v[:E] = 0.0
    return {k: v.to(torch.bfloat16).to(F64) for k, v in w.items()}


def save_checkpoint(path, config, w):
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in w.items()},
              os.path.join(path, "model.safetensors"))
    return path
