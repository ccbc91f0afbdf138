"""Plain, slow CPU implementation of the mechanisms of the layered decoder designs (test infrastructure only).

One function per mechanism, written from the equations, in float64 by default; nothing is shared with the product code.
Shapes: a sequence is [T, ...]; `pos` is the absolute position of its first row.

    embed            x_t = E[token_t] * scale + P[t]
    rms              x / sqrt(mean(x^2) + eps)                     (weighted: * w)
    token_shift      h_t + (h_{t-1} - h_t) * mu,  h_{-1} = 0
    attention        E_ts = exp(scale <rms(q_t), rms(k_s)> - a ln(1 + c (t - s))) for c0(t) <= s <= t, c0 = first position of
                     t's chunk;   o_t = sum_s E_ts v_s / (1 + sum_s E_ts)
    xielu            z / 2 + A z^2 on the right of 0, z / 2 + B (expm1(z) - z) on the left; A, B - 1/2 = softplus of the two numbers
    head             rms(x) w . head^T * logit_scale
"""
import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def embed(table, tokens, scale, pos_table, pos):
    return table[tokens] * scale + pos_table[pos:pos + tokens.shape[0]]


def token_shift(h, mu, before=None):
    """`before`: the last unshifted h of the preceding portion; zeros at the start of a sequence."""
    first = torch.zeros_like(h[:1]) if before is None else before.view(1, -1)
    prev = torch.cat([first, h[:-1]], 0)
    return h + (prev - h) * mu


def distance_bias(r1, r2, dist):
    return r1 * torch.log(1 + r2 * dist)


def sink_softmax(s):
    """Softmax over the last axis with one more score of 0 in the denominator; -inf scores are unseen."""
    m = torch.clamp(s.amax(-1, keepdim=True), min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attention(q, k, v, r1, r2, scale, chunk, eps, qpos=0):
    """q [n, H, D] rows at positions qpos..qpos+n-1; k [T, G, D], v [T, G, VD] rows at 0..T-1.  -> [n, H, VD]"""
    n, H, _ = q.shape
    T, G = k.shape[0], k.shape[1]
    qn, kn = rms(q, eps), rms(k, eps)
    i = torch.arange(qpos, qpos + n).view(-1, 1)
    j = torch.arange(T).view(1, -1)
    seen = (j <= i) & (i // chunk == j // chunk)
    dist = (i - j).clamp(min=0).to(q.dtype)
    out = torch.zeros(n, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (qn[:, h] @ kn[:, g].T) * scale - distance_bias(r1[h], r2[h], dist)
        s = s.masked_fill(~seen, float("-inf"))
        out[:, h] = sink_softmax(s) @ v[:, g]
    return out


def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def xielu(z, p, q):
    pos = softplus(p) * z * z + z / 2
    zn = z.clamp(max=0)
    neg = (0.5 + softplus(q)) * (torch.expm1(zn) - zn) + z / 2
    return torch.where(z > 0, pos, neg)


class RefModel:
    """The whole decoder over one sequence; portions go through `State` (keys, values and last unshifted rows)."""

    def __init__(self, cfg, tensors, dtype=torch.float64):
        self.cfg, self.dtype = cfg, dtype
        self.t = {k: v.to(dtype) for k, v in tensors.items()}

    def new_state(self):
        return {"n": 0, "kv": [None] * len(self.cfg["layers"]), "h": [None] * len(self.cfg["layers"])}

    def step(self, tokens, st, layers_out=None):
        """tokens [n] int64 -> logits [n, vocab]; advances `st`."""
        c, t = self.cfg, self.t
        eps = c["norm"]["eps"]
        pos, n = st["n"], len(tokens)
        x = embed(t["embed"], tokens, c["embedding"]["scale"], t["pos"], pos)
        for i, L in enumerate(c["layers"]):
            p, m = f"l{i}.", L["mixer"]
            h = rms(x, eps) * t[p + "norm1"]
            y = token_shift(h, t[p + "shift"], st["h"][i])
            st["h"][i] = h[-1].clone()
            H, G, D, VD = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            q = (y @ t[p + "mix.q"].T).view(n, H, D)
            k = (y @ t[p + "mix.k"].T).view(n, G, D)
            v = (y @ t[p + "mix.v"].T).view(n, G, VD)
            if st["kv"][i] is not None:
                k = torch.cat([st["kv"][i][0], k])
                v = torch.cat([st["kv"][i][1], v])
            st["kv"][i] = (k, v)
            o = attention(q, k, v, t[p + "mix.r1"], t[p + "mix.r2"], m["scale"], m["mask"]["size"], eps, pos)
            x = x + o.reshape(n, H * VD) @ t[p + "mix.o"].T
            if L["mlp"] is not None:
                h = rms(x, eps) * t[p + "norm2"]
                a = xielu(h @ t[p + "mlp.up"].T, t[p + "mlp.act"][0], t[p + "mlp.act"][1])
                x = x + a @ t[p + "mlp.down"].T
            if layers_out is not None:
                layers_out.append(x.clone())
        st["n"] = pos + n
        return (rms(x, eps) * t["final.norm"]) @ t["head"].T * c["logit_scale"]

    def logits(self, tokens):
        return self.step(torch.as_tensor(tokens, dtype=torch.long), self.new_state())

    def greedy(self, prompt, n_new):
        """(tokens, per-step gap between the best and the second best logit)."""
        st = self.new_state()
        lg = self.step(torch.as_tensor(prompt, dtype=torch.long), st)[-1]
        out, gaps = [], []
        for _ in range(n_new):
            top = torch.topk(lg, 2).values
            gaps.append(float(top[0] - top[1]))
            out.append(int(lg.argmax()))
            lg = self.step(torch.tensor(out[-1:]), st)[-1]
        return out, gaps
