"""Plain, slow CPU implementation of the mechanisms of the latent-attention decoder design (test infrastructure only).

One function per mechanism, written from the equations, in float64 by default; nothing is shared with the product code.
Shapes: a sequence is [T, ...]; `pos` is the absolute position of its first row.

    bigram row       (a * before + b * token) mod n;  n for the first token of a sequence
    inverse freqs    w_i = base^(-2i / n);  YaRN: w_i / F where a wave turns less than `slow` times over the original length, w_i
                     where it turns more than `fast` times, a linear ramp between the two (rounded) indexes; amplitude 1 + ln(F) / 10
    rotate           (x_2i + j x_2i+1) * amplitude * e^(j pos w_i)
    latent keys      c = rms(first rows of D h) * w,  r = rotate(the other rows of D h): what a cache holds of a token
    latent attention s_ts = (qn_t . (K c_s) + rotate(qr_t) . r_s) * scale, softmax over s <= t, o_t = sum_s p_ts (V c_s);  per head
    head gate        o * sigmoid(G h)
    gated MLP        down (gelu(gate h) * (up h)),  gelu in its tanh form
    parallel layer   x + (mixer(n) + mlp(n)),  n = rms(x) * w
    softcap          cap * tanh(z / cap)
"""
import math

import torch

from .layered_ref import rms


def bigram_rows(tokens, before, mul_before, mul_token, buckets):
    """Row per token; `before` is the token ahead of the first one, None at the start of a sequence."""
    rows, prev = [], before
    for t in tokens.tolist():
        rows.append(buckets if prev is None else (prev * mul_before + t * mul_token) % buckets)
        prev = t
    return torch.tensor(rows, dtype=torch.long)


def inverse_freqs(rot):
    """(w [dims / 2] float64, amplitude)"""
    n, base = rot["dims"], float(rot["base"])
    w = [base ** (-2.0 * i / n) for i in range(n // 2)]
    s = rot.get("scaling")
    if not s:
        return torch.tensor(w, dtype=torch.float64), 1.0

    def index_of(turns):
        return n * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(index_of(s["fast"])), 0), min(math.ceil(index_of(s["slow"])), n - 1)
    out = []
    for i, f in enumerate(w):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1 - ramp))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, rot, pos):
    """x [T, ..., n]: neighbouring pairs of the first rot.dims elements turn by position * frequency."""
    w, amp = inverse_freqs(rot)
    ang = torch.arange(pos, pos + x.shape[0], dtype=torch.float64).view(-1, *[1] * (x.dim() - 1)) * w
    c, s = (ang.cos() * amp).to(x.dtype), (ang.sin() * amp).to(x.dtype)
    y = x.clone()
    n = rot["dims"]
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y[..., 0:n:2], y[..., 1:n:2] = u * c - v * s, v * c + u * s
    return y


def latent_keys(d, w, kv_rank, rot, eps, pos):
    """d [n, kv_rank + rot_dim] projection rows -> (latents [n, kv_rank], rotated key parts [n, rot_dim])"""
    return rms(d[:, :kv_rank], eps) * w, rotate(d[:, kv_rank:], rot, pos)


def latent_attention(q, c, r, wk, wv, heads, dim, vdim, rot, scale, pos):
    """q [n, heads * (dim + rot_dim)] rows at pos..; c [T, kv_rank], r [T, rot_dim] of the positions 0..T-1;
    wk [heads * dim, kv_rank], wv [heads * vdim, kv_rank] -> [n, heads, vdim]"""
    n, T, rd = q.shape[0], c.shape[0], r.shape[1]
    q = q.view(n, heads, dim + rd)
    qr = rotate(q[..., dim:], rot, pos)
    seen = torch.arange(T).view(1, -1) <= torch.arange(pos, pos + n).view(-1, 1)
    out = torch.zeros(n, heads, vdim, dtype=q.dtype)
    for h in range(heads):
        k, v = c @ wk[h * dim:(h + 1) * dim].T, c @ wv[h * vdim:(h + 1) * vdim].T
        s = (q[:, h, :dim] @ k.T + qr[:, h] @ r.T) * scale
        out[:, h] = torch.softmax(s.masked_fill(~seen, float("-inf")), -1) @ v
    return out


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def gated_mlp(h, gate, up, down):
    return (gelu_tanh(h @ gate.T) * (h @ up.T)) @ down.T


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


class LatentRefModel:
    """The whole decoder over one sequence; portions go through a state (last token, latents and rotated key parts)."""

    GATED = ("latent_attention",)

    def __init__(self, cfg, tensors, dtype=torch.float64):
        self.cfg, self.dtype = cfg, dtype
        self.t = {k: v.to(dtype) for k, v in tensors.items()}

    def new_state(self):
        return {"n": 0, "last": None, "kv": [None] * len(self.cfg["layers"])}

    def mixer(self, i, h, st):
        L, t, eps, p = self.cfg["layers"][i], self.t, self.cfg["norm"]["eps"], f"l{i}.mix."
        m, pos = L["mixer"], st["n"]
        q = (rms(h @ t[p + "dq"].T, eps) * t[p + "dq.norm"]) @ t[p + "uq"].T
        src = m.get("kv_from")
        if src is None:
            c, r = latent_keys(h @ t[p + "dkv"].T, t[p + "dkv.norm"], m["kv_rank"], m["rot"], eps, pos)
            if st["kv"][i] is not None:
                c, r = torch.cat([st["kv"][i][0], c]), torch.cat([st["kv"][i][1], r])
            st["kv"][i] = (c, r)
        else:
            c, r = st["kv"][src]
        o = latent_attention(q, c, r, t[p + "uk"], t[p + "uv"], m["heads"], m["dim"], m["vdim"], m["rot"], m["scale"], pos)
        if L["type"] in self.GATED:
            o = o * torch.sigmoid(h @ t[p + "g"].T).unsqueeze(-1)
        return o.flatten(1) @ t[p + "o"].T

    def step(self, tokens, st, layers_out=None):
        """tokens [n] int64 -> logits [n, vocab]; advances `st`."""
        c, t = self.cfg, self.t
        eps, b = c["norm"]["eps"], c["embedding"]["bigram"]
        rows = bigram_rows(tokens, st["last"], b["mul_prev"], b["mul_cur"], b["buckets"])
        x = rms(t["embed"][tokens] + t["bigram"][rows], eps) * t["embed.norm"]
        for i, L in enumerate(c["layers"]):
            p = f"l{i}."
            h = rms(x, eps) * t[p + "norm1"]
            y = self.mixer(i, h, st)
            if L["mlp"] is not None:
                y = y + gated_mlp(h, t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"])
            x = x + y
            if layers_out is not None:
                layers_out.append(x.clone())
        st["n"] += len(tokens)
        st["last"] = int(tokens[-1])
        return softcap((rms(x, eps) * t["final.norm"]) @ t["embed"].T, c["logit_softcap"])

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
