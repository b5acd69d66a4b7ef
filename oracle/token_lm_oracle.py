"""Plain numpy restatement of the token language models (moshi_amd/tlm.py), float64, one function per mechanism, whole sequences at
once: no cache, no state hand-over, no batching.  For tests only - it shares no code with the engine and reads the same state dict.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import numpy as np

from moshi_amd.config import (ChannelDeltaConfig, DenseGLUConfig, GroupedAttentionConfig, LatentAttentionConfig, LightningConfig, MinGRUConfig,
                              MoEConfig, TokenLMConfig)


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def rms_norm(x, w, eps: float, groups: int = 1):
    """x [T, D] cut into equal groups; each is divided by its own root mean square."""
    T, D = x.shape
    g = x.reshape(T, groups, D // groups)
    return (g / np.sqrt(np.mean(g * g, axis=2, keepdims=True) + eps)).reshape(T, D) * w


def rotate(x, positions, base: float):
    """Rotary positions, halves paired: x [T, ..., R], partner of i is i + R / 2."""
    R = x.shape[-1]
    half = R // 2
    angle = positions.astype(np.float64)[:, None] * base ** (-np.arange(half) * 2.0 / R)
    angle = angle.reshape((len(positions),) + (1,) * (x.ndim - 2) + (half,))
    c, s = np.cos(angle), np.sin(angle)
    a, b = x[..., :half], x[..., half:]
    return np.concatenate([a * c - b * s, b * c + a * s], axis=-1)


def window_mask(T: int, window: int):
    """[query, key]: key no later than the query and fewer than `window` positions behind it (0: no limit)."""
    dist = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (dist >= 0) & ((dist < window) if window > 0 else True)


def latent_attention(w: Dict[str, np.ndarray], p: str, m: LatentAttentionConfig, h, eps: float):
    T, H = h.shape[0], m.heads
    pos = np.arange(T)
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(T, H, m.dim + m.rot_dim)
    down = h @ w[p + "dkv"].T
    latent = rms_norm(down[:, :m.kv_rank], w[p + "dkv.norm"], eps)
    k = (latent @ w[p + "uk"].T).reshape(T, H, m.dim)
    v = (latent @ w[p + "uv"].T).reshape(T, H, m.vdim)
    gate = sigmoid(h @ w[p + "g"].T)
    seen = window_mask(T, m.window)
    qr, kr = q[:, :, m.dim:], down[:, m.kv_rank:]
    if m.rot_dim:
        qr, kr = rotate(qr, pos, m.rot_base), rotate(kr, pos, m.rot_base)
    out = np.zeros((T, H, m.vdim))
    for head in range(H):
        score = (q[:, head, :m.dim] @ k[:, head].T + qr[:, head] @ kr.T) * m.scale
        score = np.where(seen, score, -np.inf)
        weight = np.exp(score - score.max(axis=1, keepdims=True))
        weight /= weight.sum(axis=1, keepdims=True)
        out[:, head] = (weight @ v[:, head]) * gate[:, head:head + 1]
    return out.reshape(T, H * m.vdim) @ w[p + "o"].T


def min_gru(w: Dict[str, np.ndarray], p: str, h):
    z = sigmoid(h @ w[p + "z"].T + w[p + "z.b"])
    u = h @ w[p + "x"].T + w[p + "x.b"]
    candidate = np.where(u >= 0, u + 0.5, sigmoid(u))
    g = h @ w[p + "g"].T
    state = np.zeros(z.shape[1])
    out = np.zeros_like(z)
    for t in range(h.shape[0]):
        state = (1.0 - z[t]) * state + z[t] * candidate[t]
        out[t] = state * g[t] * sigmoid(g[t])
    return out @ w[p + "o"].T


def silu(x):
    return x * sigmoid(x)


def grouped_attention(w: Dict[str, np.ndarray], p: str, m: GroupedAttentionConfig, h):
    """Query heads that share key/value heads; a window that also keeps the sequence's first positions; optionally a sink of score 0."""
    T, H, G = h.shape[0], m.heads, m.kv_heads
    q = (h @ w[p + "q"].T).reshape(T, H, m.dim)
    k = (h @ w[p + "k"].T).reshape(T, G, m.dim)
    v = (h @ w[p + "v"].T).reshape(T, G, m.vdim)
    seen = window_mask(T, m.window)
    if m.window > 0:
        seen = seen | (window_mask(T, 0) & (np.arange(T)[None, :] < m.keep_first))
    out = np.zeros((T, H, m.vdim))
    for head in range(H):
        g = head // (H // G)
        score = np.where(seen, (q[:, head] @ k[:, g].T) * m.scale, -np.inf)
        top = score.max(axis=1, keepdims=True)
        if m.sink:
            top = np.maximum(top, 0.0)
        weight = np.exp(score - top)
        total = weight.sum(axis=1, keepdims=True) + (np.exp(-top) if m.sink else 0.0)
        out[:, head] = (weight / total) @ v[:, g]
    return out.reshape(T, H * m.vdim) @ w[p + "o"].T


def causal_conv(x, taps):
    """x [T, C], taps [C, n]: the last column meets the current token, zeros stand before the start."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, x.shape[1])), x])
    return sum(padded[j:j + len(x)] * taps[:, j] for j in range(n))


def delta_rule(q, k, v, g, beta):
    """One head: q, k, g [T, dim], v [T, vdim], beta [T].  The state decays per key channel, is corrected towards v at k, and is read
    by q after the correction."""
    S = np.zeros((k.shape[1], v.shape[1]))
    out = np.zeros_like(v)
    for t in range(len(k)):
        S = g[t][:, None] * S
        S = S + np.outer(k[t], beta[t] * (v[t] - S.T @ k[t]))
        out[t] = S.T @ q[t]
    return out


def channel_delta(w: Dict[str, np.ndarray], p: str, m: ChannelDeltaConfig, h, eps: float):
    T, H, G = h.shape[0], m.heads, m.kv_heads
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    unit = lambda x: x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + 1e-6)
    q, k, v = unit(q.reshape(T, G, m.dim)) * m.dim ** -0.5, unit(k.reshape(T, G, m.dim)), v.reshape(T, H, m.vdim)
    beta = sigmoid(h @ w[p + "b"].T)
    a = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    g = np.exp(-np.exp(w[p + "A_log"])[None, :, None] * np.logaddexp(0.0, a).reshape(T, H, m.dim))
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(T, H, m.vdim)
    out = np.zeros((T, H, m.vdim))
    for head in range(H):
        s = head // (H // G)
        o = delta_rule(q[:, s], k[:, s], v[:, head], g[:, head], beta[:, head])
        out[:, head] = rms_norm(o, w[p + "norm"], eps) * gate[:, head]
    return out.reshape(T, H * m.vdim) @ w[p + "o"].T


def lightning(w: Dict[str, np.ndarray], p: str, m: LightningConfig, h, eps: float):
    T, H = h.shape[0], m.heads
    q, k, v = (silu(h @ w[p + n].T).reshape(T, H, -1) for n in "qkv")
    out = np.zeros((T, H, m.vdim))
    for head in range(H):
        S = np.zeros((m.dim, m.vdim))
        for t in range(T):
            S = m.decay[head] * S + np.outer(k[t, head], v[t, head])
            out[t, head] = S.T @ q[t, head]
    return (rms_norm(out.reshape(T, H * m.vdim), w[p + "norm"], eps) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def dense_glu(w: Dict[str, np.ndarray], p: str, m: DenseGLUConfig, h):
    g = np.minimum(h @ w[p + "gate"].T, m.limit)
    u = np.clip(h @ w[p + "up"].T, -m.limit, m.limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def embed(w: Dict[str, np.ndarray], cfg: TokenLMConfig, tokens):
    x = w["embed"][tokens] * cfg.embed_scale
    if cfg.bigram is not None:
        rows = [cfg.bigram.buckets] + [(int(a) * cfg.bigram.mul_prev + int(b) * cfg.bigram.mul_cur) % cfg.bigram.buckets for a, b in zip(tokens, tokens[1:])]
        x = x + w["bigram"][rows]
    if cfg.max_positions > 0:
        x = x + w["pos"][:len(tokens)]
    return x


def experts(w: Dict[str, np.ndarray], p: str, m: MoEConfig, h, tokens):
    out = np.zeros_like(h)
    for t, tok in enumerate(tokens):
        for e in w[p + "table"][tok]:
            a = np.maximum(w[f"{p}e{e}.up"] @ h[t], 0.0)
            out[t] += (w[f"{p}e{e}.down"] @ (a * a)) / m.top
    return out


class TokenLMOracle:
    def __init__(self, state_dict, cfg: TokenLMConfig):
        self.cfg = cfg
        self.w = {k: (v.numpy() if not v.is_floating_point() else v.double().numpy()) for k, v in state_dict.items()}

    def mixer(self, i: int, h):
        cfg, w, m, p = self.cfg, self.w, self.cfg.layers[i].mixer, f"l{i}.mix."
        if isinstance(m, LatentAttentionConfig):
            return latent_attention(w, p, m, h, cfg.norm_eps)
        if isinstance(m, MinGRUConfig):
            return min_gru(w, p, h)
        if isinstance(m, GroupedAttentionConfig):
            return grouped_attention(w, p, m, h)
        if isinstance(m, ChannelDeltaConfig):
            return channel_delta(w, p, m, h, cfg.norm_eps)
        return lightning(w, p, m, h, cfg.norm_eps)

    def residual(self, tokens, taps: Optional[List[np.ndarray]] = None):
        """The residual stream [T, width] after the last layer; `taps` collects it after every layer run."""
        cfg, w = self.cfg, self.w
        tokens = np.asarray(tokens)
        emb = embed(w, cfg, tokens)
        x = emb.copy()
        passes = 0
        for i in cfg.layer_runs:
            if cfg.loop_stop > cfg.loop_start and i == cfg.loop_start:
                if cfg.loop_inject == "project":
                    x = np.concatenate([x, emb], axis=1) @ w["loop.in"].T + w["loop.step"][passes]
                elif passes:
                    x = x + emb
                passes += 1
            layer, p = cfg.layers[i], f"l{i}."
            h = rms_norm(x, w[p + "norm1"], cfg.norm_eps, cfg.norm_groups)
            delta = self.mixer(i, h)
            if cfg.layer_scales:
                delta = delta * w[p + "ls1"]
            if layer.mlp is not None:
                h2 = rms_norm(x, w[p + "norm2"], cfg.norm_eps, cfg.norm_groups) if cfg.norms == 2 else h
                ff = dense_glu(w, p + "mlp.", layer.mlp, h2) if isinstance(layer.mlp, DenseGLUConfig) else experts(w, p + "mlp.", layer.mlp, h2, tokens)
                delta = delta + (ff * w[p + "ls2"] if cfg.layer_scales else ff)
            x = x + delta
            if taps is not None:
                taps.append(x)
        return x

    def logits(self, tokens, taps: Optional[List[np.ndarray]] = None):
        """[T, vocab]"""
        x = self.residual(tokens, taps)
        head = self.w["embed" if self.cfg.tied_head else "head"]
        return rms_norm(x, self.w["final.norm"], self.cfg.norm_eps, self.cfg.norm_groups) @ head.T * self.cfg.logit_scale

    def greedy(self, prompt, n: int, stop=()):
        toks = list(prompt)
        out = []
        for _ in range(n):
            t = int(np.argmax(self.logits(toks)[-1]))
            out.append(t)
            toks.append(t)
            if t in stop:
                break
        return out
