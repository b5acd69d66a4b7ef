"""Plain numpy restatement of the token language models (moshi_amd/tlm.py), float64, one function per mechanism, whole sequences at
once: no cache, no state hand-over, no batching.  For tests only - it shares no code with the engine and reads the same state dict.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import numpy as np

from moshi_amd.config import LatentAttentionConfig, MoEConfig, TokenLMConfig


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

    def residual(self, tokens, taps: Optional[List[np.ndarray]] = None):
        """The residual stream [T, width] after the last layer; `taps` collects it after every layer run."""
        cfg, w = self.cfg, self.w
        tokens = np.asarray(tokens)
        emb = w["embed"][tokens]
        x = emb.copy()
        passes = 0
        for i in cfg.layer_runs:
            if cfg.loop_stop > cfg.loop_start and i == cfg.loop_start:
                if passes:
                    x = x + emb
                passes += 1
            layer, p = cfg.layers[i], f"l{i}."
            h = rms_norm(x, w[p + "norm1"], cfg.norm_eps, cfg.norm_groups)
            if isinstance(layer.mixer, LatentAttentionConfig):
                delta = latent_attention(w, p + "mix.", layer.mixer, h, cfg.norm_eps)
            else:
                delta = min_gru(w, p + "mix.", h)
            delta = delta * w[p + "ls1"]
            if layer.mlp is not None:
                delta = delta + experts(w, p + "mlp.", layer.mlp, h, tokens) * w[p + "ls2"]
            x = x + delta
            if taps is not None:
                taps.append(x)
        return x

    def logits(self, tokens, taps: Optional[List[np.ndarray]] = None):
        """[T, vocab]"""
        x = self.residual(tokens, taps)
        return rms_norm(x, self.w["final.norm"], self.cfg.norm_eps, self.cfg.norm_groups) @ self.w["head"].T * self.cfg.logit_scale

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
