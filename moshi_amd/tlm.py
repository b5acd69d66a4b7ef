"""`TokenLM` - a decoder-only language model over token ids on the HIP engine (libmoshi_tlm.so, include/moshi_tlm.h).

    lm = loaders.get_token_lm("/models/some-dir", device="cuda", max_slots=32, max_tokens=65536)
    slot = lm.open()
    logits = lm.step([(slot, prompt_ids, [len(prompt_ids) - 1])])      # fp32 [wanted, vocab]
    lm.close(slot)

One step is one batch: prompt portions of some sequences beside single tokens of others.  The engine owns the paged cache and the
recurrent state; `TokenBatcher` (token_batcher.py) is the request scheduler on top.
"""
from __future__ import annotations

import ctypes as C
from typing import Dict, List, Optional, Sequence, Tuple

import torch

from . import _capi
from .config import (ChannelDeltaConfig, DenseGLUConfig, GroupedAttentionConfig, LatentAttentionConfig, LightningConfig, MinGRUConfig, MoEConfig,
                     TokenLMConfig)

Entry = Tuple[int, Sequence[int], Sequence[int]]          # slot, next tokens, wanted places among them


def _cfg_struct(cfg: TokenLMConfig, dtype: torch.dtype):
    layers = (_capi.TLMLayer * len(cfg.layers))()
    for out, layer in zip(layers, cfg.layers):
        m = layer.mixer
        if isinstance(m, LatentAttentionConfig):
            out.mixer = _capi.TLM_MIX_LATENT_ATTENTION
            out.heads, out.dim, out.vdim, out.rot_dim = m.heads, m.dim, m.vdim, m.rot_dim
            out.q_rank, out.kv_rank, out.window = m.q_rank, m.kv_rank, m.window
            out.scale, out.rot_base = m.scale, m.rot_base
        elif isinstance(m, MinGRUConfig):
            out.mixer, out.width = _capi.TLM_MIX_MINGRU, m.width
        elif isinstance(m, GroupedAttentionConfig):
            out.mixer, out.heads, out.kv_heads, out.dim, out.vdim = _capi.TLM_MIX_ATTENTION, m.heads, m.kv_heads, m.dim, m.vdim
            out.scale, out.window, out.keep_first, out.sink = m.scale, m.window, m.keep_first, int(m.sink)
        elif isinstance(m, ChannelDeltaConfig):
            out.mixer, out.heads, out.kv_heads, out.dim, out.vdim = _capi.TLM_MIX_CHANNEL_DELTA, m.heads, m.kv_heads, m.dim, m.vdim
            out.conv, out.decay_rank, out.gate_rank = m.conv, m.decay_rank, m.gate_rank
        elif isinstance(m, LightningConfig):
            out.mixer, out.heads, out.dim, out.vdim = _capi.TLM_MIX_LIGHTNING, m.heads, m.dim, m.vdim
            if len(m.decay) != m.heads:
                raise ValueError("lightning: one decay per head")
            out.decay = (C.c_double * m.heads)(*m.decay)
        else:
            raise ValueError(f"unknown mixer {type(m).__name__}")
        e = layer.mlp
        if isinstance(e, DenseGLUConfig):
            if e.activation != "clamped_swiglu":
                raise NotImplementedError("dense feed-forward: activation clamped_swiglu is implemented")
            out.mlp, out.ff, out.act, out.limit = _capi.TLM_MLP_DENSE, e.ff, _capi.TLM_ACT_CLAMPED_SWIGLU, e.limit
        elif isinstance(e, MoEConfig):
            if e.activation != "relu2" or e.router != "token_table":
                raise NotImplementedError("experts: activation relu2 and router token_table are implemented")
            out.mlp, out.experts, out.top, out.ff = _capi.TLM_MLP_MOE, e.experts, e.top, e.ff
            out.act, out.router = _capi.TLM_ACT_RELU2, _capi.TLM_ROUTE_TOKEN_TABLE
        elif e is not None:
            raise ValueError(f"unknown feed-forward {type(e).__name__}")
    s = _capi.TLMCfg()
    s.vocab, s.width, s.n_layers, s.layers = cfg.vocab, cfg.width, len(cfg.layers), layers
    s.loop_start, s.loop_stop, s.loop_times = cfg.loop_start, cfg.loop_stop, cfg.loop_times
    s.norm_groups, s.norm_eps, s.logit_scale = cfg.norm_groups, cfg.norm_eps, cfg.logit_scale
    s.loop_inject = {"add": _capi.TLM_LOOP_ADD, "project": _capi.TLM_LOOP_PROJECT}[cfg.loop_inject]
    s.norms, s.layer_scales, s.tied_head, s.embed_scale = cfg.norms, int(cfg.layer_scales), int(cfg.tied_head), cfg.embed_scale
    if cfg.bigram is not None:
        s.bigram_buckets, s.bigram_mul_prev, s.bigram_mul_cur = cfg.bigram.buckets, cfg.bigram.mul_prev, cfg.bigram.mul_cur
    s.max_positions = cfg.max_positions
    s.dtype = _capi.MMI_F32 if dtype == torch.float32 else _capi.MMI_BF16
    return s, layers


def _i32(v):
    return (C.c_int32 * max(1, len(v)))(*v)


class TokenLM:
    """Weights, cache pool and sequence slots of one model on one GPU.

    Args:
        state_dict: tensors named as in model.safetensors (weights.token_lm_state_spec).
        dtype: torch.bfloat16 (bf16 operands, fp32 accumulation, fp32 where the design wants it) or torch.float32 (all fp32).
        max_slots: live sequences.  max_tokens: tokens the cache pool holds over all of them (rounded up to pages).
        max_step_tokens: tokens of one step (activation buffers); default = the pool.
    """

    def __init__(self, state_dict: Dict[str, torch.Tensor], config: TokenLMConfig, device: torch.device | str = "cuda",
                 dtype: torch.dtype = torch.bfloat16, max_slots: int = 32, max_tokens: int = 65536, max_step_tokens: Optional[int] = None,
                 lib: Optional[_capi.Lib] = None):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("dtype must be torch.bfloat16 or torch.float32")
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        if lib is None:
            if self.device.type != "cuda":
                raise RuntimeError("moshi_amd.TokenLM runs on an MI355X (device='cuda'); there is no CPU path")
            lib = _capi.load_tlm()
        self._lib = lib
        self._handle = C.c_void_p()
        self.vocab, self.max_slots = config.vocab, int(max_slots)
        self.max_positions = config.max_positions              # longest sequence; 0: the pool alone bounds it
        self.max_step_tokens = int(max_step_tokens or max_tokens)
        cfg, keep_layers = _cfg_struct(config, dtype)
        state = {k: (v if v.dtype == torch.int32 else v.to(torch.bfloat16)).to(self.device) for k, v in state_dict.items()}
        descs, keep = _capi.tensor_descs(state)
        with _capi.device_scope(self.device):
            self._sync()
            self._lib.check(self._lib.mmi_tlm_create(C.byref(cfg), descs, len(state), self.max_slots, int(max_tokens), self.max_step_tokens,
                                                     C.byref(self._handle)))
        del keep, keep_layers

    def _sync(self):
        if self.device.type == "cuda":
            torch.cuda.synchronize(self.device)

    def __del__(self):
        try:
            if self._handle.value:
                self._lib.mmi_tlm_destroy(self._handle)
                self._handle = C.c_void_p()
        except Exception:
            pass

    # ---- sequences -------------------------------------------------------------------------------------------------
    def open(self) -> int:
        """Admit a sequence; BufferError when every slot is taken."""
        s = C.c_int32(0)
        self._lib.check(self._lib.mmi_tlm_open(self._handle, C.byref(s)))
        return int(s.value)

    def close(self, slot: int) -> None:
        self._lib.check(self._lib.mmi_tlm_close(self._handle, int(slot)))

    def info(self, which: int, slot: int = -1) -> int:
        return int(self._lib.mmi_tlm_info(self._handle, which, slot))

    @property
    def page_tokens(self) -> int:
        return self.info(_capi.TLM_PAGE_TOKENS)

    @property
    def total_pages(self) -> int:
        return self.info(_capi.TLM_TOTAL_PAGES)

    @property
    def free_pages(self) -> int:
        return self.info(_capi.TLM_FREE_PAGES)

    @property
    def free_slots(self) -> int:
        return self.info(_capi.TLM_FREE_SLOTS)

    def position(self, slot: int) -> int:
        return self.info(_capi.TLM_POSITION, slot)

    def pages_needed(self, slot: int, n: int) -> int:
        """Pages to hand out before `n` more tokens fit (slot -1: an empty sequence)."""
        return int(self._lib.mmi_tlm_pages_needed(self._handle, slot, n))

    # ---- computation -----------------------------------------------------------------------------------------------
    def step(self, entries: Sequence[Entry], out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Append each entry's tokens to its sequence; returns fp32 logits [wanted, vocab] in the order of the entries and of their
        wanted places.  A token of -1 stands for the one `sample` last drew for that slot (it never visits the host).
        BufferError, with nothing changed, when the pool has too few free pages."""
        slots, counts, tokens, want = [], [], [], []
        order = None
        for slot, toks, w in entries:
            base = len(tokens)
            slots.append(int(slot))
            counts.append(len(toks))
            tokens.extend(int(t) for t in toks)
            want.extend(base + int(p) for p in w)
        if any(b <= a for a, b in zip(want, want[1:])):         # the engine takes ascending rows
            uniq = sorted(set(want))
            order = [uniq.index(p) for p in want]
            want = uniq
        if out is None or order is not None:
            buf = torch.empty((len(want), self.vocab), dtype=torch.float32, device=self.device)
        else:
            assert out.shape == (len(want), self.vocab) and out.dtype == torch.float32 and out.is_contiguous()
            buf = out
        self._lib.check(self._lib.mmi_tlm_step(self._handle, len(slots), _i32(slots), _i32(counts), _i32(tokens), len(want), _i32(want),
                                               buf.data_ptr() if want else None, _capi.stream_ptr(self.device)))
        return buf if order is None else buf[torch.tensor(order, device=self.device)]

    def sample(self, logits: torch.Tensor, slots: Sequence[int], temp: Sequence[float] | float = 0.0, top_k: Sequence[int] | int = 0,
               seed: int = 0) -> torch.Tensor:
        """One token per row (int32, on the device); temp <= 0 is greedy, top_k 0 the whole vocabulary."""
        n = len(slots)
        temp = [float(temp)] * n if isinstance(temp, (int, float)) else [float(t) for t in temp]
        top_k = [int(top_k)] * n if isinstance(top_k, int) else [int(k) for k in top_k]
        assert logits.shape == (n, self.vocab) and logits.is_contiguous()
        out = torch.empty((n,), dtype=torch.int32, device=self.device)
        self._lib.check(self._lib.mmi_tlm_sample(self._handle, n, logits.data_ptr(), _i32(slots), (C.c_float * n)(*temp), _i32(top_k), int(seed),
                                                 out.data_ptr(), _capi.stream_ptr(self.device)))
        return out

    # ---- diagnostics -----------------------------------------------------------------------------------------------
    def step_with_taps(self, entries: Sequence[Entry]) -> Tuple[torch.Tensor, torch.Tensor]:
        """`step`, and the residual stream after every layer run: fp32 [layer runs, tokens, width]."""
        n = sum(len(t) for _, t, _ in entries)
        taps = torch.zeros((self.info(_capi.TLM_LAYER_RUNS), n, self.config.width), dtype=torch.float32, device=self.device)
        self._lib.check(self._lib.mmi_tlm_set_taps(self._handle, taps.data_ptr()))
        try:
            logits = self.step(entries)
            self._sync()
        finally:
            self._lib.mmi_tlm_set_taps(self._handle, None)
        return logits, taps

    def launch_list(self) -> List[Tuple[str, str, int]]:
        """(site, kernel, weight bytes) of the last step's launches."""
        return _capi.launch_list(lambda b, n: self._lib.mmi_tlm_launch_list(self._handle, b, n), with_bytes=True)
