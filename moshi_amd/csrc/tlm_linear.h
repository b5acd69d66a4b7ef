// Mixers of the token language models that carry a matrix per head and sequence, S [dim][vdim] fp32:
//
//   lightning      S <- d S + k v^T                                                  o = S^T q      d: a constant per head
//   channel delta  S <- g * S (per row); u = b (v - S^T k); S <- S + k u^T           o = S^T q      g: per head, row and token
//
// Everything in this file is fp32 (v_mfma_f32_16x16x4_f32, an exact fma chain), in the bf16 format too.  Sequences that bring at most
// TLM_SMALL tokens in a step go through k_tlm_state_step, token by token with S in registers.  Prompt portions are cut into chunks of 64
// tokens: what does not depend on S is computed for all chunks in parallel, then k_tlm_chunk_scan walks a sequence's chunks with S in the
// registers of four waves per 16 columns.  With G_t the product of the decays from the chunk's first token to t (per row of S):
//
//   u_t + b_t sum_(s<t) (k_t G_t/G_s k_s) u_s = b_t (v_t - S_0^T (G_t k_t))          a unit lower triangular system, (I + A) U = B
//   o_t = S_0^T (G_t q_t) + sum_(s<=t) (q_t G_t/G_s k_s) u_s                         P
//   S_end = G_end S_0 + sum_s (G_end/G_s k_s) u_s^T
//
// so W = (I + A)^-1 diag(b) (G K) and U0 = (I + A)^-1 diag(b) V turn the system into U = U0 - W S_0.  Decay ratios are never formed by a
// division or from logarithms: inside 16 tokens they are running products, across them (product to the end of s's 16) x (whole 16s between)
// x (product from the start of t's 16), so that they lose nothing however strong the decay is, and underflow to the zero they stand for.
#pragma once
#include "tlm_kernels.h"

constexpr int TLM_CHUNK = 64;
constexpr int TLM_SMALL = 4;             // up to here a sequence's tokens are stepped one by one
constexpr int TLM_PST = 68;              // row stride of a 64-column panel in LDS: rows stay 16-byte aligned, columns spread over the banks

struct TlmUnit { int row0, n, slot, par, fresh, chunk0, n_chunks, pad; };      // one sequence of the step; fresh: position 0, the state is zero

// Heads are padded to 16 in both sizes; every per-head section of a buffer has the padded stride.
struct TlmLinArgs {
    const float* in; int in_ld;          // the input projection: columns q0 .. (kv_heads), k0 .. (kv_heads), v0 .. (heads), b0 .. (delta: one per head)
    int q0, k0, v0, b0;
    int heads, kv_heads, dim, vdim, dim_p, vdim_p;
    float q_scale, eps;
    const float* conv_w; float* conv_state; int conv_c, taps;      // delta: [taps][channels]; [slot][2][taps - 1][channels], read one copy and write the other
    const float* decay;                  // delta: [row][heads][dim_p]; lightning: powers 0 .. TLM_CHUNK of every head's constant
    const float* gate; int gate_ld;      // factor of the normalised output
    const float* nw;                     // its weight (delta: per head column, lightning: per column)
    float* state;                        // [slot][heads][dim_p][vdim_p]
    const TlmUnit* small; const TlmUnit* unit; const TlmSeg* chunk;
    float* qkv;                          // delta: convolved and normalised [row][conv_c], same columns as `in`
    float *w, *qg, *kt, *u0, *p, *gend;  // per (chunk, head): [64][dim_p], [64][dim_p], [dim_p][64], [64][vdim_p], [64][64], [dim_p]
    float* o;                            // [row][heads][vdim_p] before the norm
    void* out; int out_ks;               // packed operand of the output projection
};

__device__ __forceinline__ float tlm_silu(float x) { return x * tlm_sigmoid(x); }

// channel c of the convolution at token t of a sequence whose rows start at row0 of the projection
__device__ __forceinline__ float tlm_conv(const TlmLinArgs& a, const float* old, int fresh, int row0, int t, int c) {
    float s = 0.f;
    for (int j = 0; j < a.taps; ++j) {
        const int at = t - (a.taps - 1) + j;
        float x = 0.f;
        if (at >= 0) x = a.in[(long)(row0 + at) * a.in_ld + c];
        else if (!fresh) x = old[(long)(a.taps - 1 + at) * a.conv_c + c];
        s = mmi_fma(a.conv_w[(long)j * a.conv_c + c], x, s);
    }
    return s;
}
// the last taps - 1 inputs of channel c after n tokens
__device__ __forceinline__ void tlm_conv_keep(const TlmLinArgs& a, const float* old, float* now, int fresh, int row0, int n, int c) {
    for (int s = 0; s < a.taps - 1; ++s) {
        const int at = n - (a.taps - 1) + s;
        float x = 0.f;
        if (at >= 0) x = a.in[(long)(row0 + at) * a.in_ld + c];
        else if (!fresh) x = old[(long)(n + s) * a.conv_c + c];
        now[(long)s * a.conv_c + c] = x;
    }
}

// ------------------------------------------------------------------------------------------------
// few tokens: one workgroup per (sequence, head), S in registers (thread: 4 columns of every parts-th row)
// ------------------------------------------------------------------------------------------------
inline int tlm_step_groups(int vdim_p) {                  // column groups of 4, a power of two
    int g = 4;
    while (4 * g < vdim_p) g *= 2;
    return g;
}
template <class Tr, bool DELTA, int RT>
__global__ __launch_bounds__(1024) void k_tlm_state_step(TlmLinArgs a, int cgp) {
    MMI_DYN_SHARED(float, sh);                             // q, k, g [dim_p], v [vdim_p], red [2][parts][vdim_p]
    const int tid = (int)threadIdx.x, nthr = (int)blockDim.x, lane = tid & 63;
    const int parts = nthr / cgp, cg = tid & (cgp - 1), part = tid / cgp, col = 4 * cg;
    const TlmUnit un = a.small[blockIdx.x];
    const int h = (int)blockIdx.y, rep = a.heads / a.kv_heads, kh = h / rep, D = a.dim_p, V = a.vdim_p;
    float *q = sh, *k = q + D, *g = k + D, *v = g + D, *red = v + V;
    const bool mine = col < V;
    float* S = a.state + ((long)un.slot * a.heads + h) * D * V;
    f32x4 s[RT];
#pragma unroll
    for (int i = 0; i < RT; ++i) {
        const int d = part + parts * i;
        s[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (!un.fresh && mine && d < D) s[i] = *reinterpret_cast<const f32x4*>(S + (long)d * V + col);
    }
    const float* old = nullptr;
    float* now = nullptr;
    if constexpr (DELTA) {
        old = a.conv_state + ((long)un.slot * 2 + un.par) * (a.taps - 1) * a.conv_c;
        now = a.conv_state + ((long)un.slot * 2 + (un.par ^ 1)) * (a.taps - 1) * a.conv_c;
    }
    for (int t = 0; t < un.n; ++t) {
        const long row = un.row0 + t;
        const float* in = a.in + row * a.in_ld;
        for (int i = tid; i < 2 * D + V; i += nthr) {
            const int c = i < D ? a.q0 + kh * D + i : (i < 2 * D ? a.k0 + kh * D + i - D : a.v0 + h * V + i - 2 * D);
            float x;
            if constexpr (DELTA) x = tlm_silu(tlm_conv(a, old, un.fresh, un.row0, t, c));
            else x = in[c];
            if (i < 2 * D) q[i] = x;
            else v[i - 2 * D] = x;
        }
        if constexpr (DELTA)
            for (int i = tid; i < D; i += nthr) g[i] = a.decay[(row * a.heads + h) * D + i];
        __syncthreads();
        float qq = 0.f, kk = 0.f, kq = 0.f;                // every wave sums for itself
        for (int i = lane; i < D; i += 64) {
            qq = mmi_fma(q[i], q[i], qq);
            kk = mmi_fma(k[i], k[i], kk);
            kq = mmi_fma(k[i], q[i], kq);
        }
        kq = tlm_wave_sum(kq);
        float iq = 1.f, ik = 1.f, beta = 1.f, dec = 1.f;
        if constexpr (DELTA) {
            iq = a.q_scale / sqrtf(tlm_wave_sum(qq) + 1e-6f);
            ik = 1.0f / sqrtf(tlm_wave_sum(kk) + 1e-6f);
            kq *= iq * ik;
            beta = in[a.b0 + h];
        } else {
            dec = a.decay[h * (TLM_CHUNK + 1) + 1];
        }
        f32x4 ak = {0.f, 0.f, 0.f, 0.f}, aq = ak;
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            const int d = part + parts * i;
            if (d >= D) continue;
            s[i] *= DELTA ? g[d] : dec;
            if constexpr (DELTA) ak += (k[d] * ik) * s[i];
            aq += (q[d] * iq) * s[i];
        }
        if (mine) {
            *reinterpret_cast<f32x4*>(red + (long)part * V + col) = aq;
            if constexpr (DELTA) *reinterpret_cast<f32x4*>(red + (long)(parts + part) * V + col) = ak;
        }
        __syncthreads();
        f32x4 u = {0.f, 0.f, 0.f, 0.f}, o = u;
        if (mine) {
            for (int p = 0; p < parts; ++p) {
                o += *reinterpret_cast<const f32x4*>(red + (long)p * V + col);
                if constexpr (DELTA) u += *reinterpret_cast<const f32x4*>(red + (long)(parts + p) * V + col);
            }
            const f32x4 vv = *reinterpret_cast<const f32x4*>(v + col);
            u = DELTA ? beta * (vv - u) : vv;
            o += kq * u;
        }
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            const int d = part + parts * i;
            if (d < D) s[i] += (k[d] * ik) * u;
        }
        if constexpr (DELTA) {
            float ss = o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
            for (int x = 1; x < cgp; x *= 2) ss += mmi_shfl_xor(ss, x);      // (the groups of one row part are neighbours in a wave)
            const float inv = 1.0f / sqrtf(ss / (float)a.vdim + a.eps);
            if (part == 0 && mine) {
                const f32x4 w = *reinterpret_cast<const f32x4*>(a.nw + col), gt = *reinterpret_cast<const f32x4*>(a.gate + row * a.gate_ld + h * V + col);
                Tr::store4((typename Tr::elem*)a.out + tlm_index<Tr>(row, h * V + col, a.out_ks), o * inv * w * gt);
            }
        } else if (part == 0 && mine) {
            *reinterpret_cast<f32x4*>(a.o + (row * a.heads + h) * V + col) = o;
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < RT; ++i) {
        const int d = part + parts * i;
        if (mine && d < D) *reinterpret_cast<f32x4*>(S + (long)d * V + col) = s[i];
    }
    if constexpr (DELTA)
        for (int i = tid; i < 2 * D + V; i += nthr) {
            if (i < 2 * D && h % rep) continue;            // query and key channels are shared by the heads of a group
            tlm_conv_keep(a, old, now, un.fresh, un.row0, un.n, i < D ? a.q0 + kh * D + i : (i < 2 * D ? a.k0 + kh * D + i - D : a.v0 + h * V + i - 2 * D));
        }
}

// ------------------------------------------------------------------------------------------------
// chunks: convolutions and unit norms (delta).  grid: chunks, 2 kv_heads + heads; a wave takes 16 tokens, its lanes the channels of a head
// ------------------------------------------------------------------------------------------------
inline __global__ __launch_bounds__(256) void k_tlm_conv(TlmLinArgs a) {
    const int lane = (int)threadIdx.x & 63, wave = (int)threadIdx.x >> 6, y = (int)blockIdx.y;
    const TlmSeg ck = a.chunk[blockIdx.x];
    const int kind = y < a.kv_heads ? 0 : (y < 2 * a.kv_heads ? 1 : 2);
    const int width = kind == 2 ? a.vdim_p : a.dim_p;
    const int c0 = kind == 0 ? a.q0 + y * a.dim_p : (kind == 1 ? a.k0 + (y - a.kv_heads) * a.dim_p : a.v0 + (y - 2 * a.kv_heads) * a.vdim_p);
    const float* old = a.conv_state + ((long)ck.slot * 2 + ck.par) * (a.taps - 1) * a.conv_c;
    const int first = ck.row0 - ck.index * TLM_CHUNK;      // the sequence's first row of this step
    for (int t = wave; t < ck.n; t += 4) {
        float x[4], ss = 0.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int c = lane + 64 * i;
            x[i] = c < width ? tlm_silu(tlm_conv(a, old, ck.fresh, first, ck.index * TLM_CHUNK + t, c0 + c)) : 0.f;
            ss = mmi_fma(x[i], x[i], ss);
        }
        float f = 1.f;
        if (kind != 2) f = (kind == 0 ? a.q_scale : 1.0f) / sqrtf(tlm_wave_sum(ss) + 1e-6f);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int c = lane + 64 * i;
            if (c < width) a.qkv[(long)(ck.row0 + t) * a.conv_c + c0 + c] = x[i] * f;
        }
    }
    if (ck.last) {
        float* now = a.conv_state + ((long)ck.slot * 2 + (ck.par ^ 1)) * (a.taps - 1) * a.conv_c;
        for (int c = (int)threadIdx.x; c < width; c += 256) tlm_conv_keep(a, old, now, ck.fresh, first, ck.index * TLM_CHUNK + ck.n, c0 + c);
    }
}

// ------------------------------------------------------------------------------------------------
// chunks, lightning: P, the decayed queries, the decayed transposed keys.  grid: chunks, heads
// ------------------------------------------------------------------------------------------------
inline __global__ __launch_bounds__(256) void k_tlm_chunk_lightning(TlmLinArgs a) {
    const int lane = (int)threadIdx.x & 63, wave = (int)threadIdx.x >> 6, bl = lane & 15, kq = lane >> 4, h = (int)blockIdx.y;
    const TlmSeg ck = a.chunk[blockIdx.x];
    const int D = a.dim_p;
    const long id = (long)blockIdx.x * a.heads + h;
    MMI_SHARED float pw[TLM_CHUNK + 1];
    for (int i = (int)threadIdx.x; i <= TLM_CHUNK; i += 256) pw[i] = a.decay[h * (TLM_CHUNK + 1) + i];
    __syncthreads();
    const float* qp = a.in + (long)ck.row0 * a.in_ld + a.q0 + h * D;
    const float* kp = a.in + (long)ck.row0 * a.in_ld + a.k0 + h * D;
    auto fetch = [&](const float* base, int t, int d) __attribute__((always_inline)) {
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        return t < ck.n ? *reinterpret_cast<const f32x4*>(base + (long)t * a.in_ld + d) : zero;
    };
    f32x4 acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int d = 0; d < D; d += 16) {
        const f32x4 qv = fetch(qp, 16 * wave + bl, d + 4 * kq);
        f32x4 kv[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) kv[j] = fetch(kp, 16 * j + bl, d + 4 * kq);
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (j <= wave) acc[j] = TlmF32::mfma(__builtin_bit_cast(u32x4, qv), __builtin_bit_cast(u32x4, kv[j]), acc[j]);
    }
    float* P = a.p + id * (TLM_CHUNK * TLM_CHUNK);
#pragma unroll
    for (int j = 0; j < 4; ++j)
        if (j <= wave)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = 16 * wave + 4 * kq + r, s = 16 * j + bl;
                P[t * TLM_CHUNK + s] = s <= t ? acc[j][r] * pw[t - s] : 0.f;
            }
    float* Q = a.qg + id * TLM_CHUNK * D;
    float* K = a.kt + id * TLM_CHUNK * D;
    const float ke = lane < ck.n ? pw[ck.n - 1 - lane] : 0.f;
    for (int d = 4 * wave; d < D; d += 16) {               // lane: token
        *reinterpret_cast<f32x4*>(Q + (long)lane * D + d) = fetch(qp, lane, d) * pw[lane + 1];
        const f32x4 kv = fetch(kp, lane, d);
#pragma unroll
        for (int e = 0; e < 4; ++e) K[(long)(d + e) * TLM_CHUNK + lane] = kv[e] * ke;
    }
    for (int d = (int)threadIdx.x; d < D; d += 256) a.gend[id * D + d] = pw[ck.n];
}

// ------------------------------------------------------------------------------------------------
// chunks, delta: P, W, U0, the decayed queries and transposed keys.  grid: chunks, heads; wave w owns tokens 16 w .. 16 w + 15
// ------------------------------------------------------------------------------------------------
inline size_t tlm_chunk_delta_smem() { return (size_t)(4 * TLM_CHUNK * TLM_PST + 4 * 64 + 4 * 16 * 20 + TLM_CHUNK) * sizeof(float); }
inline __global__ __launch_bounds__(256) void k_tlm_chunk_delta(TlmLinArgs a) {
    MMI_DYN_SHARED(float, sh);
    float *K = sh, *Q = K + TLM_CHUNK * TLM_PST, *G = Q + TLM_CHUNK * TLM_PST, *A = G + TLM_CHUNK * TLM_PST;      // [64][TLM_PST] each
    float *tot = A + TLM_CHUNK * TLM_PST, *ti = tot + 4 * 64, *beta = ti + 4 * 16 * 20;                            // [4][64], [4][16][20], [64]
    const int tid = (int)threadIdx.x, lane = tid & 63, wave = mmi_uniform(tid >> 6), bl = lane & 15, kq = lane >> 4, h = (int)blockIdx.y;
    const TlmSeg ck = a.chunk[blockIdx.x];
    const int D = a.dim_p, V = a.vdim_p, kh = h / (a.heads / a.kv_heads);
    const long id = (long)blockIdx.x * a.heads + h;
    const float* qkv = a.qkv + (long)ck.row0 * a.conv_c;
    float *Wg = a.w + id * TLM_CHUNK * D, *Qg = a.qg + id * TLM_CHUNK * D, *Kt = a.kt + id * TLM_CHUNK * D, *Ug = a.u0 + id * TLM_CHUNK * V;
    float* P = a.p + id * (TLM_CHUNK * TLM_CHUNK);
    if (tid < TLM_CHUNK) beta[tid] = tid < ck.n ? a.in[(long)(ck.row0 + tid) * a.in_ld + a.b0 + h] : 0.f;
    float dA[16], dP[16];                                  // pairs (16 w + bl, 16 w + s) of this lane's quarter of the channels
#pragma unroll
    for (int s = 0; s < 16; ++s) dA[s] = dP[s] = 0.f;
    // blocks below the diagonal: wave w takes entries w and w + 4 of (3,0) (3,1) (3,2) (2,0) (2,1) (1,0)
    const int bi[2] = {wave < 3 ? 3 : 2, wave == 0 ? 2 : 1}, bj[2] = {wave < 3 ? wave : 0, wave == 0 ? 1 : 0};
    const int nblk = wave < 2 ? 2 : 1;
    f32x4 oA[2], oP[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) oA[b] = oP[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int c0 = 0; c0 < D; c0 += 64) {
        const int cn = min(64, D - c0);                    // a multiple of 16
        __syncthreads();
        for (int i = tid; i < TLM_CHUNK * 16; i += 256) {
            const int t = i >> 4, c = 4 * (i & 15);
            f32x4 qv = {0.f, 0.f, 0.f, 0.f}, kv = qv, gv = {1.f, 1.f, 1.f, 1.f};
            if (t < ck.n && c < cn) {
                qv = *reinterpret_cast<const f32x4*>(qkv + (long)t * a.conv_c + a.q0 + kh * D + c0 + c);
                kv = *reinterpret_cast<const f32x4*>(qkv + (long)t * a.conv_c + a.k0 + kh * D + c0 + c);
                gv = *reinterpret_cast<const f32x4*>(a.decay + ((long)(ck.row0 + t) * a.heads + h) * D + c0 + c);
            }
            *reinterpret_cast<f32x4*>(Q + t * TLM_PST + c) = qv;
            *reinterpret_cast<f32x4*>(K + t * TLM_PST + c) = kv;
            *reinterpret_cast<f32x4*>(G + t * TLM_PST + c) = gv;
        }
        __syncthreads();
        for (int c = 4 * kq; c < cn; c += 16) {            // the 16 x 16 blocks on the diagonal, pair by pair with a running decay
            const int t0 = 16 * wave;
            const f32x4 kt = *reinterpret_cast<const f32x4*>(K + (t0 + bl) * TLM_PST + c), qt = *reinterpret_cast<const f32x4*>(Q + (t0 + bl) * TLM_PST + c);
            f32x4 d = {1.f, 1.f, 1.f, 1.f};
#pragma unroll
            for (int s = 15; s >= 0; --s) {
                if (s > bl) continue;
                const f32x4 x = d * *reinterpret_cast<const f32x4*>(K + (t0 + s) * TLM_PST + c);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    dA[s] = mmi_fma(kt[e], x[e], dA[s]);
                    dP[s] = mmi_fma(qt[e], x[e], dP[s]);
                }
                d *= *reinterpret_cast<const f32x4*>(G + (t0 + s) * TLM_PST + c);
            }
        }
        __syncthreads();
        {                                                  // K -> k x (decay from the start of its 16), Q likewise, G -> k x (decay to the end)
            const int c = lane;
            float g[16], kk[16];
            float run = 1.f;
#pragma unroll
            for (int t = 0; t < 16; ++t) {
                const int at = (16 * wave + t) * TLM_PST + c;
                g[t] = G[at];
                kk[t] = K[at];
                run *= g[t];
                K[at] = kk[t] * run;
                Q[at] *= run;
            }
            tot[wave * 64 + c] = run;
            run = 1.f;
#pragma unroll
            for (int t = 15; t >= 0; --t) {
                G[(16 * wave + t) * TLM_PST + c] = kk[t] * run;
                run *= g[t];
            }
        }
        __syncthreads();
#pragma unroll
        for (int b = 0; b < 2; ++b) {
            if (b >= nblk) continue;
            for (int c = 4 * kq; c < cn; c += 16) {
                f32x4 mid = {1.f, 1.f, 1.f, 1.f};
                for (int m = bj[b] + 1; m < bi[b]; ++m) mid *= *reinterpret_cast<const f32x4*>(tot + m * 64 + c);
                const u32x4 kv = __builtin_bit_cast(u32x4, *reinterpret_cast<const f32x4*>(G + (16 * bj[b] + bl) * TLM_PST + c) * mid);
                oA[b] = TlmF32::mfma(*reinterpret_cast<const u32x4*>(K + (16 * bi[b] + bl) * TLM_PST + c), kv, oA[b]);
                oP[b] = TlmF32::mfma(*reinterpret_cast<const u32x4*>(Q + (16 * bi[b] + bl) * TLM_PST + c), kv, oP[b]);
            }
        }
        for (int i = tid; i < TLM_CHUNK * 16; i += 256) {  // decayed queries, right sides of W
            const int t = i >> 4, c = 4 * (i & 15);
            if (c >= cn) continue;
            f32x4 f = {1.f, 1.f, 1.f, 1.f};
            for (int m = 0; m < t >> 4; ++m) f *= *reinterpret_cast<const f32x4*>(tot + m * 64 + c);
            *reinterpret_cast<f32x4*>(Qg + (long)t * D + c0 + c) = *reinterpret_cast<const f32x4*>(Q + t * TLM_PST + c) * f;
            *reinterpret_cast<f32x4*>(Wg + (long)t * D + c0 + c) = *reinterpret_cast<const f32x4*>(K + t * TLM_PST + c) * f * beta[t];
        }
        for (int c = wave; c < cn; c += 4) {               // lane: token
            float f = 1.f;
            for (int m = (lane >> 4) + 1; m < 4; ++m) f *= tot[m * 64 + c];
            Kt[(long)(c0 + c) * TLM_CHUNK + lane] = G[lane * TLM_PST + c] * f;
        }
        if (tid < cn) a.gend[id * D + c0 + tid] = tot[tid] * tot[64 + tid] * tot[128 + tid] * tot[192 + tid];
    }
    // - A: the strictly lower triangle (columns right of it inside the diagonal blocks: zero), P
#pragma unroll
    for (int s = 0; s < 16; ++s) {
        float x = dA[s], y = dP[s];
        x += mmi_shfl_xor(x, 16);
        x += mmi_shfl_xor(x, 32);
        y += mmi_shfl_xor(y, 16);
        y += mmi_shfl_xor(y, 32);
        const int t = 16 * wave + bl, at = 16 * wave + s;
        if (kq == 0) {
            A[t * TLM_PST + at] = s < bl ? -beta[t] * x : 0.f;
            P[t * TLM_CHUNK + at] = s <= bl ? y : 0.f;
        }
    }
#pragma unroll
    for (int b = 0; b < 2; ++b)
        if (b < nblk)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = 16 * bi[b] + 4 * kq + r, s = 16 * bj[b] + bl;
                A[t * TLM_PST + s] = -beta[t] * oA[b][r];
                P[t * TLM_CHUNK + s] = oP[b][r];
            }
    __syncthreads();
    {                                                      // (I + A_ww)^-1, one column per lane
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float s = t == bl ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < t; ++j) s = mmi_fma(A[(16 * wave + t) * TLM_PST + 16 * wave + j], x[j], s);
            x[t] = s;
            if (kq == 0) ti[(wave * 16 + t) * 20 + bl] = s;
        }
    }
    __syncthreads();
    // forward substitution by blocks of 16, one 16-column strip of [W | U0] at a time
    const int nd = D / 16, ns = nd + V / 16;
    for (int st = wave; st < ns; st += 4) {
        float* dst = st < nd ? Wg + 16 * st + bl : Ug + 16 * (st - nd) + bl;
        const int ld = st < nd ? D : V;
        f32x4 x[4];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = 16 * i + 4 * kq + r;
                if (st < nd) x[i][r] = dst[(long)t * ld];
                else x[i][r] = t < ck.n ? beta[t] * qkv[(long)t * a.conv_c + a.v0 + h * V + 16 * (st - nd) + bl] : 0.f;
            }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            f32x4 b = x[i];
#pragma unroll
            for (int j = 0; j < i; ++j)
                b = TlmF32::mfma(*reinterpret_cast<const u32x4*>(A + (16 * i + bl) * TLM_PST + 16 * j + 4 * kq), __builtin_bit_cast(u32x4, x[j]), b);
            x[i] = TlmF32::mfma(*reinterpret_cast<const u32x4*>(ti + (i * 16 + bl) * 20 + 4 * kq), __builtin_bit_cast(u32x4, b), f32x4{0.f, 0.f, 0.f, 0.f});
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) dst[(long)(16 * i + 4 * kq + r) * ld] = x[i][r];
    }
}

// ------------------------------------------------------------------------------------------------
// chunks: the walk over a sequence's chunks.  One workgroup per (sequence, head, 16 columns of S); wave w holds rows of S in the layout the
// matrix core leaves them in, which is also the layout it takes them as an operand; the waves' shares of W S and Qg S meet in LDS.
// grid: 8 x ceil(sequences x heads / 8) x vdim_p / 16, the column blocks of one head on one XCD (they read the same W, Qg, Kt, P)
// ------------------------------------------------------------------------------------------------
template <bool DELTA, int NDW>
__global__ __launch_bounds__(256, 1) void k_tlm_chunk_scan(TlmLinArgs a, int n_units) {
    MMI_SHARED __attribute__((aligned(16))) f32x4 red[2][DELTA ? 2 : 1][4][4][64];      // [parity][Qg S, W S][wave][token block][lane]
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15, kq = lane >> 4;
    const int ncb = a.vdim_p / 16, j0 = (int)blockIdx.x >> 3;
    const int uh = ((int)blockIdx.x & 7) + 8 * (j0 / ncb), cb = j0 % ncb;
    if (uh >= n_units * a.heads) return;
    const TlmUnit un = a.unit[uh / a.heads];
    const int h = uh % a.heads, D = a.dim_p, V = a.vdim_p, nd = D / 16;
    float* S = a.state + ((long)un.slot * a.heads + h) * D * V + 16 * cb + bl;
    f32x4 s[NDW];
#pragma unroll
    for (int i = 0; i < NDW; ++i) {
        s[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int d = wave * NDW + i;
        if (!un.fresh && d < nd)
#pragma unroll
            for (int r = 0; r < 4; ++r) s[i][r] = S[(long)(16 * d + 4 * kq + r) * V];
    }
    struct Frags {
        u32x4 w[DELTA ? 4 : 1][NDW], q[4][NDW], k[NDW][4], p[4];
        f32x4 u[4], g[NDW];
    };
    auto load = [&](Frags& f, int c) __attribute__((always_inline)) {
        const long id = (long)(un.chunk0 + c) * a.heads + h;
        const int n = min(TLM_CHUNK, un.n - c * TLM_CHUNK);
#pragma unroll
        for (int i = 0; i < NDW; ++i) {
            const int d = min(wave * NDW + i, nd - 1);     // (past the end: a valid address, against rows of S that stay zero)
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const long at = id * TLM_CHUNK * D + (long)(16 * t + bl) * D + 16 * d + 4 * kq;
                if constexpr (DELTA) f.w[t][i] = *reinterpret_cast<const u32x4*>(a.w + at);
                f.q[t][i] = *reinterpret_cast<const u32x4*>(a.qg + at);
                f.k[i][t] = *reinterpret_cast<const u32x4*>(a.kt + id * TLM_CHUNK * D + (long)(16 * d + bl) * TLM_CHUNK + 16 * t + 4 * kq);
            }
            f.g[i] = *reinterpret_cast<const f32x4*>(a.gend + id * D + 16 * d + 4 * kq);
        }
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            f.p[t] = *reinterpret_cast<const u32x4*>(a.p + id * (TLM_CHUNK * TLM_CHUNK) + (16 * wave + bl) * TLM_CHUNK + 16 * min(t, wave) + 4 * kq);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int tok = 16 * t + 4 * kq + r;
                if constexpr (DELTA) f.u[t][r] = a.u0[(id * TLM_CHUNK + tok) * V + 16 * cb + bl];
                else f.u[t][r] = tok < n ? a.in[(long)(un.row0 + c * TLM_CHUNK + tok) * a.in_ld + a.v0 + h * V + 16 * cb + bl] : 0.f;
            }
        }
    };
    Frags f;
    load(f, 0);
    for (int c = 0; c < un.n_chunks; ++c) {
        const int n = min(TLM_CHUNK, un.n - c * TLM_CHUNK);
        f32x4 x[4], y[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            x[t] = y[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < NDW; ++i) {
                if constexpr (DELTA) x[t] = TlmF32::mfma(f.w[t][i], __builtin_bit_cast(u32x4, s[i]), x[t]);
                y[t] = TlmF32::mfma(f.q[t][i], __builtin_bit_cast(u32x4, s[i]), y[t]);
            }
            if constexpr (DELTA) red[c & 1][DELTA][wave][t][lane] = x[t];
            red[c & 1][0][wave][t][lane] = y[t];
        }
        Frags nx;                                          // (the last chunk asks for itself again)
        load(nx, min(c + 1, un.n_chunks - 1));
        mmi_sched_barrier();
        __syncthreads();
        f32x4 u[4], o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            u[t] = f.u[t];
            if constexpr (DELTA)
#pragma unroll
                for (int v = 0; v < 4; ++v) u[t] -= red[c & 1][DELTA][v][t][lane];
        }
#pragma unroll
        for (int v = 0; v < 4; ++v) o += red[c & 1][0][v][wave][lane];
#pragma unroll
        for (int t = 0; t < 4; ++t)
            if (t <= wave) o = TlmF32::mfma(f.p[t], __builtin_bit_cast(u32x4, u[t]), o);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int tok = 16 * wave + 4 * kq + r;
            if (tok < n) a.o[((long)(un.row0 + c * TLM_CHUNK + tok) * a.heads + h) * V + 16 * cb + bl] = o[r];
        }
#pragma unroll
        for (int i = 0; i < NDW; ++i) {
            s[i] *= f.g[i];
#pragma unroll
            for (int t = 0; t < 4; ++t) s[i] = TlmF32::mfma(f.k[i][t], __builtin_bit_cast(u32x4, u[t]), s[i]);
            if (wave * NDW + i >= nd) s[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        }
        f = nx;
    }
#pragma unroll
    for (int i = 0; i < NDW; ++i) {
        const int d = wave * NDW + i;
        if (d < nd)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[(long)(16 * d + 4 * kq + r) * V] = s[i][r];
    }
}

// ------------------------------------------------------------------------------------------------
// RMS norm of a head's output (`per_head`) or of all heads' together, weight, gate -> packed operand; one workgroup per row: of the whole
// step, or (`chunk`) 64 per chunk
// ------------------------------------------------------------------------------------------------
template <class Tr>
__global__ __launch_bounds__(256) void k_tlm_gated_norm(TlmLinArgs a, int per_head, const TlmSeg* chunk) {
    MMI_DYN_SHARED(float, inv);                            // [heads], then [4]
    const int tid = (int)threadIdx.x, lane = tid & 63, wave = tid >> 6, V = a.vdim_p, ld = a.heads * V;
    long row = (int)blockIdx.x;
    if (chunk) {
        const TlmSeg ck = chunk[blockIdx.x >> 6];
        if ((int)(blockIdx.x & 63) >= ck.n) return;
        row = ck.row0 + (int)(blockIdx.x & 63);
    }
    const float* o = a.o + row * ld;
    if (per_head) {
        for (int h = wave; h < a.heads; h += 4) {
            float s = 0.f;
            for (int c = lane; c < V; c += 64) s = mmi_fma(o[h * V + c], o[h * V + c], s);
            s = tlm_wave_sum(s);
            if (lane == 0) inv[h] = 1.0f / sqrtf(s / (float)a.vdim + a.eps);
        }
    } else {
        float s = 0.f;
        for (int c = 4 * tid; c < ld; c += 1024) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(o + c);
            s += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        }
        s = tlm_wave_sum(s);
        float* part = inv + a.heads;
        if (lane == 0) part[wave] = s;
        __syncthreads();
        s = 1.0f / sqrtf((part[0] + part[1] + part[2] + part[3]) / (float)(a.heads * a.vdim) + a.eps);
        for (int h = tid; h < a.heads; h += 256) inv[h] = s;
    }
    __syncthreads();
    for (int c = 4 * tid; c < ld; c += 1024) {
        const int h = c / V;
        const f32x4 w = *reinterpret_cast<const f32x4*>(a.nw + (per_head ? c - h * V : c)), g = *reinterpret_cast<const f32x4*>(a.gate + row * a.gate_ld + c);
        Tr::store4((typename Tr::elem*)a.out + tlm_index<Tr>(row, c, a.out_ks), *reinterpret_cast<const f32x4*>(o + c) * inv[h] * w * g);
    }
}
