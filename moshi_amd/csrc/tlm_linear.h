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
    const float* decay;                  // delta: projection [row][heads][dim_p] (tlm_decay); lightning: powers 0 .. TLM_CHUNK of every head's constant
    const float* decay_c;                // delta: [2][heads][dim_p] summand, factor
    const float* gate; int gate_ld;      // the normalised output's factor, before its sigmoid
    const float* nw;                     // its weight (delta: per head column, lightning: per column)
    float* state;                        // [slot][heads][dim_p][vdim_p]
    const TlmUnit* small; const TlmUnit* unit; const TlmSeg* chunk;
    float* qkv;                          // delta: convolved and normalised [row][conv_c], same columns as `in`
    // per (chunk, head), in fragments of 16 x 16 (a lane's four elements together, so that the walk's loads are contiguous): w and qg
    // [64][dim_p], kt [dim_p][64], p [64][64] by tlm_tile; u0 [64][vdim_p] in the layout of the matrix core's sums; gend [dim_p]
    float *w, *qg, *kt, *u0, *p, *gend;
    float* o;                            // [row][heads][vdim_p] before the norm
    void* out; int out_ks;               // packed operand of the output projection
};

// decay of channel d of a head: exp(-factor softplus(z)), z = projection + summand, as 2^(-factor log2(1 + e^z)).  With u = e^z rounded
// and w = 1 + u rounded, log2(w) u / (w - 1) is log2(1 + u) to the last bits however small u is.
__device__ __forceinline__ float tlm_decay(const TlmLinArgs& a, long row, int h, int d) {
    constexpr float LOG2E = 1.44269504088896340736f;
    const int c = h * a.dim_p + d;
    const float z = a.decay[row * a.heads * a.dim_p + c] + a.decay_c[c];
    const float u = mmi_fast_exp2f(fminf(z, 30.f) * LOG2E), w = 1.0f + u;
    float l = w > 1.0f ? mmi_fast_log2f(w) * u / (w - 1.0f) : u * LOG2E;
    if (z > 20.f) l = z * LOG2E;
    return mmi_fast_exp2f(-a.decay_c[a.heads * a.dim_p + c] * l);
}
__device__ __forceinline__ float tlm_silu(float x) { return x * tlm_sigmoid(x); }

// element (row, k) of an operand with `ks` 16-wide blocks per 16 rows
MMI_HD long tlm_tile(int row, int k, int ks) { return (((long)(row >> 4) * ks + (k >> 4)) * 64 + ((k & 15) >> 2) * 16 + (row & 15)) * 4 + (k & 3); }

// channel(s) from c of the convolution at token t of a sequence whose rows start at row0 of the projection; four taps are requested at a
// time (a tap before the sequence's start reads some valid address and counts as zero).  `now`: where the taps - 1 inputs that the next
// step's first token needs stay, or null
template <class T>
__device__ __forceinline__ T tlm_conv(const TlmLinArgs& a, const float* old, int fresh, int row0, int t, int c, float* now) {
    T s = T{};
    for (int j0 = 0; j0 < a.taps; j0 += 4) {
        T x[4], w[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int tap = min(j0 + j, a.taps - 1), at = t - (a.taps - 1) + tap;
            x[j] = *reinterpret_cast<const T*>(at >= 0 || fresh ? a.in + (long)(row0 + max(at, 0)) * a.in_ld + c : old + (long)(a.taps - 1 + at) * a.conv_c + c);
            w[j] = *reinterpret_cast<const T*>(a.conv_w + (long)tap * a.conv_c + c);
            if (j0 + j >= a.taps || (at < 0 && fresh)) x[j] = T{};
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) s += w[j] * x[j];
        if (now)
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (j0 + j >= 1 && j0 + j < a.taps) *reinterpret_cast<T*>(now + (long)(j0 + j - 1) * a.conv_c + c) = x[j];
    }
    return s;
}

// ------------------------------------------------------------------------------------------------
// few tokens: one workgroup per (sequence, head), S in registers (thread: 4 columns of every parts-th row)
// ------------------------------------------------------------------------------------------------
inline int tlm_step_groups(int vdim_p) {                  // column groups of 4, a power of two
    int g = 4;
    while (4 * g < vdim_p) g *= 2;
    return g;
}
template <class Tr, bool DELTA, int RT, int MAXB>
__global__ __launch_bounds__(MAXB, MAXB == 512 && !DELTA ? 5 : 4) void k_tlm_state_step(TlmLinArgs a, int cgp) {
    MMI_DYN_SHARED(float, sh);                             // q, k, g [parts * RT] (zeros from dim_p on), v [vdim_p], red [2][parts][vdim_p]
    const int tid = (int)threadIdx.x, nthr = (int)blockDim.x, lane = tid & 63;
    const int parts = nthr / cgp, cg = tid & (cgp - 1), part = tid / cgp, col = 4 * cg;
    const TlmUnit un = a.small[blockIdx.x];
    const int h = (int)blockIdx.y, rep = a.heads / a.kv_heads, kh = h / rep, D = a.dim_p, V = a.vdim_p;
    float *q = sh, *k = q + parts * RT, *g = k + parts * RT, *v = g + parts * RT, *red = v + V;
    for (int i = D + tid; i < parts * RT; i += nthr) q[i] = k[i] = g[i] = 0.f;
    const bool mine = col < V;
    float* S = a.state + ((long)un.slot * a.heads + h) * D * V;
    f32x4 s[RT];
#pragma unroll
    for (int i = 0; i < RT; ++i) s[i] = mmi_load_nt(reinterpret_cast<const f32x4*>(S + (long)min(part + parts * i, D - 1) * V + min(col, V - 4)));
#pragma unroll
    for (int i = 0; i < RT; ++i)
        if (un.fresh || !mine || part + parts * i >= D) s[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    const float* old = nullptr;
    float* now = nullptr;
    if constexpr (DELTA) {
        old = a.conv_state + ((long)un.slot * 2 + un.par) * (a.taps - 1) * a.conv_c;
        now = a.conv_state + ((long)un.slot * 2 + (un.par ^ 1)) * (a.taps - 1) * a.conv_c;
    }
    for (int t = 0; t < un.n; ++t) {
        const long row = un.row0 + t;
        const float* in = a.in + row * a.in_ld;
        // everything the token needs is requested before anything is used: q, k, v and (delta) the decays, one value per thread and round
        f32x4 gt = {0.f, 0.f, 0.f, 0.f}, nw = gt;
        float beta = 0.f;
        if constexpr (DELTA) {
            beta = in[a.b0 + h];
            gt = *reinterpret_cast<const f32x4*>(a.gate + row * a.gate_ld + h * V + min(col, V - 4));
            nw = *reinterpret_cast<const f32x4*>(a.nw + min(col, V - 4));
        }
#pragma unroll 1
        for (int i = tid; i < (DELTA ? 3 : 2) * D + V; i += nthr) {
            if (DELTA && i >= 2 * D + V) {
                g[i - 2 * D - V] = tlm_decay(a, row, h, i - 2 * D - V);
                continue;
            }
            const int c = i < D ? a.q0 + kh * D + i : (i < 2 * D ? a.k0 + kh * D + i - D : a.v0 + h * V + i - 2 * D);
            float x;
            if constexpr (DELTA) x = tlm_silu(tlm_conv<float>(a, old, un.fresh, un.row0, t, c, t + 1 == un.n && (i >= 2 * D || h % rep == 0) ? now : nullptr));      // (the heads of a group share query and key channels)
            else x = in[c];
            if (i < D) q[i] = x;
            else if (i < 2 * D) k[i - D] = x;
            else v[i - 2 * D] = x;
        }
        __syncthreads();
        float qq = 0.f, kk = 0.f, kq = 0.f;                // every wave sums for itself
#pragma unroll 1
        for (int i = lane; i < D; i += 64) {
            qq = mmi_fma(q[i], q[i], qq);
            kk = mmi_fma(k[i], k[i], kk);
            kq = mmi_fma(k[i], q[i], kq);
        }
        kq = tlm_wave_sum(kq);
        float iq = 1.f, ik = 1.f, dec = 1.f;
        if constexpr (DELTA) {
            iq = a.q_scale / sqrtf(tlm_wave_sum(qq) + 1e-6f);
            ik = 1.0f / sqrtf(tlm_wave_sum(kk) + 1e-6f);
            kq *= iq * ik;
            beta = tlm_sigmoid(beta);
        } else {
            dec = a.decay[h * (TLM_CHUNK + 1) + 1];
        }
        f32x4 ak = {0.f, 0.f, 0.f, 0.f}, aq = ak;
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            const int d = part + parts * i;
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
#pragma unroll 4
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
            s[i] += (k[d] * ik) * u;
        }
        if constexpr (DELTA) {
            float ss = o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
            for (int x = 1; x < cgp; x *= 2) ss += mmi_shfl_xor(ss, x);      // (the groups of one row part are neighbours in a wave)
            const float inv = 1.0f / sqrtf(ss / (float)a.vdim + a.eps);
            if (part == 0 && mine) {
#pragma unroll
                for (int e = 0; e < 4; ++e) gt[e] = tlm_sigmoid(gt[e]);
                Tr::store4((typename Tr::elem*)a.out + tlm_index<Tr>(row, h * V + col, a.out_ks), o * inv * nw * gt);
            }
        } else if (part == 0 && mine) {
            *reinterpret_cast<f32x4*>(a.o + (row * a.heads + h) * V + col) = o;
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < RT; ++i) {
        const int d = part + parts * i;
        if (mine && d < D) mmi_store_nt(reinterpret_cast<f32x4*>(S + (long)d * V + col), s[i]);
    }
}

// ------------------------------------------------------------------------------------------------
// chunks: convolutions and unit norms (delta).  grid: chunks, 2 kv_heads + heads; a lane takes 4 channels, a power of two of lanes a token
// ------------------------------------------------------------------------------------------------
inline __global__ __launch_bounds__(256) void k_tlm_conv(TlmLinArgs a, int kgroups, int vgroups) {
    const int y = (int)blockIdx.y;
    const TlmSeg ck = a.chunk[blockIdx.x];
    const int kind = y < a.kv_heads ? 0 : (y < 2 * a.kv_heads ? 1 : 2);
    const int width = kind == 2 ? a.vdim_p : a.dim_p, groups = kind == 2 ? vgroups : kgroups;
    const int c0 = kind == 0 ? a.q0 + y * a.dim_p : (kind == 1 ? a.k0 + (y - a.kv_heads) * a.dim_p : a.v0 + (y - 2 * a.kv_heads) * a.vdim_p);
    const float* old = a.conv_state + ((long)ck.slot * 2 + ck.par) * (a.taps - 1) * a.conv_c;
    float* now = a.conv_state + ((long)ck.slot * 2 + (ck.par ^ 1)) * (a.taps - 1) * a.conv_c;
    const int first = ck.row0 - ck.index * TLM_CHUNK;      // the sequence's first row of this step
    const int c = 4 * ((int)threadIdx.x & (groups - 1)), step = 256 / groups;
    for (int t0 = 0; t0 < ck.n; t0 += step) {              // (every lane of a wave goes round as often)
        const int t = t0 + (int)threadIdx.x / groups;
        f32x4 x = {0.f, 0.f, 0.f, 0.f};
        if (t < ck.n && c < width) {
            x = tlm_conv<f32x4>(a, old, ck.fresh, first, ck.index * TLM_CHUNK + t, c0 + c, ck.last && t + 1 == ck.n ? now : nullptr);
#pragma unroll
            for (int e = 0; e < 4; ++e) x[e] = tlm_silu(x[e]);
        }
        if (kind != 2) {
            float ss = x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
            for (int m = 1; m < groups; m *= 2) ss += mmi_shfl_xor(ss, m);
            x *= (kind == 0 ? a.q_scale : 1.0f) / sqrtf(ss + 1e-6f);
        }
        if (t < ck.n && c < width) *reinterpret_cast<f32x4*>(a.qkv + (long)(ck.row0 + t) * a.conv_c + c0 + c) = x;
    }
}

// ------------------------------------------------------------------------------------------------
// chunks, lightning: P, the decayed queries, the decayed transposed keys.  grid: chunks, heads
// ------------------------------------------------------------------------------------------------
inline __global__ __launch_bounds__(256, 4) void k_tlm_chunk_lightning(TlmLinArgs a) {
    const int tid = (int)threadIdx.x, lane = tid & 63, wave = mmi_uniform(tid >> 6), bl = lane & 15, kq = lane >> 4, h = (int)blockIdx.y;
    const TlmSeg ck = a.chunk[blockIdx.x];
    const int D = a.dim_p;
    const long id = (long)blockIdx.x * a.heads + h;
    MMI_SHARED __attribute__((aligned(16))) float Q[TLM_CHUNK * TLM_PST], K[TLM_CHUNK * TLM_PST], pw[TLM_CHUNK + 1];
    for (int i = tid; i <= TLM_CHUNK; i += 256) pw[i] = a.decay[h * (TLM_CHUNK + 1) + i];
    const float* qp = a.in + (long)ck.row0 * a.in_ld + a.q0 + h * D;
    const float* kp = a.in + (long)ck.row0 * a.in_ld + a.k0 + h * D;
    float *Qg = a.qg + id * TLM_CHUNK * D, *Kt = a.kt + id * TLM_CHUNK * D, *P = a.p + id * (TLM_CHUNK * TLM_CHUNK);
    f32x4 acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int c0 = 0; c0 < D; c0 += 64) {                   // panels of 64 channels (a multiple of 16 in the last one)
        const int cn = min(64, D - c0);
        f32x4 qv[4], kv[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {                      // (rows and columns past the end: a valid address, as zeros)
            const int t = (tid >> 4) + 16 * i, c = min(4 * (tid & 15), cn - 4);
            qv[i] = *reinterpret_cast<const f32x4*>(qp + (long)min(t, ck.n - 1) * a.in_ld + c0 + c);
            kv[i] = *reinterpret_cast<const f32x4*>(kp + (long)min(t, ck.n - 1) * a.in_ld + c0 + c);
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = (tid >> 4) + 16 * i, c = 4 * (tid & 15);
            if (t >= ck.n || c >= cn) qv[i] = kv[i] = f32x4{0.f, 0.f, 0.f, 0.f};
            *reinterpret_cast<f32x4*>(Q + t * TLM_PST + c) = qv[i];
            *reinterpret_cast<f32x4*>(K + t * TLM_PST + c) = kv[i];
            if (c < cn) *reinterpret_cast<f32x4*>(Qg + tlm_tile(t, c0 + c, D / 16)) = qv[i] * pw[t + 1];
        }
        __syncthreads();
        for (int c = 4 * kq; c < cn; c += 16) {
            const u32x4 q = *reinterpret_cast<const u32x4*>(Q + (16 * wave + bl) * TLM_PST + c);
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (j <= wave) acc[j] = TlmF32::mfma(q, *reinterpret_cast<const u32x4*>(K + (16 * j + bl) * TLM_PST + c), acc[j]);
        }
        for (int i = wave; i < cn / 4; i += 4) {           // transposed fragments: 16 channels x 16 tokens
            const int c = 16 * (i >> 2) + bl, t = 16 * (i & 3) + 4 * kq;
            f32x4 v;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = t + e < ck.n ? K[(t + e) * TLM_PST + c] * pw[ck.n - 1 - t - e] : 0.f;
            *reinterpret_cast<f32x4*>(Kt + tlm_tile(c0 + c, t, 4)) = v;
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
        if (j <= wave)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = 16 * wave + 4 * kq + r, s = 16 * j + bl;
                P[tlm_tile(t, s, 4)] = s <= t ? acc[j][r] * pw[t - s] : 0.f;
            }
    for (int d = tid; d < D; d += 256) a.gend[id * D + d] = pw[ck.n];
}

// ------------------------------------------------------------------------------------------------
// chunks, delta: P, W, U0, the decayed queries and transposed keys.  grid: chunks, heads; wave w owns tokens 16 w .. 16 w + 15
// ------------------------------------------------------------------------------------------------
inline size_t tlm_chunk_delta_smem() { return (size_t)(3 * TLM_CHUNK * TLM_PST + 4 * 64 + TLM_CHUNK) * sizeof(float); }
inline __global__ __launch_bounds__(256, 2) void k_tlm_chunk_delta(TlmLinArgs a) {
    MMI_DYN_SHARED(float, sh);
    float *K = sh, *Q = K + TLM_CHUNK * TLM_PST, *G = Q + TLM_CHUNK * TLM_PST;      // [64][TLM_PST] each
    float *tot = G + TLM_CHUNK * TLM_PST, *beta = tot + 4 * 64;                     // [4][64], [64]
    float *A = K, *ti = Q;                                                          // once the panels are done: [64][TLM_PST], [4][16][20]
    const int tid = (int)threadIdx.x, lane = tid & 63, wave = mmi_uniform(tid >> 6), bl = lane & 15, kq = lane >> 4, h = (int)blockIdx.y;
    const TlmSeg ck = a.chunk[blockIdx.x];
    const int D = a.dim_p, V = a.vdim_p, kh = h / (a.heads / a.kv_heads);
    const long id = (long)blockIdx.x * a.heads + h;
    const float* qkv = a.qkv + (long)ck.row0 * a.conv_c;
    float *Wg = a.w + id * TLM_CHUNK * D, *Qg = a.qg + id * TLM_CHUNK * D, *Kt = a.kt + id * TLM_CHUNK * D, *Ug = a.u0 + id * TLM_CHUNK * V;
    float* P = a.p + id * (TLM_CHUNK * TLM_CHUNK);
    if (tid < TLM_CHUNK) beta[tid] = tid < ck.n ? tlm_sigmoid(a.in[(long)(ck.row0 + tid) * a.in_ld + a.b0 + h]) : 0.f;
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
#pragma unroll
                for (int e = 0; e < 4; ++e) gv[e] = tlm_decay(a, ck.row0 + t, h, c0 + c + e);
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
            *reinterpret_cast<f32x4*>(Qg + tlm_tile(t, c0 + c, D / 16)) = *reinterpret_cast<const f32x4*>(Q + t * TLM_PST + c) * f;
            *reinterpret_cast<f32x4*>(Wg + tlm_tile(t, c0 + c, D / 16)) = *reinterpret_cast<const f32x4*>(K + t * TLM_PST + c) * f * beta[t];
        }
        for (int i = wave; i < cn / 4; i += 4) {           // transposed fragments: 16 channels x 16 tokens
            const int c = 16 * (i >> 2) + bl, t = 16 * (i & 3) + 4 * kq;
            float f = 1.f;
            for (int m = (i & 3) + 1; m < 4; ++m) f *= tot[m * 64 + c];
            f32x4 v;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = G[(t + e) * TLM_PST + c] * f;
            *reinterpret_cast<f32x4*>(Kt + tlm_tile(c0 + c, t, 4)) = v;
        }
        if (tid < cn) a.gend[id * D + c0 + tid] = tot[tid] * tot[64 + tid] * tot[128 + tid] * tot[192 + tid];
    }
    __syncthreads();
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
            P[tlm_tile(t, at, 4)] = s <= bl ? y : 0.f;
        }
    }
#pragma unroll
    for (int b = 0; b < 2; ++b)
        if (b < nblk)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = 16 * bi[b] + 4 * kq + r, s = 16 * bj[b] + bl;
                A[t * TLM_PST + s] = -beta[t] * oA[b][r];
                P[tlm_tile(t, s, 4)] = oP[b][r];
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
    // forward substitution by blocks of 16; a wave takes four 16-column strips of [W | U0] at a time
    const int nd = D / 16, ns = nd + V / 16;
    for (int s0 = wave; s0 < ns; s0 += 16) {
        f32x4 x[4][4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int st = min(s0 + 4 * k, ns - 1);        // (past the end: the last strip again, not stored)
            const float* src = st < nd ? Wg : qkv + a.v0 + h * V + 16 * (st - nd) + bl;
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int t = 16 * i + 4 * kq + r;
                    x[k][i][r] = src[st < nd ? tlm_tile(t, 16 * st + bl, nd) : (long)min(t, ck.n - 1) * a.conv_c];
                }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int t = 16 * i + 4 * kq + r;
                    x[k][i][r] = t < ck.n ? x[k][i][r] * (st < nd ? 1.f : beta[t]) : 0.f;
                }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
#pragma unroll
            for (int j = 0; j < i; ++j) {
                const u32x4 av = *reinterpret_cast<const u32x4*>(A + (16 * i + bl) * TLM_PST + 16 * j + 4 * kq);
#pragma unroll
                for (int k = 0; k < 4; ++k) x[k][i] = TlmF32::mfma(av, __builtin_bit_cast(u32x4, x[k][j]), x[k][i]);
            }
            const u32x4 tv = *reinterpret_cast<const u32x4*>(ti + (i * 16 + bl) * 20 + 4 * kq);
#pragma unroll
            for (int k = 0; k < 4; ++k) x[k][i] = TlmF32::mfma(tv, __builtin_bit_cast(u32x4, x[k][i]), f32x4{0.f, 0.f, 0.f, 0.f});
        }
#pragma unroll
        for (int k = 0; k < 4; ++k)
            if (s0 + 4 * k < ns)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int st = s0 + 4 * k;
                    if (st >= nd) *reinterpret_cast<f32x4*>(Ug + (((long)i * (V / 16) + st - nd) * 64 + lane) * 4) = x[k][i];
                    else
#pragma unroll
                        for (int r = 0; r < 4; ++r) Wg[tlm_tile(16 * i + 4 * kq + r, 16 * st + bl, nd)] = x[k][i][r];
                }
    }
}

// ------------------------------------------------------------------------------------------------
// chunks: the walk over a sequence's chunks.  One workgroup per (sequence, head, 16 columns of S).  Wave w owns token block w of every chunk
// and a quarter of the rows of S, in the layout the matrix core leaves them in, which is also the layout it takes them as an operand; S and
// U go round through LDS.
// grid: 8 x ceil(sequences x heads / 8) x vdim_p / 16, the column blocks of one head on one XCD (they read the same W, Qg, Kt, P)
// ------------------------------------------------------------------------------------------------
__device__ __forceinline__ float tlm_f(unsigned v) { return __builtin_bit_cast(float, v); }
template <bool DELTA, int NDW>
__global__ __launch_bounds__(256, 1) void k_tlm_chunk_scan(TlmLinArgs a, int n_units) {
    constexpr int ND = 4 * NDW;                            // 16-row blocks of S; past the model's: zeros
    MMI_SHARED __attribute__((aligned(16))) f32x4 Sl[ND][64], Ul[4][64];
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
        Sl[d][lane] = s[i];
    }
    __syncthreads();
    struct Frags {
        u32x4 w[DELTA ? ND : 1], q[ND], k[NDW][4], p[4];
        f32x4 u, g[NDW];
    };
    auto load = [&](Frags& f, int c) __attribute__((always_inline)) {      // (blocks past the end: a valid address, against rows of S that stay zero)
        const long id = (long)(un.chunk0 + c) * a.heads + h;
        const int n = min(TLM_CHUNK, un.n - c * TLM_CHUNK);
#pragma unroll
        for (int d = 0; d < ND; ++d) {
            const long at = id * TLM_CHUNK * D + (((long)wave * nd + min(d, nd - 1)) * 64 + lane) * 4;
            if constexpr (DELTA) f.w[d] = *reinterpret_cast<const u32x4*>(a.w + at);
            f.q[d] = *reinterpret_cast<const u32x4*>(a.qg + at);
        }
#pragma unroll
        for (int i = 0; i < NDW; ++i) {
            const int d = min(wave * NDW + i, nd - 1);
#pragma unroll
            for (int t = 0; t < 4; ++t) f.k[i][t] = *reinterpret_cast<const u32x4*>(a.kt + id * TLM_CHUNK * D + (((long)d * 4 + t) * 64 + lane) * 4);
            f.g[i] = *reinterpret_cast<const f32x4*>(a.gend + id * D + 16 * d + 4 * kq);
        }
#pragma unroll
        for (int t = 0; t < 4; ++t)
            f.p[t] = *reinterpret_cast<const u32x4*>(a.p + id * (TLM_CHUNK * TLM_CHUNK) + ((wave * 4 + min(t, wave)) * 64 + lane) * 4);
        if constexpr (DELTA) {
            f.u = *reinterpret_cast<const f32x4*>(a.u0 + id * TLM_CHUNK * V + (((long)wave * ncb + cb) * 64 + lane) * 4);
        } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int tok = 16 * wave + 4 * kq + r;
                const float v = a.in[(long)(un.row0 + c * TLM_CHUNK + min(tok, n - 1)) * a.in_ld + a.v0 + h * V + 16 * cb + bl];
                f.u[r] = tok < n ? v : 0.f;
            }
        }
    };
    auto chunk = [&](const Frags& f, int c) __attribute__((always_inline)) {
        const int n = min(TLM_CHUNK, un.n - c * TLM_CHUNK);
        // four independent sums go round, one step of four each: a matrix instruction never waits for the one before it
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        f32x4 x0 = zero, x1 = zero, o0 = zero, o1 = zero;
        if constexpr (!DELTA) Ul[wave][lane] = f.u;
#pragma unroll
        for (int d = 0; d < ND; d += 2) {
            const f32x4 sa = Sl[d][lane], sb = Sl[d + 1][lane];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                if constexpr (DELTA) {
                    x0 = mmi_mfma_f32_16x16x4(tlm_f(f.w[d][e]), sa[e], x0);
                    x1 = mmi_mfma_f32_16x16x4(tlm_f(f.w[d + 1][e]), sb[e], x1);
                }
                o0 = mmi_mfma_f32_16x16x4(tlm_f(f.q[d][e]), sa[e], o0);
                o1 = mmi_mfma_f32_16x16x4(tlm_f(f.q[d + 1][e]), sb[e], o1);
            }
        }
        if constexpr (DELTA) Ul[wave][lane] = f.u - (x0 + x1);
        __syncthreads();
        f32x4 u[4], sh[NDW];
#pragma unroll
        for (int t = 0; t < 4; ++t) u[t] = Ul[t][lane];
#pragma unroll
        for (int i = 0; i < NDW; ++i) {
            s[i] *= f.g[i];
            sh[i] = zero;
        }
#pragma unroll
        for (int t = 0; t < 4; t += 2)
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
                for (int i = 0; i < NDW; ++i) {
                    s[i] = mmi_mfma_f32_16x16x4(tlm_f(f.k[i][t][e]), u[t][e], s[i]);
                    sh[i] = mmi_mfma_f32_16x16x4(tlm_f(f.k[i][t + 1][e]), u[t + 1][e], sh[i]);
                }
#pragma unroll
        for (int i = 0; i < NDW; ++i) {
            s[i] += sh[i];
            if (wave * NDW + i >= nd) s[i] = zero;
            Sl[wave * NDW + i][lane] = s[i];
        }
#pragma unroll
        for (int t = 0; t < 4; t += 2)                     // (blocks right of the diagonal: zeros instead)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                o0 = mmi_mfma_f32_16x16x4(t <= wave ? tlm_f(f.p[t][e]) : 0.f, u[t][e], o0);
                o1 = mmi_mfma_f32_16x16x4(t + 1 <= wave ? tlm_f(f.p[t + 1][e]) : 0.f, u[t + 1][e], o1);
            }
        const f32x4 o = o0 + o1;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int tok = 16 * wave + 4 * kq + r;
            if (tok < n) a.o[((long)(un.row0 + c * TLM_CHUNK + tok) * a.heads + h) * V + 16 * cb + bl] = o[r];
        }
        __syncthreads();
    };
    if constexpr (NDW <= 2) {
        // the next chunk's operands are on their way while a chunk is computed (the last one asks for itself again)
        Frags fa, fb;
        load(fa, 0);
        for (int c = 0; c < un.n_chunks; c += 2) {
            load(fb, min(c + 1, un.n_chunks - 1));
            mmi_sched_barrier();
            chunk(fa, c);
            if (c + 1 == un.n_chunks) break;
            load(fa, min(c + 2, un.n_chunks - 1));
            mmi_sched_barrier();
            chunk(fb, c + 1);
        }
    } else {
        Frags f;
        for (int c = 0; c < un.n_chunks; ++c) {
            load(f, c);
            chunk(f, c);
        }
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
        const f32x4 w = *reinterpret_cast<const f32x4*>(a.nw + (per_head ? c - h * V : c));
        f32x4 g = *reinterpret_cast<const f32x4*>(a.gate + row * a.gate_ld + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) g[e] = tlm_sigmoid(g[e]);
        Tr::store4((typename Tr::elem*)a.out + tlm_index<Tr>(row, c, a.out_ks), *reinterpret_cast<const f32x4*>(o + c) * inv[h] * w * g);
    }
}
