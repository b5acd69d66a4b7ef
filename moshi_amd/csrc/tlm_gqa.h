// Grouped attention of the token language models: query heads that share key/value heads, keys and values in pages of 64 tokens.
//
//   key cache    [page][kv head] blocks of 64 rows (keys) in the fragment order of tlm_index, k = dimension
//   value cache  tlm_value_index: the transposed operand of the value product, written element by element by the projection's epilogue
//   columns      (token, query head of the group) pairs of one sequence and one key/value head: column c = token c / rep, head c % rep
//
// D is a template bound on both the query/key and the value size (64, 128, 256); fragments past the model's sizes repeat a valid address
// against zero query fragments, or are dropped at the end.  A window that keeps the first positions walks two runs of key blocks.
#pragma once
#include "tlm_kernels.h"

struct TlmGqaArgs {
    const void* q;                       // packed rows token * heads + head
    const void *kc, *vc;
    void* out; int out_ks;               // packed rows token, columns head * 16 nd + d
    int heads, kv_heads, rep, q_ks, nd;
    TlmMask mask;
    int sink;                            // one is added to the denominator
    int n_entries, n_tiles, nsplit;
    const int* tile0;                    // [entries + 1] first column tile (k_tlm_gqa_tile: column group) of each entry
    const int* erow0; const int* elen; const int* epos0; const int* eslot;
    TlmPages pages;
    float* po;                           // nsplit > 1: [tile][kv head][split][nd][64] f32x4 un-normalised sums
    float* pml;                          // [tile][kv head][split][2][16]: running maximum, sum of weights
};

// the key blocks (32 keys) that columns at positions plo .. phi read: [0, n0) and [b0, b1)
struct TlmWalk {
    int n0, b0, b1;
    __device__ __forceinline__ TlmWalk(const TlmMask& m, int plo, int phi) {
        const int klo = m.window > 0 && plo - m.window + 1 > 0 ? plo - m.window + 1 : 0;
        b0 = klo / 32;
        b1 = phi / 32 + 1;
        n0 = m.window > 0 ? min(b0, (m.keep + 31) / 32) : 0;
    }
    __device__ __forceinline__ int size() const { return n0 + b1 - b0; }
    __device__ __forceinline__ int block(int i) const { return i < n0 ? i : b0 + i - n0; }
};

template <class Tr, int D>
struct TlmGqa {
    static constexpr int NK = D / Tr::KSTEP, ND = D / 16, NB = 32 / Tr::KSTEP;      // k-steps; value blocks; fragments per value block and 32 keys
    static constexpr int F = 2 * NK + ND * NB;                                      // fragments per 32 keys
    // fragment f of key block kb: keys 0-15 and 16-31 of every k-step, then the values
    static __device__ __forceinline__ const u32x4* at(const TlmGqaArgs& a, long pg, int kb, int f) {      // pg = page * kv_heads + kv head
        if (f < 2 * NK) return (const u32x4*)a.kc + ((pg * 4 + (kb & 1) * 2 + (f & 1)) * a.q_ks + min(f >> 1, a.q_ks - 1)) * 64;
        const int d = (f - 2 * NK) / NB, b = (f - 2 * NK) % NB;
        return (const u32x4*)a.vc + ((pg * (TLM_PAGE / Tr::KSTEP) + (kb & 1) * NB + b) * a.nd + min(d, a.nd - 1)) * 64;
    }
    static __device__ __forceinline__ u32x4 query(const TlmGqaArgs& a, const TlmCols& c, int g, int col, int kq, int s) {
        const int t = col / a.rep;
        const long row = (long)(a.erow0[c.entry] + t) * a.heads + g * a.rep + col - t * a.rep;
        const u32x4 zero = {0u, 0u, 0u, 0u};
        return s < a.q_ks ? ((const u32x4*)a.q)[((row >> 4) * a.q_ks + s) * 64 + kq * 16 + (row & 15)] : zero;
    }
    static __device__ __forceinline__ TlmCols find(const TlmGqaArgs& a, int tile) {
        TlmCols c = tlm_find_tile(a, tile);
        c.ncol = a.elen[c.entry] * a.rep;
        return c;
    }
    static __device__ __forceinline__ void store(const TlmGqaArgs& a, const TlmCols& c, int g, int bl, int kq, int d, f32x4 v) {
        const int col = c.c0 + bl;
        if (col >= c.ncol) return;
        const int t = col / a.rep, head = g * a.rep + col - t * a.rep;
        Tr::store4((typename Tr::elem*)a.out + tlm_index<Tr>(a.erow0[c.entry] + t, (head * a.nd + d) * 16 + 4 * kq, a.out_ks), v);
    }
};

// Few column tiles (decoding): the four waves of a workgroup share one column tile, each takes every 4th key block straight from the
// cache - the block after it is requested fragment by fragment as the registers fall free - and their sums meet in LDS.
// grid: column tiles (rounded up to 8), kv heads, splits of the keys (k_tlm_gqa_combine)
template <class Tr, int D>
__global__ __launch_bounds__(256, Tr::V == 8 && D <= 128 ? 2 : 1) void k_tlm_gqa(TlmGqaArgs a) {
    typedef TlmGqa<Tr, D> P;
    constexpr int WK = 4, NK = P::NK, ND = P::ND, NB = P::NB, F = P::F, VG = 4 * NB;
    MMI_SHARED float ml[2][4][16];
    MMI_SHARED __attribute__((aligned(16))) f32x4 ob[4 * 8 * 64];
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15, kq = lane >> 4;
    const int tile = (int)blockIdx.x, g = (int)blockIdx.y, split = (int)blockIdx.z;
    const TlmCols c = P::find(a, tile);
    const int col = c.c0 + bl < c.ncol ? c.c0 + bl : c.ncol - 1;
    const int pos0 = a.epos0[c.entry];
    const int pc = pos0 + col / a.rep;                             // position of this lane's column
    const TlmWalk w(a.mask, pos0 + c.c0 / a.rep, pos0 + min(c.c0 + 15, c.ncol - 1) / a.rep);
    int i0 = 0, i1 = w.size();
    if (a.nsplit > 1) {
        const int per = (i1 + a.nsplit - 1) / a.nsplit;
        i0 = min(i1, split * per);
        i1 = min(i1, i0 + per);
    }
    const int* bt = a.pages.table + (long)a.eslot[c.entry] * a.pages.ld;
    u32x4 q[NK];
#pragma unroll
    for (int s = 0; s < NK; ++s) q[s] = P::query(a, c, g, col, kq, s);
    f32x4 acc[ND];
#pragma unroll
    for (int d = 0; d < ND; ++d) acc[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = a.sink ? 0.f : -1e30f, l = 0.f;                      // (a sink of score 0 takes part in the maximum)
    u32x4 fr[F];
    int nb = 0;                                                    // block the registers are being loaded with
    long pg = 0;
    auto aim = [&](int i) __attribute__((always_inline)) {         // (past the end: the last block again)
        nb = w.block(min(i, i1 - 1));
        pg = (long)tlm_page(a.pages, bt, nb >> 1) * a.kv_heads + g;
    };
    auto load = [&](int f) __attribute__((always_inline)) { fr[f] = mmi_load_nt(P::at(a, pg, nb, f) + lane); };
    if (i0 + wave < i1) {
        aim(i0 + wave);
#pragma unroll
        for (int f = 0; f < F; ++f) load(f);
    }
    for (int i = i0 + wave; i < i1; i += WK) {
        const int kb = nb;
        aim(i + WK);
        f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
        for (int k = 0; k < NK; ++k) {
            s0 = Tr::mfma(fr[2 * k], q[k], s0);
            s1 = Tr::mfma(fr[2 * k + 1], q[k], s1);
        }
#pragma unroll
        for (int f = 0; f < 2 * NK; ++f) load(f);
        mmi_sched_barrier();
        u32x4 pf[NB];
        const float al = tlm_softmax_block<Tr>(a.mask, s0, s1, kb * 32 + 4 * kq, pc - (kb * 32 + 4 * kq), m, l, pf);
        if (mmi_any(al != 1.f)) {
#pragma unroll
            for (int d = 0; d < ND; ++d) acc[d] *= al;
        }
#pragma unroll
        for (int f0 = 2 * NK; f0 < F; f0 += VG) {
#pragma unroll
            for (int f = f0; f < f0 + VG; ++f) acc[(f - 2 * NK) / NB] = Tr::mfma(fr[f], pf[(f - 2 * NK) % NB], acc[(f - 2 * NK) / NB]);
#pragma unroll
            for (int f = f0; f < f0 + VG; ++f) load(f);
            mmi_sched_barrier();
        }
    }
    l += mmi_shfl_xor(l, 16);
    l += mmi_shfl_xor(l, 32);
    if (kq == 0) {
        ml[0][wave][bl] = m;
        ml[1][wave][bl] = l;
    }
    __syncthreads();
    float M = -1e30f, L = 0.f;
#pragma unroll
    for (int v = 0; v < WK; ++v) M = fmaxf(M, ml[0][v][bl]);
#pragma unroll
    for (int v = 0; v < WK; ++v) L += ml[1][v][bl] * exp2f(ml[0][v][bl] - M);
    const float f = exp2f(m - M);
    const float inv = a.nsplit > 1 ? 1.f : 1.0f / (a.sink ? L + exp2f(-M) : L);
    const long part = ((long)tile * a.kv_heads + g) * a.nsplit + split;
#pragma unroll
    for (int d0 = 0; d0 < ND; d0 += 8) {
        if (d0 >= a.nd) break;
        if (d0) __syncthreads();
#pragma unroll
        for (int d = 0; d < 8; ++d)
            if (d0 + d < ND) ob[(wave * 8 + d) * 64 + lane] = acc[d0 + d < ND ? d0 + d : 0] * f;
        __syncthreads();
#pragma unroll
        for (int d = wave; d < 8; d += WK) {
            if (d0 + d >= a.nd) break;
            f32x4 v = ob[d * 64 + lane];
#pragma unroll
            for (int o = 1; o < WK; ++o) v += ob[(o * 8 + d) * 64 + lane];
            if (a.nsplit > 1) *reinterpret_cast<f32x4*>(a.po + ((part * a.nd + d0 + d) * 64 + lane) * 4) = v;
            else P::store(a, c, g, bl, kq, d0 + d, v * inv);
        }
    }
    if (a.nsplit > 1 && wave == 0 && kq == 0) {
        a.pml[part * 32 + bl] = M;
        a.pml[part * 32 + 16 + bl] = L;
    }
}

// the splits (at most 16) of one column tile -> output; a wave takes one 16-wide block of values, all its loads in flight together.
// grid: column tiles, kv heads, blocks / 4
template <class Tr>
__global__ __launch_bounds__(256) void k_tlm_gqa_combine(TlmGqaArgs a) {
    typedef TlmGqa<Tr, 64> P;                                      // (nothing below depends on the bound)
    constexpr int MAXS = 16;
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15, kq = lane >> 4;
    const int tile = (int)blockIdx.x, g = (int)blockIdx.y, d = wave + 4 * (int)blockIdx.z;
    if (d >= a.nd) return;
    const long part = ((long)tile * a.kv_heads + g) * a.nsplit;
    float m[MAXS], l[MAXS];
    f32x4 v[MAXS];
#pragma unroll
    for (int s = 0; s < MAXS; ++s) {                               // (past the end: the last split again, with weight zero)
        const long p = part + min(s, a.nsplit - 1);
        m[s] = a.pml[p * 32 + bl];
        l[s] = a.pml[p * 32 + 16 + bl];
        v[s] = *reinterpret_cast<const f32x4*>(a.po + ((p * a.nd + d) * 64 + lane) * 4);
    }
    const TlmCols c = P::find(a, tile);
    float M = m[0], L = 0.f;
#pragma unroll
    for (int s = 1; s < MAXS; ++s) M = fmaxf(M, m[s]);
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < MAXS; ++s) {
        const float f = s < a.nsplit ? exp2f(m[s] - M) : 0.f;
        L = mmi_fma(l[s], f, L);
        o += v[s] * f;
    }
    P::store(a, c, g, bl, kq, d, o * (1.0f / (a.sink ? L + exp2f(-M) : L)));
}

// Many columns (prompts): four waves x QT column tiles of one sequence and kv head walk the same keys; a block's fragments are staged
// through LDS once for all of them, the next block in flight in registers.  grid: column groups (64 QT columns), kv heads
template <class Tr, int D>
struct TlmGqaTile {
    static constexpr int QT = Tr::V == 8 || D <= 128 ? 2 : 1, NF = TlmGqa<Tr, D>::F;
    static constexpr size_t smem() { return (size_t)2 * NF * 1024; }
};
template <class Tr, int D>
__global__ __launch_bounds__(256, Tr::V == 8 && D <= 128 ? 2 : 1) void k_tlm_gqa_tile(TlmGqaArgs a) {
    typedef TlmGqa<Tr, D> P;
    constexpr int NK = P::NK, ND = P::ND, QT = TlmGqaTile<Tr, D>::QT, NF = P::F, NI = NF / 4;
    typedef TlmAttnStream<Tr, ND, 0, QT, (ND >= 16 ? 4 : 8)> S;
    static_assert(NF % 4 == 0 && S::F == NF, "whole fragments per wave, the stream's order");
    MMI_DYN_SHARED(u32x4, lds);
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15, kq = lane >> 4;
    const int g = (int)blockIdx.y;
    TlmCols c = P::find(a, (int)gridDim.x - 1 - (int)blockIdx.x);  // (tile0 counts groups of 64 QT columns here; the last see most keys: they start first)
    c.c0 *= 4 * QT;
    const int pos0 = a.epos0[c.entry];
    const TlmWalk w(a.mask, pos0 + c.c0 / a.rep, pos0 + min(c.c0 + 64 * QT - 1, c.ncol - 1) / a.rep);
    const int n = w.size();
    const int* bt = a.pages.table + (long)a.eslot[c.entry] * a.pages.ld;
    u32x4 q[QT][NK];
    S sm;
    sm.clear(a.sink ? 0.f : -1e30f);
    int pc[QT], c0[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        c0[t] = c.c0 + (wave * QT + t) * 16;
        const int col = c0[t] + bl < c.ncol ? c0[t] + bl : c.ncol - 1;
        pc[t] = pos0 + col / a.rep;
#pragma unroll
        for (int s = 0; s < NK; ++s) q[t][s] = P::query(a, c, g, col, kq, s);
    }
    u32x4 st[2][NI];                                               // wave w brings fragments w, w + 4, ..; two blocks ahead of their use
    long pg = (long)tlm_page(a.pages, bt, w.block(0) >> 1) * a.kv_heads + g;      // page of the block fetched next
    auto fetch = [&](int set, int i) __attribute__((always_inline)) {      // (past the end: the last block again)
        const int kb = w.block(min(i, n - 1));
#pragma unroll
        for (int f = 0; f < NI; ++f) st[set][f] = P::at(a, pg, kb, wave + 4 * f)[lane];
        pg = (long)tlm_page(a.pages, bt, w.block(min(i + 1, n - 1)) >> 1) * a.kv_heads + g;
    };
    auto stage = [&](int buf) __attribute__((always_inline)) {
#pragma unroll
        for (int f = 0; f < NI; ++f) lds[(buf * NF + wave + 4 * f) * 64 + lane] = st[buf][f];
    };
    auto block = [&](int i, int buf) __attribute__((always_inline)) {      // block i in LDS buffer `buf`; i + 1 in register set buf ^ 1
        fetch(buf, i + 2);
        mmi_sched_barrier();
        const int kb = w.block(min(i, n - 1));
        const u32x4* base = lds + buf * NF * 64 + lane;
        auto at = [&](int f) __attribute__((always_inline)) -> const u32x4* { return base + f * 64; };
        auto qf = [&](int t, int k) __attribute__((always_inline)) { return q[t][k]; };
        int d0[QT];
#pragma unroll
        for (int t = 0; t < QT; ++t) d0[t] = pc[t] - (kb * 32 + 4 * kq);
        sm.load(0, 0, at);
#pragma unroll
        for (int s = 0; s < S::NG; ++s) {
            if (s + 1 < S::NG) sm.load((s + 1) & 1, s + 1, at);
            mmi_sched_barrier();
            sm.use(a.mask, qf, s & 1, s, kb * 32 + 4 * kq, d0);
        }
        stage(buf ^ 1);
        __syncthreads();
    };
    fetch(0, 0);
    fetch(1, 1);
    stage(0);
    __syncthreads();
    for (int i = 0; i < n; i += 2) {
        block(i, 0);
        if (i + 1 < n) block(i + 1, 1);
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        float l = sm.l[t];
        l += mmi_shfl_xor(l, 16);
        l += mmi_shfl_xor(l, 32);
        const float inv = 1.0f / (a.sink ? l + exp2f(-sm.m[t]) : l);
        TlmCols o = c;
        o.c0 = c0[t];
#pragma unroll
        for (int d = 0; d < ND; ++d)
            if (d < a.nd) P::store(a, o, g, bl, kq, d, sm.acc[t][d] * inv);
    }
}
