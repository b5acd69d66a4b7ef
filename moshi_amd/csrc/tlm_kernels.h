// Kernels of the token language models (tlm_engine.hip): decoder-only networks over token ids whose layers are described by data
// (mmi_tlm_cfg), served from a paged cache and per-sequence recurrent state, any mixture of prompt portions and single tokens per step.
//
// Every kernel is written once for two number formats: TlmBf16 (bf16 operands on v_mfma_f32_16x16x32_bf16, fp32 accumulation) and
// TlmF32 (fp32 operands on v_mfma_f32_16x16x4_f32, an exact fma chain).  Positions, angles, attention scores and weights, norms, the
// residual stream, gates and recurrent state are fp32 in both.
//
// Data layout in HBM
//   fragment     64 lanes x 16 bytes: 16 rows x KSTEP reduction indices (bf16: 32, fp32: 16); lane (i, kq) = 16 kq + i holds row i,
//                k = V kq .. V kq + V - 1 (V = 8 bf16 / 4 fp32).  It is the A operand (row = output feature), the B operand (row = token)
//                and, at fp32, four 16x16x4 steps at once: element e of every lane is one step (any k order serves, both operands use it).
//   weights      Wp[n-tile][k-step][lane][V]            (16-row tiles, zero padded; the layout of the Moshi LM's 16-row tile)
//   activations  Xp[row / 16][k-step][lane][V]          (tlm_index; written by the producing epilogue)
//   key cache    the same matrix with row = 64 page + offset: k = latent, then the rotated key part
//                There is no second copy for the values (the value IS the latent): the transposed operand of the value product comes out
//                of the matrix core, K x identity (TlmFlip) - lane (d, kq) of its accumulators holds keys 4 kq .. 4 kq + 3, exactly the
//                keys whose scores the same lane holds after S = K Q^T, so the softmax weights become an operand without leaving the lane.
//   residual     x[token][ld] fp32
#pragma once
#include "mmi_common.h"

struct TlmBf16 {
    typedef uint16_t elem;
    static constexpr int V = 8, KSTEP = 32;
    static __device__ __forceinline__ f32x4 mfma(u32x4 a, u32x4 b, f32x4 c) { return mmi_mfma_bf16_16x16x32(a, b, c); }
    static __device__ __forceinline__ uint16_t cvt(float v) { return mmi_f32_to_bf16(v); }
    static __device__ __forceinline__ void store4(uint16_t* p, f32x4 v) {
        u32x2 o = {mmi_pack_bf16x2(v[0], v[1]), mmi_pack_bf16x2(v[2], v[3])};
        *reinterpret_cast<u32x2*>(p) = o;
    }
    static __device__ __forceinline__ void store2(uint16_t* p, float a, float b) { *reinterpret_cast<uint32_t*>(p) = mmi_pack_bf16x2(a, b); }
};
struct TlmF32 {
    typedef float elem;
    static constexpr int V = 4, KSTEP = 16;
    static __device__ __forceinline__ f32x4 mfma(u32x4 a, u32x4 b, f32x4 c) {
        const f32x4 fa = __builtin_bit_cast(f32x4, a), fb = __builtin_bit_cast(f32x4, b);
#pragma unroll
        for (int e = 0; e < 4; ++e) c = mmi_mfma_f32_16x16x4(fa[e], fb[e], c);
        return c;
    }
    static __device__ __forceinline__ float cvt(float v) { return v; }
    static __device__ __forceinline__ void store4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
    static __device__ __forceinline__ void store2(float* p, float a, float b) { *reinterpret_cast<f32x2*>(p) = f32x2{a, b}; }
};

// element (row, k) of a fragment-packed matrix with `ks` k-steps per row tile
template <class Tr>
MMI_HD long tlm_index(long row, int k, int ks) {
    return (((row >> 4) * ks + k / Tr::KSTEP) * 64 + ((k % Tr::KSTEP) / Tr::V) * 16 + (row & 15)) * Tr::V + k % Tr::V;
}

constexpr int TLM_PAGE = 64;         // tokens per cache page

__device__ __forceinline__ float tlm_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float tlm_wave_sum(float x) {
    x = mmi_group_sum<16>(x);
    x += mmi_shfl_xor(x, 16);
    x += mmi_shfl_xor(x, 32);
    return x;
}

// ------------------------------------------------------------------------------------------------
// weight import: bf16 checkpoint tensor -> fragments, through a row and a column map (-1 = zero padding).  Source element
// (row r, column c) is src[r * sr + c * sc], so a transposed operand is the same call with the strides exchanged.
// ------------------------------------------------------------------------------------------------
template <class Tr>
__global__ void k_tlm_pack(const uint16_t* __restrict__ src, long sr, long sc, const int* __restrict__ rowmap, const int* __restrict__ colmap,
                           typename Tr::elem* __restrict__ dst, int NT, int KS, int tmul, int toff, int keep) {
    const long idx = (long)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= (long)NT * KS * 64 * Tr::V) return;
    const int e = (int)(idx % Tr::V);
    const long f = idx / Tr::V;
    const int lane = (int)(f & 63);
    const int ks = (int)((f >> 6) % KS), nt = (int)((f >> 6) / KS);
    const int r = rowmap[nt * 16 + (lane & 15)];
    if (r < 0 && keep) return;                     // (rows another call has filled)
    const int c = colmap[ks * Tr::KSTEP + (lane >> 4) * Tr::V + e];
    const uint16_t h = (r < 0 || c < 0) ? (uint16_t)0 : src[(long)r * sr + (long)c * sc];
    const long at = (((long)nt * tmul + toff) * KS + ks) * 64 * Tr::V + (long)lane * Tr::V + e;      // tile nt of this call is tile nt * tmul + toff of the matrix
    if constexpr (Tr::V == 8) dst[at] = h;
    else dst[at] = mmi_bf16_to_f32(h);
}
// bf16 vector -> fp32, gathered through a map, zero where the map is negative
__global__ void k_tlm_vec(const uint16_t* __restrict__ src, const int* __restrict__ map, float* __restrict__ dst, int n) {
    const int i = (int)(blockIdx.x * blockDim.x + threadIdx.x);
    if (i < n) dst[i] = map[i] < 0 ? 0.f : mmi_bf16_to_f32(src[map[i]]);
}

// ------------------------------------------------------------------------------------------------
// step preparation
// ------------------------------------------------------------------------------------------------
struct TlmRope { const float* freq; int half, ld; float* out; };      // out [row][ld][2]: (cos, sin), (1, 0) past `half`
struct TlmPrepArgs {
    int T, n_ropes;
    const int* n_updates;
    const int* htok;          // token per row; negative: the token last sampled for the row's slot
    const int* pos;
    const int* rslot;
    const int* last_tok;      // [slots]
    int* tok;
    const int* updates;       // (block-table index, page) pairs
    int* block_table;
    const TlmRope* rope;
    int buckets; long mul_prev, mul_cur;       // bigram embedding (buckets 0: none)
    const int* prev;          // per row: -1 first token of its sequence, -2 the row before it, otherwise the index of the token in prev_tok
    const int* next;          // per row: where in prev_tok its token goes (the last of an entry), or -1
    int* prev_tok;            // [slots][2]: a step reads one copy and writes the other
    int* brow;                // out: row of the bigram table
};
__global__ void k_tlm_prepare(TlmPrepArgs a) {
    const int i0 = (int)(blockIdx.x * blockDim.x + threadIdx.x), n = (int)(gridDim.x * blockDim.x);
    for (int i = i0; i < *a.n_updates; i += n) a.block_table[a.updates[2 * i]] = a.updates[2 * i + 1];
    for (int i = i0; i < a.T; i += n) {
        const int t = a.htok[i] >= 0 ? a.htok[i] : a.last_tok[a.rslot[i]];
        a.tok[i] = t;
        if (a.buckets > 0) {
            const int w = a.prev[i];
            int b = a.buckets;
            if (w != -1) {
                const int p = w >= 0 ? a.prev_tok[w] : (a.htok[i - 1] >= 0 ? a.htok[i - 1] : a.last_tok[a.rslot[i]]);
                b = (int)(((long)p * a.mul_prev + (long)t * a.mul_cur) % a.buckets);
                if (b < 0) b += a.buckets;
            }
            a.brow[i] = b;
            if (a.next[i] >= 0) a.prev_tok[a.next[i]] = t;
        }
    }
    for (int r = 0; r < a.n_ropes; ++r) {
        const TlmRope q = a.rope[r];
        for (long i = i0; i < (long)a.T * q.ld; i += n) {
            const int row = (int)(i / q.ld), j = (int)(i % q.ld);
            float c = 1.f, s = 0.f;
            if (j < q.half) {
                const float ang = (float)a.pos[row] * q.freq[j];
                c = cosf(ang);
                s = sinf(ang);
            }
            q.out[2 * i] = c;
            q.out[2 * i + 1] = s;
        }
    }
}

// Token-table routing: the experts of a row are table[token][0 .. top).  One workgroup per routed layer sorts the step's
// (row, choice) pairs by expert - the order inside an expert is irrelevant, every pair is computed and stored on its own - and cuts
// each expert's run into tiles of `tile` pairs.
struct TlmRouteLayer { const int* table; int experts, top; };
struct TlmRouteArgs {
    const TlmRouteLayer* layers;
    const int* tok;
    int T, tile;
    int* list;                // [layer][list_ld] pair ids row * top + choice, by expert
    long list_ld;
    int* tiles;               // [layer][tile_ld][3]: expert, first pair, pairs
    long tile_ld;
    int* n_tiles;             // [layer]
};
__global__ __launch_bounds__(1024) void k_tlm_route(TlmRouteArgs a) {
    MMI_DYN_SHARED(unsigned, cnt);                       // [experts] pair counts, then [experts] insertion points
    const TlmRouteLayer L = a.layers[blockIdx.x];
    const int E = L.experts, top = L.top, tid = (int)threadIdx.x, nthr = (int)blockDim.x;
    unsigned* at = cnt + E;
    for (int e = tid; e < E; e += nthr) cnt[e] = 0u;
    __syncthreads();
    const int n = a.T * top;
    for (int i = tid; i < n; i += nthr) mmi_atomic_add(&cnt[L.table[(long)a.tok[i / top] * top + i % top]], 1u);
    __syncthreads();
    if (tid == 0) {
        unsigned s = 0;
        int nt = 0;
        int* tl = a.tiles + (long)blockIdx.x * a.tile_ld * 3;
        for (int e = 0; e < E; ++e) {
            const int c = (int)cnt[e];
            at[e] = s;
            for (int o = 0; o < c; o += a.tile) {
                tl[3 * nt] = e;
                tl[3 * nt + 1] = (int)s + o;
                tl[3 * nt + 2] = c - o < a.tile ? c - o : a.tile;
                ++nt;
            }
            s += (unsigned)c;
        }
        a.n_tiles[blockIdx.x] = nt;
    }
    __syncthreads();
    int* list = a.list + (long)blockIdx.x * a.list_ld;
    for (int i = tid; i < n; i += nthr) list[mmi_atomic_add(&at[L.table[(long)a.tok[i / top] * top + i % top]], 1u)] = i;
}

// ------------------------------------------------------------------------------------------------
// residual update + grouped RMS norm: one workgroup per row
//   x <- x + ls1 * sum_p mix[p] + ls2 * (1 / top) * sum_choice sum_p dn[p]   (the split-K partials of the two sublayers' last products;
//        no ls: factor 1), or x <- sum_p mix[p] (`replace`: the product at the start of a repeated pass)
//   x <- emb[token] (first layer) or x + emb[token] (start of a repeated pass); x <- x + vec; then h = norm(x) * w -> packed operand, and
//   a second one with weights of its own; `raw`: x itself as a packed operand
//   emb[token] = table[token] * scale + bigram[row of (previous, token)] + pos[position]
// ------------------------------------------------------------------------------------------------
enum { TLM_EMB_NONE = 0, TLM_EMB_SET = 1, TLM_EMB_ADD = 2 };
struct TlmEmbArgs {
    const uint16_t* table; const int* tok; float scale;
    const uint16_t* bigram; const int* brow;       // or null
    const uint16_t* pos; const int* at;            // or null
};
struct TlmResidArgs {
    float* x;
    int width, ld;                       // ld: row stride of x, mix, dn (width rounded up to 16)
    const float* mix; int mix_p; long mix_ps; const float* ls1; int replace;
    const float* dn; int dn_p; long dn_ps; int top; const float* ls2;
    TlmEmbArgs emb; int emb_mode;
    const float* vec;
    float* tap;                          // copy of the residual stream before the embedding is added again, or null
    const float* w; int groups; float eps;
    void* out; int KS;                   // packed; null: no norm
    const float* w2; void* out2;
    void* raw; int raw_ks;               // packed x, or null
    void* emb_out; int emb_k0;           // TLM_EMB_SET: packed copy of the embedding from column emb_k0 of rows of raw_ks k-steps, or null
    const int* rows;                     // row list (the residual is then not written back), or null
};
template <class Tr>
__global__ __launch_bounds__(1024) void k_tlm_resid_norm(TlmResidArgs a) {
    MMI_DYN_SHARED(float, row);          // [ld] the row, then [groups * parts] partial sums, then [groups] 1 / rms
    const int tid = (int)threadIdx.x, lane = tid & 63, wave = tid >> 6, nthr = (int)blockDim.x, nw = nthr >> 6;
    const int r = a.rows ? a.rows[blockIdx.x] : (int)blockIdx.x;
    float* x = a.x + (long)r * a.ld;
    for (int k = 4 * tid; k < a.ld; k += 4 * nthr) {
        f32x4 v = {0.f, 0.f, 0.f, 0.f}, ev = v;
        if (a.emb_mode != TLM_EMB_NONE) {
            const TlmEmbArgs& E = a.emb;
            const uint16_t* e = E.table + (long)E.tok[r] * a.width + k;
            const uint16_t* eb = E.bigram ? E.bigram + (long)E.brow[r] * a.width + k : nullptr;
            const uint16_t* ep = E.pos ? E.pos + (long)E.at[r] * a.width + k : nullptr;
#pragma unroll
            for (int q = 0; q < 4; ++q)
                if (k + q < a.width) {
                    ev[q] = mmi_bf16_to_f32(e[q]) * E.scale;
                    if (eb) ev[q] += mmi_bf16_to_f32(eb[q]);
                    if (ep) ev[q] += mmi_bf16_to_f32(ep[q]);
                }
        }
        if (a.emb_mode == TLM_EMB_SET) {
            v = ev;
            if (a.emb_out) Tr::store4((typename Tr::elem*)a.emb_out + tlm_index<Tr>(blockIdx.x, a.emb_k0 + k, a.raw_ks), ev);
        } else {
            if (!a.replace) v = *reinterpret_cast<const f32x4*>(x + k);
            f32x4 d = {0.f, 0.f, 0.f, 0.f};
            if (a.mix) {
#pragma unroll 8
                for (int p = 0; p < a.mix_p; ++p) d += *reinterpret_cast<const f32x4*>(a.mix + p * a.mix_ps + (long)r * a.ld + k);
                if (a.ls1) d *= *reinterpret_cast<const f32x4*>(a.ls1 + k);
            }
            if (a.dn) {
                f32x4 f = {0.f, 0.f, 0.f, 0.f};
                for (int c = 0; c < a.top; ++c)
#pragma unroll 8
                    for (int p = 0; p < a.dn_p; ++p) f += *reinterpret_cast<const f32x4*>(a.dn + p * a.dn_ps + ((long)r * a.top + c) * a.ld + k);
                f *= 1.0f / (float)a.top;
                d += a.ls2 ? f * *reinterpret_cast<const f32x4*>(a.ls2 + k) : f;
            }
            v += d;
            if (a.tap) *reinterpret_cast<f32x4*>(a.tap + (long)r * a.ld + k) = v;
            if (a.emb_mode == TLM_EMB_ADD) v += ev;
        }
        if (a.vec) v += *reinterpret_cast<const f32x4*>(a.vec + k);
        if (a.raw) Tr::store4((typename Tr::elem*)a.raw + tlm_index<Tr>(blockIdx.x, k, a.raw_ks), v);
        if (!a.rows) *reinterpret_cast<f32x4*>(x + k) = v;
        *reinterpret_cast<f32x4*>(row + k) = v;
    }
    if (!a.out) return;                                       // uniform over the grid
    const int gs = a.width / a.groups;
    const int parts = a.groups < nw ? nw / a.groups : 1;        // waves per group
    float* part = row + a.ld;
    float* inv = part + a.groups * parts;
    __syncthreads();
    const int per = (gs + parts - 1) / parts;
    for (int t = wave; t < a.groups * parts; t += nw) {
        const int g = t / parts, p = t - g * parts;
        const int lo = p * per, hi = lo + per < gs ? lo + per : gs;
        float s = 0.f;
        for (int k = lo + lane; k < hi; k += 64) s = mmi_fma(row[g * gs + k], row[g * gs + k], s);
        s = tlm_wave_sum(s);
        if (lane == 0) part[t] = s;
    }
    __syncthreads();
    for (int g = tid; g < a.groups; g += nthr) {
        float s = 0.f;
        for (int p = 0; p < parts; ++p) s += part[g * parts + p];
        inv[g] = 1.0f / sqrtf(s / (float)gs + a.eps);
    }
    __syncthreads();
    typename Tr::elem* out = (typename Tr::elem*)a.out;
    for (int k = 4 * tid; k < a.ld; k += 4 * nthr) {
        f32x4 v = *reinterpret_cast<const f32x4*>(row + k);
        const f32x4 w = *reinterpret_cast<const f32x4*>(a.w + k);
#pragma unroll
        for (int q = 0; q < 4; ++q) v[q] = k + q < a.width ? v[q] * inv[(k + q) / gs] : 0.f;
        Tr::store4(out + tlm_index<Tr>(blockIdx.x, k, a.KS), v * w);
        if (a.out2) Tr::store4((typename Tr::elem*)a.out2 + tlm_index<Tr>(blockIdx.x, k, a.KS), v * *reinterpret_cast<const f32x4*>(a.w2 + k));
    }
}

// ------------------------------------------------------------------------------------------------
// matrix products: up to three of them per launch, each dense, grouped (per head) or routed (per expert)
// ------------------------------------------------------------------------------------------------
enum { TLM_EPI_F32 = 0, TLM_EPI_PACK = 1, TLM_EPI_ROPE = 2, TLM_EPI_GRU = 3, TLM_EPI_LOGITS = 4, TLM_EPI_SILU = 5, TLM_EPI_GLU = 6, TLM_EPI_QKV = 7 };
enum { TLM_ACT_NONE = 0, TLM_ACT_RELU2 = 1 };
// queries, keys and values of grouped attention: head by head, every head padded to whole tiles; keys and values go to the cache
struct TlmQkv {
    void *kc, *vc;
    const int* crow;                     // cache row of the token: 64 page + offset
    int q_nt, k_nt, h_nt, v_nt;          // tiles of all query heads, of all key heads, per query / key head, per value head
    int heads, kv_heads;
};
struct TlmJob {
    const u32x4* wp; long wgs;           // packed weights; fragments x 64 per group
    const u32x4* xp; int xks, xkg;       // packed activations, their k-steps per row tile; k-step offset per group
    int KS, NT, groups, ksplit;
    int rows, rblocks;                   // dense rows; row blocks (routed: the bound on the number of tiles)
    int in_mul, in_gadd;                 // activation row of row r in group g: r * in_mul + g * in_gadd
    const int* list;                     // routed: pair list, tiles (expert, first, pairs), their number; activation row = pair / in_div
    const int* tiles;
    const int* n_tiles;
    int in_div;
    int epi, act, act_nt;                // SILU: the first act_nt tiles
    void* out; int out_ld; long out_ps;  // fp32: row stride, stride per K split; packed: k-steps per row tile
    int out_mul, out_gadd, out_k0, out_kg;
    const float* bias;                   // GRU: [2][width]
    TlmQkv qkv;
    const float* gate; int gate_ld;      // PACK: factor per (row, group), or null
    const float* rope; int rope_ld;      // ROPE: (cos, sin) per row
    int n_valid;                         // LOGITS: columns
    float scale;                         // LOGITS: factor; GLU: limit
    int blocks;
};
struct TlmJobs {
    TlmJob j[3];
    int n;
};

// cached values of grouped attention: the transposed operand of the value product, [page][kv head][keys / KSTEP][16-wide value blocks]
// fragments whose reduction order is the one the softmax weights have in the registers after S = K Q^T (bf16: keys 4 kq .. 4 kq + 3 of
// both 16-key halves)
template <class Tr>
MMI_HD long tlm_value_index(int crow, int g, int kv_heads, int d, int nd) {
    const int o = crow & (TLM_PAGE - 1), ko = o % Tr::KSTEP, half = ko >> 4;
    const long blk = ((long)(crow / TLM_PAGE) * kv_heads + g) * (TLM_PAGE / Tr::KSTEP) + o / Tr::KSTEP;
    return ((blk * nd + (d >> 4)) * 64 + ((ko & 15) >> 2) * 16 + (d & 15)) * Tr::V + 4 * half + (ko & 3);
}

template <class Tr, int EPI>
__device__ __forceinline__ void tlm_epilogue(const TlmJob& j, int g, int split, int id, int nt, int quad, f32x4 v) {
    const int n0 = nt * 16 + 4 * quad;
    const long orow = (long)id * j.out_mul + (long)g * j.out_gadd;
    if constexpr (EPI == TLM_EPI_F32) {
        *reinterpret_cast<f32x4*>((float*)j.out + split * j.out_ps + orow * j.out_ld + n0) = v;
    } else if constexpr (EPI == TLM_EPI_PACK) {
        if (j.act == TLM_ACT_RELU2) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float r = v[e] > 0.f ? v[e] : 0.f;
                v[e] = r * r;
            }
        }
        if (j.gate) v *= j.gate[(long)id * j.gate_ld + g];
        Tr::store4((typename Tr::elem*)j.out + tlm_index<Tr>(orow, j.out_k0 + g * j.out_kg + n0, j.out_ld), v);
    } else if constexpr (EPI == TLM_EPI_ROPE) {
        // rotation pairs are adjacent (the weight rows are interleaved at load)
        const f32x4 cs = *reinterpret_cast<const f32x4*>(j.rope + ((long)id * j.rope_ld + n0 / 2) * 2);
        const f32x4 o = {v[0] * cs[0] - v[1] * cs[1], v[1] * cs[0] + v[0] * cs[1], v[2] * cs[2] - v[3] * cs[3], v[3] * cs[2] + v[2] * cs[3]};
        Tr::store4((typename Tr::elem*)j.out + tlm_index<Tr>(orow, j.out_k0 + g * j.out_kg + n0, j.out_ld), o);
    } else if constexpr (EPI == TLM_EPI_GRU) {
        // n-tiles alternate gate, candidate, output gate of the same 16 channels
        const int kind = nt % 3, c = (nt / 3) * 16 + 4 * quad;
        const int w = j.out_ld;
        f32x4 o;
        if (kind == 2) {
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] = v[e] * tlm_sigmoid(v[e]);
        } else {
            v += *reinterpret_cast<const f32x4*>(j.bias + kind * w + c);
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] = (kind == 1 && v[e] >= 0.f) ? v[e] + 0.5f : tlm_sigmoid(v[e]);
        }
        *reinterpret_cast<f32x4*>((float*)j.out + (orow * 3 + kind) * w + c) = o;
    } else if constexpr (EPI == TLM_EPI_SILU) {
        if (nt < j.act_nt) {
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] *= tlm_sigmoid(v[e]);
        }
        *reinterpret_cast<f32x4*>((float*)j.out + orow * j.out_ld + n0) = v;
    } else if constexpr (EPI == TLM_EPI_GLU) {
        // gate and up rows alternate (the weight rows are interleaved at load)
        float y[2];
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            const float g = fminf(v[2 * e], j.scale), u = fminf(fmaxf(v[2 * e + 1], -j.scale), j.scale);
            y[e] = g * tlm_sigmoid(1.702f * g) * (u + 1.0f);
        }
        Tr::store2((typename Tr::elem*)j.out + tlm_index<Tr>(orow, n0 / 2, j.out_ld), y[0], y[1]);
    } else if constexpr (EPI == TLM_EPI_QKV) {
        const TlmQkv& z = j.qkv;
        if (nt < z.q_nt) {
            const int h = nt / z.h_nt;
            Tr::store4((typename Tr::elem*)j.out + tlm_index<Tr>((long)id * z.heads + h, n0 - h * z.h_nt * 16, j.out_ld), v);
        } else if (nt < z.q_nt + z.k_nt) {
            const int g = (nt - z.q_nt) / z.h_nt, cr = z.crow[id];
            const long row = ((long)(cr / TLM_PAGE) * z.kv_heads + g) * TLM_PAGE + (cr & (TLM_PAGE - 1));
            Tr::store4((typename Tr::elem*)z.kc + tlm_index<Tr>(row, n0 - (z.q_nt + g * z.h_nt) * 16, j.out_ld), v);
        } else {
            const int t = nt - z.q_nt - z.k_nt, g = t / z.v_nt, cr = z.crow[id], d = n0 - (z.q_nt + z.k_nt + g * z.v_nt) * 16;
            typename Tr::elem* o = (typename Tr::elem*)z.vc + tlm_value_index<Tr>(cr, g, z.kv_heads, d, z.v_nt);
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e * Tr::V] = Tr::cvt(v[e]);
        }
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (n0 + e < j.n_valid) ((float*)j.out)[orow * j.out_ld + n0 + e] = v[e] * j.scale;
    }
}

template <int E>
struct TlmEpi { static constexpr int value = E; };
// f(TlmEpi<kind>()) once per workgroup: the kinds' code is laid out one after the other, not interleaved per tile
template <class F>
__device__ __forceinline__ void tlm_with_epilogue(int epi, F f) {
    if (epi == TLM_EPI_F32) f(TlmEpi<TLM_EPI_F32>());
    else if (epi == TLM_EPI_PACK) f(TlmEpi<TLM_EPI_PACK>());
    else if (epi == TLM_EPI_ROPE) f(TlmEpi<TLM_EPI_ROPE>());
    else if (epi == TLM_EPI_GRU) f(TlmEpi<TLM_EPI_GRU>());
    else if (epi == TLM_EPI_SILU) f(TlmEpi<TLM_EPI_SILU>());
    else if (epi == TLM_EPI_GLU) f(TlmEpi<TLM_EPI_GLU>());
    else if (epi == TLM_EPI_QKV) f(TlmEpi<TLM_EPI_QKV>());
    else f(TlmEpi<TLM_EPI_LOGITS>());
}

// Few rows (<= 16 MT per block): the weights are an HBM stream.  A workgroup owns NTW n-tiles; its waves split K, each with U k-steps
// of weight fragments in flight per register buffer; partial tiles are summed through LDS in a fixed order.  Every activation fragment
// (an L2 read) meets NTW weight fragments, so that with many rows the activations do not cost more than the weights.
template <class Tr, int MT, int NTW, int WAVES, int U>
__global__ __launch_bounds__(WAVES * 64, WAVES == 4 ? 2 : 1) void k_tlm_gemm_rows(TlmJobs jobs) {
    int b = (int)blockIdx.x, ji = 0;
    while (ji + 1 < jobs.n && b >= jobs.j[ji].blocks) b -= jobs.j[ji++].blocks;
    const TlmJob j = jobs.j[ji];             // (a copy: its fields live in scalar registers)
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15;
    const int ntb = (j.NT + NTW - 1) / NTW, nt0 = (b % ntb) * NTW;
    b /= ntb;
    const int split = b % j.ksplit;
    b /= j.ksplit;
    int g = b % j.groups, rb = b / j.groups, r0 = rb * 16 * MT, n;
    if (j.list) {
        if (rb >= *j.n_tiles) return;
        g = j.tiles[3 * rb];
        r0 = j.tiles[3 * rb + 1];
        n = j.tiles[3 * rb + 2];
    } else {
        n = j.rows - r0 < 16 * MT ? j.rows - r0 : 16 * MT;
    }
    const u32x4* xq[MT];                                      // rows past n repeat the last one, and are dropped at the end
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int i = m * 16 + bl < n ? m * 16 + bl : n - 1;
        const int id = j.list ? j.list[r0 + i] : r0 + i;
        const long in = j.list ? id / j.in_div : (long)id * j.in_mul + (long)g * j.in_gadd;
        xq[m] = j.xp + ((in >> 4) * j.xks + (long)g * j.xkg) * 64 + (in & 15) + (lane >> 4) * 16;
    }
    // K range of this split, then of this wave
    const int sper = (j.KS + j.ksplit - 1) / j.ksplit;
    const int s0 = min(j.KS, split * sper), s1 = min(j.KS, s0 + sper);
    const int wper = (s1 - s0 + WAVES - 1) / WAVES;
    const int k0 = min(s1, s0 + wave * wper), nk = min(s1, k0 + wper) - k0;
    const u32x4* wq[NTW];
#pragma unroll
    for (int t = 0; t < NTW; ++t) wq[t] = j.wp + (long)g * j.wgs + ((long)min(nt0 + t, j.NT - 1) * j.KS + k0) * 64 + lane;
    f32x4 acc[NTW][MT];
#pragma unroll
    for (int t = 0; t < NTW; ++t)
#pragma unroll
        for (int m = 0; m < MT; ++m) acc[t][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    u32x4 wA[U][NTW], wB[U][NTW], xA[U][MT], xB[U][MT];
#define TLM_LOAD(W_, X_, base)                                                                              \
    _Pragma("unroll") for (int u = 0; u < U; ++u) {                                                         \
        _Pragma("unroll") for (int t = 0; t < NTW; ++t) W_[u][t] = mmi_load_nt(wq[t] + (long)((base) + u) * 64); \
        _Pragma("unroll") for (int m = 0; m < MT; ++m) X_[u][m] = xq[m][(long)(k0 + (base) + u) * 64];      \
    }
#define TLM_MMA1(W_, X_, u)                                                                                 \
        _Pragma("unroll") for (int m = 0; m < MT; ++m)                                                      \
            _Pragma("unroll") for (int t = 0; t < NTW; ++t) acc[t][m] = Tr::mfma(W_[u][t], X_[u][m], acc[t][m]);
#define TLM_MMA(W_, X_)                                                                                     \
    _Pragma("unroll") for (int u = 0; u < U; ++u) { TLM_MMA1(W_, X_, u) }
    // no load of the steady state is conditional, so that the wait before a product only covers the older buffer
    const int nfull = nk / U, rem = nk - nfull * U;
    if (nfull > 0) {
        TLM_LOAD(wA, xA, 0);
        int i = 0;
        for (; i + 2 < nfull; i += 2) {
            TLM_LOAD(wB, xB, (i + 1) * U);
            mmi_sched_barrier();
            TLM_MMA(wA, xA);
            TLM_LOAD(wA, xA, (i + 2) * U);
            mmi_sched_barrier();
            TLM_MMA(wB, xB);
        }
        if (nfull - i == 2) {
            TLM_LOAD(wB, xB, (i + 1) * U);
            mmi_sched_barrier();
            TLM_MMA(wA, xA);
            TLM_MMA(wB, xB);
        } else {
            TLM_MMA(wA, xA);
        }
    }
    if (rem > 0) {                                            // fewer than U k-steps: requested together, from valid addresses
#pragma unroll
        for (int u = 0; u < U - 1; ++u) {
            const int k = nfull * U + min(u, rem - 1);
#pragma unroll
            for (int t = 0; t < NTW; ++t) wA[u][t] = mmi_load_nt(wq[t] + (long)k * 64);
#pragma unroll
            for (int m = 0; m < MT; ++m) xA[u][m] = xq[m][(long)(k0 + k) * 64];
        }
#pragma unroll
        for (int u = 0; u < U - 1; ++u)
            if (u < rem) { TLM_MMA1(wA, xA, u) }
    }
#undef TLM_MMA1
#undef TLM_LOAD
#undef TLM_MMA
    MMI_SHARED __attribute__((aligned(16))) f32x4 red[WAVES * NTW * MT * 64];
#pragma unroll
    for (int t = 0; t < NTW; ++t)
#pragma unroll
        for (int m = 0; m < MT; ++m) red[((wave * NTW + t) * MT + m) * 64 + lane] = acc[t][m];
    __syncthreads();
    tlm_with_epilogue(j.epi, [&](auto epi) __attribute__((always_inline)) {
#pragma unroll 1
        for (int q = wave; q < NTW * MT; q += WAVES) {
            const int t = q / MT, i = (q - t * MT) * 16 + bl;
            if (i >= n || nt0 + t >= j.NT) continue;
            f32x4 v = red[q * 64 + lane];
#pragma unroll
            for (int w = 1; w < WAVES; ++w) v += red[(w * NTW * MT + q) * 64 + lane];
            tlm_epilogue<Tr, decltype(epi)::value>(j, g, split, j.list ? j.list[r0 + i] : r0 + i, nt0 + t, lane >> 4, v);
        }
    });
}

// Many rows: 2 x 2 waves over a tile of 32 FN features x 32 FM rows, SK k-steps per stage, double-buffered in LDS, with the loads of the
// two stages after the current one in flight in registers.  Operands arrive as whole fragments (one 16-byte vector per lane), so
// staging and operand reads are conflict-free without a swizzle.
template <class Tr, int FN, int FM, int SK>
__global__ __launch_bounds__(256, 2) void k_tlm_gemm_tile(TlmJobs jobs) {
    constexpr int NF = 2 * FN + 2 * FM, NI = NF / 4;          // fragments per k-step; per wave
    MMI_SHARED __attribute__((aligned(16))) u32x4 lds[2 * SK * NF * 64];
    // consecutive workgroups go round the 8 XCDs: give each XCD a contiguous run of tiles so that its L2 sees the shared operand
    const int nb = (int)gridDim.x, xper = nb >> 3, xrem = nb & 7, xcd = (int)blockIdx.x & 7;
    int b = xcd * xper + (xcd < xrem ? xcd : xrem) + ((int)blockIdx.x >> 3), ji = 0;
    while (ji + 1 < jobs.n && b >= jobs.j[ji].blocks) b -= jobs.j[ji++].blocks;
    const TlmJob j = jobs.j[ji];             // (a copy: its fields live in scalar registers)
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15;
    const int ntb = (j.NT + 2 * FN - 1) / (2 * FN);
    int g, rb, nb0, n, r0;
    if (j.list) {
        nb0 = b % ntb;
        rb = b / ntb;
        if (rb >= *j.n_tiles) return;
        g = j.tiles[3 * rb];
        r0 = j.tiles[3 * rb + 1];
        n = j.tiles[3 * rb + 2];
    } else {
        rb = b % j.rblocks;
        b /= j.rblocks;
        nb0 = b % ntb;
        g = b / ntb;
        r0 = rb * 32 * FM;
        n = j.rows - r0 < 32 * FM ? j.rows - r0 : 32 * FM;
    }
    const int nt0 = nb0 * 2 * FN;
    const u32x4* wbase = j.wp + (long)g * j.wgs;
    int off[NI];                                              // fragment i of this wave, lane: 16-byte vectors from its operand's base
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int f = wave + 4 * i;
        if (4 * i < 2 * FN) {
            const int nt = nt0 + f < j.NT ? nt0 + f : j.NT - 1;
            off[i] = nt * j.KS * 64 + lane;
        } else {
            const int m = (f - 2 * FN) * 16 + bl, ii = m < n ? m : n - 1;
            const int id = j.list ? j.list[r0 + ii] : r0 + ii;
            const long in = j.list ? id / j.in_div : (long)id * j.in_mul + (long)g * j.in_gadd;
            off[i] = (int)((in >> 4) * j.xks + (long)g * j.xkg) * 64 + (int)(in & 15) + (lane >> 4) * 16;
        }
    }
    const int wn = wave & 1, wm = wave >> 1;
    f32x4 acc[FN][FM];
#pragma unroll
    for (int x = 0; x < FN; ++x)
#pragma unroll
        for (int y = 0; y < FM; ++y) acc[x][y] = f32x4{0.f, 0.f, 0.f, 0.f};
    u32x4 st[2][SK][NI];
#define TLM_FETCH(set, stage)                                                                   \
    _Pragma("unroll") for (int kk = 0; kk < SK; ++kk) {                                         \
        const int k_ = (stage) * SK + kk < j.KS ? (stage) * SK + kk : j.KS - 1;                 \
        _Pragma("unroll") for (int i = 0; i < NI; ++i) st[set][kk][i] = (4 * i < 2 * FN ? wbase : j.xp)[(unsigned)(off[i] + k_ * 64)];  \
    }
#define TLM_STAGE(set, buf)                                                                     \
    _Pragma("unroll") for (int kk = 0; kk < SK; ++kk)                                           \
        _Pragma("unroll") for (int i = 0; i < NI; ++i) lds[(((buf) * SK + kk) * NF + wave + 4 * i) * 64 + lane] = st[set][kk][i];
#define TLM_COMPUTE(buf, stage)                                                                 \
    _Pragma("unroll") for (int kk = 0; kk < SK; ++kk)                                           \
        if ((stage) * SK + kk < j.KS) {                                                         \
            const u32x4* base = lds + (((buf) * SK + kk) * NF) * 64 + lane;                     \
            u32x4 bv[FM];                                                                       \
            _Pragma("unroll") for (int y = 0; y < FM; ++y) bv[y] = base[(2 * FN + wm * FM + y) * 64]; \
            _Pragma("unroll") for (int x = 0; x < FN; ++x) {                                    \
                const u32x4 av = base[(wn * FN + x) * 64];                                      \
                _Pragma("unroll") for (int y = 0; y < FM; ++y) acc[x][y] = Tr::mfma(av, bv[y], acc[x][y]); \
            }                                                                                   \
        }
    // (fetches past the end repeat the last k-step: an unconditional load keeps the wait in front of a stage to the older set)
    const int ns = (j.KS + SK - 1) / SK;
    TLM_FETCH(0, 0);
    TLM_FETCH(1, 1);
    TLM_STAGE(0, 0);
    __syncthreads();
    for (int s = 0; s < ns; s += 2) {                         // stage s in buffer 0 and register set 0, stage s + 1 in 1 and 1
        TLM_FETCH(0, s + 2);
        mmi_sched_barrier();
        TLM_COMPUTE(0, s);
        TLM_STAGE(1, 1);
        __syncthreads();
        TLM_FETCH(1, s + 3);
        mmi_sched_barrier();
        TLM_COMPUTE(1, s + 1);
        TLM_STAGE(0, 0);
        __syncthreads();
    }
#undef TLM_COMPUTE
#undef TLM_FETCH
#undef TLM_STAGE
    tlm_with_epilogue(j.epi, [&](auto epi) __attribute__((always_inline)) {
#pragma unroll
        for (int y = 0; y < FM; ++y) {
            const int m = (wm * FM + y) * 16 + bl;
            if (m >= n) continue;
            const int id = j.list ? j.list[r0 + m] : r0 + m;
            // through LDS (a lane reads what it wrote), so that the epilogue's code is there once per y and not once per tile
            f32x4* buf = reinterpret_cast<f32x4*>(lds) + wave * FN * 64 + lane;
#pragma unroll
            for (int x = 0; x < FN; ++x) buf[x * 64] = acc[x][y];
            const int nx = min(FN, j.NT - nt0 - wn * FN);
#pragma unroll 1
            for (int x = 0; x < nx; ++x) tlm_epilogue<Tr, decltype(epi)::value>(j, g, 0, id, nt0 + wn * FN + x, lane >> 4, buf[x * 64]);
        }
    });
}

// ------------------------------------------------------------------------------------------------
// latent attention
// ------------------------------------------------------------------------------------------------
// One workgroup per token, on the columns [query latent | latent | rotated key part | head gates] of the input projection (fp32
// split-K partials): the two RMS norms, the rotation of the key part, the cache write and the sigmoid of the gates.
struct TlmLatentArgs {
    const float* in; int in_p; long in_ps; int ld;       // ld: columns per row (every section rounded up to 16)
    int q_rank, kv_rank, rot, heads;
    int qp, kvp, rp;                                     // section widths
    const float* qw; const float* cw; float eps;
    const float* rope; int rope_ld;
    const int* crow;                                     // cache row of the token: 64 page + offset
    void* q; int q_ks;
    void* kc; int k_ks, rot_k0;
    float* gate; int gate_ld;
};
template <class Tr>
__global__ __launch_bounds__(256) void k_tlm_latent(TlmLatentArgs a) {
    typedef typename Tr::elem elem;
    MMI_DYN_SHARED(float, row);                          // [ld]
    MMI_SHARED float part[2][4];
    const int t = (int)blockIdx.x, tid = (int)threadIdx.x, lane = tid & 63, wave = tid >> 6;
    float sq = 0.f, sc = 0.f;
    for (int k = 4 * tid; k < a.ld; k += 1024) {
        f32x4 v = *reinterpret_cast<const f32x4*>(a.in + (long)t * a.ld + k);
#pragma unroll 4
        for (int p = 1; p < a.in_p; ++p) v += *reinterpret_cast<const f32x4*>(a.in + p * a.in_ps + (long)t * a.ld + k);
        *reinterpret_cast<f32x4*>(row + k) = v;
        const float s = v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];     // the padding columns are zero
        if (k < a.qp) sq += s;
        else if (k < a.qp + a.kvp) sc += s;
    }
    sq = tlm_wave_sum(sq);
    sc = tlm_wave_sum(sc);
    if (lane == 0) {
        part[0][wave] = sq;
        part[1][wave] = sc;
    }
    __syncthreads();
    const float iq = 1.0f / sqrtf((part[0][0] + part[0][1] + part[0][2] + part[0][3]) / (float)a.q_rank + a.eps);
    const float ic = 1.0f / sqrtf((part[1][0] + part[1][1] + part[1][2] + part[1][3]) / (float)a.kv_rank + a.eps);
    const long cr = a.crow[t];
    for (int k = 4 * tid; k < a.ld; k += 1024) {
        f32x4 v = *reinterpret_cast<const f32x4*>(row + k);
        if (k < a.qp) {
            v *= iq * *reinterpret_cast<const f32x4*>(a.qw + k);
            Tr::store4((elem*)a.q + tlm_index<Tr>(t, k, a.q_ks), v);
        } else if (k < a.qp + a.kvp) {
            const int d = k - a.qp;
            v *= ic * *reinterpret_cast<const f32x4*>(a.cw + d);
            Tr::store4((elem*)a.kc + tlm_index<Tr>(cr, d, a.k_ks), v);
        } else if (k < a.qp + a.kvp + a.rp) {
            const int d = k - a.qp - a.kvp;
            const f32x4 cs = *reinterpret_cast<const f32x4*>(a.rope + ((long)t * a.rope_ld + d / 2) * 2);
            const f32x4 o = {v[0] * cs[0] - v[1] * cs[1], v[1] * cs[0] + v[0] * cs[1], v[2] * cs[2] - v[3] * cs[3], v[3] * cs[2] + v[2] * cs[3]};
            Tr::store4((elem*)a.kc + tlm_index<Tr>(cr, a.rot_k0 + d, a.k_ks), o);
        } else {
            const int h = k - a.qp - a.kvp - a.rp;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (h + e < a.heads) a.gate[(long)t * a.gate_ld + h + e] = tlm_sigmoid(v[e]);
        }
    }
}

// Attention over the latent cache.  All heads share one key per position - (latent, rotated part) against the queries absorbed
// through the key projection - and the value is the latent itself, so (token, head) pairs are the columns of one product and a key
// fragment serves 16 of them.  A column tile never mixes sequences.  Keys are walked in blocks of 32; a column sees key j of its
// token at position i when 0 <= i - j < window.
// which keys a position sees, and the factor of the scores (times log2(e)): the last `window` ones (0: all), and the first `keep`
struct TlmMask { int window, keep; float scale; };
// pages of a sequence: the block table's first `keep` entries are for the pages that no window releases, the others are a ring
struct TlmPages { const int* table; int ld, keep; };
__device__ __forceinline__ int tlm_page(const TlmPages& p, const int* row, int i) { return row[i < p.keep ? i : p.keep + (i - p.keep) % (p.ld - p.keep)]; }

struct TlmAttnArgs {
    const void* q;                       // packed rows token * heads + head
    const void* kc;
    void* out; int out_rows;             // packed rows head * out_rows + token, latent columns (the value projection reads head by head)
    int heads, q_ks, nd, out_ks;
    TlmMask mask;
    int n_entries, n_tiles, nsplit;
    const int* tile0;                    // [entries + 1] first column tile (k_tlm_attn_tile: column group) of each entry
    const int* erow0; const int* elen; const int* epos0; const int* eslot;
    TlmPages pages;                      // table [slot][ld]
    float* po;                           // nsplit > 1: [tile][split][nd][64] f32x4 un-normalised sums
    float* pml;                          // [tile][split][2][16]: running maximum, sum of weights
};
struct TlmCols { int entry, c0, ncol; };
template <class Args>
__device__ __forceinline__ TlmCols tlm_find_tile(const Args& a, int tile) {
    // the last entry whose first tile is <= tile: all prefixes compared at once (a binary search would be a chain of dependent loads)
    unsigned below = 0;
    for (int e = mmi_lane(); e < a.n_entries; e += 64) below += a.tile0[e] <= tile ? 1u : 0u;
    const int lo = mmi_uniform((int)mmi_wave_sum_u32(below) - 1);
    TlmCols c;
    c.entry = lo;
    c.c0 = (tile - a.tile0[lo]) * 16;
    c.ncol = a.elen[lo] * a.heads;
    return c;
}

template <class Tr>
__device__ __forceinline__ void tlm_attn_store(const TlmAttnArgs& a, const TlmCols& c, int bl, int kq, int db, f32x4 v) {
    const int col = c.c0 + bl;
    if (col >= c.ncol) return;
    const int t = col / a.heads;
    const long orow = (long)(col - t * a.heads) * a.out_rows + a.erow0[c.entry] + t;
    Tr::store4((typename Tr::elem*)a.out + tlm_index<Tr>(orow, db * 16 + 4 * kq, a.out_ks), v);
}

// Shapes are template bounds - ND 16-wide latent blocks, RK k-steps of the rotated part - and the loops run over the bounds without a
// branch, so that a block's loads are all in flight together: fragments past the model's own sizes repeat a valid address against zero
// query fragments, value blocks past them are dropped at the end.
template <class Tr, int ND, int RK>
struct TlmQuery {
    static constexpr int LK = ND * 16 / Tr::KSTEP, NK = LK + RK;
    static constexpr int NB = 32 / (4 * Tr::V);                    // value fragments per 32 keys and latent block
    u32x4 f[NK];
    static __device__ __forceinline__ u32x4 fragment(const TlmAttnArgs& a, const u32x4* qp, int s) {
        const int o = s < LK ? s : a.out_ks + s - LK;
        const u32x4 zero = {0u, 0u, 0u, 0u};
        return (s < LK ? s < a.out_ks : o < a.q_ks) ? qp[o * 64] : zero;
    }
    __device__ __forceinline__ void load(const TlmAttnArgs& a, long qrow, int kq) {
        const u32x4* qp = (const u32x4*)a.q + (qrow >> 4) * a.q_ks * 64 + kq * 16 + (qrow & 15);
#pragma unroll
        for (int s = 0; s < NK; ++s) f[s] = fragment(a, qp, s);
    }
};
// 32 (16 at fp32) keys x KSTEP latent dimensions -> the transposed operand, through the matrix core: K x identity is exact
template <class Tr>
struct TlmFlip {
    static constexpr int H = Tr::KSTEP / 16;                       // 16-wide latent blocks per k-step
    u32x4 id[H];
    __device__ __forceinline__ void init(int bl, int kq) {
#pragma unroll
        for (int h = 0; h < H; ++h) {
            if constexpr (Tr::V == 8) {
                const int e = 16 * h + bl - 8 * kq;                // k = 8 kq + e meets column bl where k = 16 h + bl
#pragma unroll
                for (int i = 0; i < 4; ++i) id[h][i] = e == 2 * i ? 0x00003f80u : (e == 2 * i + 1 ? 0x3f800000u : 0u);
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i) id[h][i] = 4 * kq + i == bl ? 0x3f800000u : 0u;
            }
        }
    }
    // bf16: latent block h of the two 16-key fragments of a k-step; fp32: of one
    __device__ __forceinline__ u32x4 turn(u32x4 k0, u32x4 k1, int h) const {
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        const f32x4 a = Tr::mfma(k0, id[h], zero);
        if constexpr (Tr::V == 8) {
            const f32x4 b = Tr::mfma(k1, id[h], zero);
            return u32x4{mmi_pack_bf16x2(a[0], a[1]), mmi_pack_bf16x2(a[2], a[3]), mmi_pack_bf16x2(b[0], b[1]), mmi_pack_bf16x2(b[2], b[3])};
        } else {
            return __builtin_bit_cast(u32x4, a);
        }
    }
};
// k-step of the cache that fragment s of the bound stands for
template <int LK>
__device__ __forceinline__ int tlm_kstep_of(const TlmAttnArgs& a, int s) {
    return s < LK ? min(s, a.out_ks - 1) : min(a.out_ks + s - LK, a.q_ks - 1);
}
// scores of 32 keys -> softmax weights as operand fragments, the running maximum and sum moved on; returns the factor of older sums
// (the lane's keys are k0 .. k0 + 3 and k0 + 16 .. k0 + 19, its column's position is k0 + d0)
template <class Tr>
__device__ __forceinline__ float tlm_softmax_block(const TlmMask& a, f32x4 s0, f32x4 s1, int k0, int d0, float& m, float& l, u32x4 (&pf)[32 / (4 * Tr::V)]) {
    constexpr int NB = 32 / (4 * Tr::V);
    float mx = m;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int e0 = d0 - r, e1 = d0 - r - 16;
        s0[r] = e0 >= 0 && (a.window <= 0 || e0 < a.window || k0 + r < a.keep) ? s0[r] * a.scale : -INFINITY;
        s1[r] = e1 >= 0 && (a.window <= 0 || e1 < a.window || k0 + r + 16 < a.keep) ? s1[r] * a.scale : -INFINITY;
        mx = fmaxf(mx, fmaxf(s0[r], s1[r]));
    }
    mx = fmaxf(mx, mmi_shfl_xor(mx, 16));
    mx = fmaxf(mx, mmi_shfl_xor(mx, 32));
    const float al = exp2f(m - mx);
    m = mx;
    l *= al;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        s0[r] = exp2f(s0[r] - mx);
        s1[r] = exp2f(s1[r] - mx);
        l += s0[r] + s1[r];
    }
    if constexpr (NB == 1) {
        pf[0] = u32x4{mmi_pack_bf16x2(s0[0], s0[1]), mmi_pack_bf16x2(s0[2], s0[3]), mmi_pack_bf16x2(s1[0], s1[1]), mmi_pack_bf16x2(s1[2], s1[3])};
    } else {
        pf[0] = __builtin_bit_cast(u32x4, s0);
        pf[NB - 1] = __builtin_bit_cast(u32x4, s1);
    }
    return al;
}

// One block of 32 keys as a stream of fragments out of LDS - keys 0-15 and 16-31 of every k-step, then the turned values - consumed in
// groups of G, the next group read while one is used.
template <class Tr, int ND, int RK, int QT, int G>
struct TlmAttnStream {
    typedef TlmQuery<Tr, ND, RK> Q;
    static constexpr int NB = Q::NB, NK = Q::NK, F = 2 * NK + ND * NB, NG = ((F + G - 1) / G + 1) / 2 * 2;      // an even number of groups: group g always meets buffer g & 1
    u32x4 fr[2][G];
    f32x4 s[QT][2];
    u32x4 pf[QT][NB];
    float m[QT], l[QT];
    f32x4 acc[QT][ND];
    __device__ __forceinline__ void clear(float m0 = -1e30f) {
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            m[t] = m0;
            l[t] = 0.f;
#pragma unroll
            for (int d = 0; d < ND; ++d) acc[t][d] = f32x4{0.f, 0.f, 0.f, 0.f};
        }
    }
    // at(f): address of fragment f for this lane
    template <class At>
    __device__ __forceinline__ void load(int buf, int g, At at) {
#pragma unroll
        for (int i = 0; i < G; ++i)
            if (g * G + i < F) fr[buf][i] = *at(g * G + i);
    }
    // q(t, k): query fragment k of column tile t
    template <class Qf>
    __device__ __forceinline__ void use(const TlmMask& a, Qf q, int buf, int g, int k0, const int (&d0)[QT]) {
#pragma unroll
        for (int i = 0; i < G; ++i) {
            const int f = g * G + i;
            if (f >= F) continue;
            if (f < 2 * NK) {
#pragma unroll
                for (int t = 0; t < QT; ++t) s[t][f & 1] = Tr::mfma(fr[buf][i], q(t, f >> 1), f < 2 ? f32x4{0.f, 0.f, 0.f, 0.f} : s[t][f & 1]);
                if (f == 2 * NK - 1) soften(a, k0, d0);
            } else {
                const int d = (f - 2 * NK) / NB;
#pragma unroll
                for (int t = 0; t < QT; ++t) acc[t][d] = Tr::mfma(fr[buf][i], pf[t][(f - 2 * NK) % NB], acc[t][d]);
            }
        }
    }
    // scores -> softmax weights; the sums so far are rescaled when some column's maximum has moved
    __device__ __forceinline__ void soften(const TlmMask& a, int k0, const int (&d0)[QT]) {
        float al[QT];
        bool moved = false;
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            al[t] = tlm_softmax_block<Tr>(a, s[t][0], s[t][1], k0, d0[t], m[t], l[t], pf[t]);
            moved = moved || al[t] != 1.f;
        }
        if (mmi_any(moved)) {
#pragma unroll
            for (int t = 0; t < QT; ++t)
#pragma unroll
                for (int d = 0; d < ND; ++d) acc[t][d] *= al[t];
        }
    }
};

// Few column tiles (decoding): the four waves of a workgroup share one column tile, each takes every 4th key block straight from the
// cache, and their sums meet in LDS.  gridDim.y > 1: the keys are also split over workgroups (k_tlm_attn_combine).
template <class Tr, int ND, int RK>
__global__ __launch_bounds__(256, Tr::V == 8 && ND <= 16 ? 2 : 1) void k_tlm_attn(TlmAttnArgs a) {      // two workgroups per CU where the registers allow it
    typedef TlmQuery<Tr, ND, RK> Q;
    constexpr int NB = Q::NB, WK = 4;
    MMI_SHARED float ml[2][4][16];
    MMI_SHARED __attribute__((aligned(16))) f32x4 ob[4 * 8 * 64];
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15, kq = lane >> 4, split = (int)blockIdx.y;
    // consecutive workgroups go round the 8 XCDs: neighbouring tiles (heads of one sequence read the same keys) to one XCD's L2
    const int tile = ((int)blockIdx.x & 7) * ((int)gridDim.x >> 3) + ((int)blockIdx.x >> 3);
    if (tile >= a.n_tiles) return;
    const TlmCols c = tlm_find_tile(a, tile);
    const int col = c.c0 + bl < c.ncol ? c.c0 + bl : c.ncol - 1;
    const int pos0 = a.epos0[c.entry];
    const int pc = pos0 + col / a.heads;                           // position of this lane's column
    const int plo = pos0 + c.c0 / a.heads, phi = pos0 + (min(c.c0 + 15, c.ncol - 1)) / a.heads;
    const int klo = a.mask.window > 0 && plo - a.mask.window + 1 > 0 ? plo - a.mask.window + 1 : 0;
    int b0 = klo / 32, b1 = phi / 32 + 1;
    if (a.nsplit > 1) {
        const int per = (b1 - b0 + a.nsplit - 1) / a.nsplit;
        b0 = min(b1, b0 + split * per);
        b1 = min(b1, b0 + per);
    }
    const int* bt = a.pages.table + (long)a.eslot[c.entry] * a.pages.ld;
    f32x4 acc[ND];
#pragma unroll
    for (int d = 0; d < ND; ++d) acc[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -1e30f, l = 0.f;
    TlmFlip<Tr> flip;
    flip.init(bl, kq);
    // the waves share the column tile: its query fragments stay in LDS, the registers are for keys in flight
    MMI_SHARED __attribute__((aligned(16))) u32x4 ql[Q::NK * 64];
    {
        const long qrow = (long)a.erow0[c.entry] * a.heads + col;
        const u32x4* qp = (const u32x4*)a.q + (qrow >> 4) * a.q_ks * 64 + kq * 16 + (qrow & 15);
        for (int s = wave; s < Q::NK; s += WK) ql[s * 64 + lane] = Q::fragment(a, qp, s);
        __syncthreads();
    }
    // A block's key fragments stay in registers from the scores to the values (turned there), and each one's register asks for the next
    // block's fragment as soon as it has been used: a block is read once, and nearly a whole block is always in flight.
    constexpr int NK = Q::NK, LK = Q::LK, FH = TlmFlip<Tr>::H, GK = 4;
    u32x4 fr[NK][2];
    const u32x4* kp = (const u32x4*)a.kc;
    auto block = [&](int kb) __attribute__((always_inline)) {
        const long page = tlm_page(a.pages, bt, min(kb, b1 - 1) >> 1);    // (past the end: the last block again)
        kp = (const u32x4*)a.kc + (page * 4 + (kb & 1) * 2) * a.q_ks * 64 + lane;
    };
    auto load = [&](int k) __attribute__((always_inline)) {
        const int o = tlm_kstep_of<LK>(a, k);
        fr[k][0] = kp[o * 64];
        fr[k][1] = kp[(a.q_ks + o) * 64];
    };
    if (b0 + wave < b1) {
        block(b0 + wave);
#pragma unroll
        for (int k = 0; k < NK; ++k) load(k);
    }
    for (int kb = b0 + wave; kb < b1; kb += WK) {
        block(kb + WK);
        f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
        for (int k = 0; k < NK; ++k) {
            const u32x4 qv = ql[k * 64 + lane];
            s0 = Tr::mfma(fr[k][0], qv, s0);
            s1 = Tr::mfma(fr[k][1], qv, s1);
        }
#pragma unroll
        for (int k = LK; k < NK; ++k) load(k);
        mmi_sched_barrier();
        u32x4 pf[NB];
        const float al = tlm_softmax_block<Tr>(a.mask, s0, s1, kb * 32 + 4 * kq, pc - (kb * 32 + 4 * kq), m, l, pf);
        if (mmi_any(al != 1.f)) {
#pragma unroll
            for (int d = 0; d < ND; ++d) acc[d] *= al;
        }
#pragma unroll
        for (int k0 = 0; k0 < LK; k0 += GK) {
#pragma unroll
            for (int k = k0; k < k0 + GK && k < LK; ++k)
#pragma unroll
                for (int h = 0; h < FH; ++h) {
                    acc[k * FH + h] = Tr::mfma(flip.turn(fr[k][0], fr[k][1], h), pf[0], acc[k * FH + h]);
                    if constexpr (NB == 2) acc[k * FH + h] = Tr::mfma(flip.turn(fr[k][1], fr[k][1], h), pf[NB - 1], acc[k * FH + h]);
                }
#pragma unroll
            for (int k = k0; k < k0 + GK && k < LK; ++k) load(k);
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
    for (int w = 0; w < WK; ++w) M = fmaxf(M, ml[0][w][bl]);
#pragma unroll
    for (int w = 0; w < WK; ++w) L += ml[1][w][bl] * exp2f(ml[0][w][bl] - M);
    const float f = exp2f(m - M);
    const float inv = a.nsplit > 1 ? 1.f : 1.0f / L;
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
            for (int w = 1; w < WK; ++w) v += ob[(w * 8 + d) * 64 + lane];
            if (a.nsplit > 1) *reinterpret_cast<f32x4*>(a.po + ((((long)tile * a.nsplit + split) * a.nd + d0 + d) * 64 + lane) * 4) = v;
            else tlm_attn_store<Tr>(a, c, bl, kq, d0 + d, v * inv);
        }
    }
    if (a.nsplit > 1 && wave == 0 && kq == 0) {
        float* p = a.pml + ((long)tile * a.nsplit + split) * 32;
        p[bl] = M;
        p[16 + bl] = L;
    }
}

// Many columns (prompts): four waves x QT column tiles of one sequence walk the same keys; a block's fragments are staged through LDS
// once for all of them (NBUF buffers, the next block in flight in registers while this one is used).
template <class Tr, int ND, int RK>
struct TlmAttnTile {
    static constexpr int QT = ND <= (Tr::V == 8 ? 16 : 8) ? 2 : 1;
    static constexpr int NF = 2 * TlmQuery<Tr, ND, RK>::NK + ND * TlmQuery<Tr, ND, RK>::NB;      // fragments per 32 keys
    static constexpr int NBUF = 2 * NF <= 152 ? 2 : 1;
    static constexpr size_t smem() { return (size_t)NBUF * NF * 1024; }
};
template <class Tr, int ND, int RK>
__global__ __launch_bounds__(256) void k_tlm_attn_tile(TlmAttnArgs a) {
    typedef TlmQuery<Tr, ND, RK> Q;
    typedef TlmAttnTile<Tr, ND, RK> P;
    constexpr int NB = Q::NB, NK = Q::NK, QT = P::QT, NF = P::NF, NBUF = P::NBUF, NI = (NK + 3) / 4, FH = TlmFlip<Tr>::H;
    MMI_DYN_SHARED(u32x4, lds);
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15, kq = lane >> 4;
    int g = (int)blockIdx.x;
    TlmCols c;                                                     // (tile0 counts groups of 64 QT columns here)
    {
        c = tlm_find_tile(a, g);
        c.c0 *= 4 * QT;
    }
    const int pos0 = a.epos0[c.entry];
    const int plo = pos0 + c.c0 / a.heads, phi = pos0 + min(c.c0 + 64 * QT - 1, c.ncol - 1) / a.heads;
    const int klo = a.mask.window > 0 && plo - a.mask.window + 1 > 0 ? plo - a.mask.window + 1 : 0;
    const int b0 = klo / 32, b1 = phi / 32 + 1;
    const int* bt = a.pages.table + (long)a.eslot[c.entry] * a.pages.ld;
    typedef TlmAttnStream<Tr, ND, RK, QT, (ND >= 16 ? 4 : 8)> S;
    Q q[QT];
    S sm;
    sm.clear();
    TlmFlip<Tr> flip;
    flip.init(bl, kq);
    int pc[QT], c0[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        c0[t] = c.c0 + (wave * QT + t) * 16;
        const int col = c0[t] + bl < c.ncol ? c0[t] + bl : c.ncol - 1;
        pc[t] = pos0 + col / a.heads;
        q[t].load(a, (long)a.erow0[c.entry] * a.heads + col, kq);
    }
    // fragments of a block in LDS: keys 0-15 and 16-31 of each k-step, then the turned values; wave w brings k-steps w, w + 4, ..
    u32x4 st[NI][2];
    auto page_of = [&](int kb) __attribute__((always_inline)) { return tlm_page(a.pages, bt, min(kb, b1 - 1) >> 1); };
    long page = page_of(b0);                                       // of the block fetched next
    auto fetch = [&](int kb) __attribute__((always_inline)) {
        const u32x4* kp = (const u32x4*)a.kc + (page * 4 + (kb & 1) * 2) * a.q_ks * 64 + lane;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int o = tlm_kstep_of<Q::LK>(a, min(wave + 4 * i, NK - 1));
            st[i][0] = kp[o * 64];
            st[i][1] = kp[(a.q_ks + o) * 64];
        }
        page = page_of(kb + 1);
    };
    auto stage = [&](int buf) __attribute__((always_inline)) {
        u32x4* base = lds + buf * NF * 64 + lane;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int k = wave + 4 * i;
            if (4 * i + 3 >= NK && k >= NK) continue;
            base[(2 * k) * 64] = st[i][0];
            base[(2 * k + 1) * 64] = st[i][1];
            if (4 * i + 3 >= Q::LK && k >= Q::LK) continue;          // the rotated part has no value
#pragma unroll
            for (int h = 0; h < FH; ++h) {
                const int d = k * FH + h;
                if constexpr (NB == 1) {
                    base[(2 * NK + d) * 64] = flip.turn(st[i][0], st[i][1], h);
                } else {
                    base[(2 * NK + d * NB) * 64] = flip.turn(st[i][0], st[i][0], h);
                    base[(2 * NK + d * NB + NB - 1) * 64] = flip.turn(st[i][1], st[i][1], h);
                }
            }
        }
    };
    fetch(b0);
    stage(0);
    __syncthreads();
    int cur = 0;
    for (int kb = b0; kb < b1; ++kb) {
        fetch(kb + 1);                                             // (past the end: the last block's page again)
        mmi_sched_barrier();
        const u32x4* base = lds + cur * NF * 64 + lane;
        auto at = [&](int f) __attribute__((always_inline)) -> const u32x4* { return base + f * 64; };
        auto qf = [&](int t, int k) __attribute__((always_inline)) { return q[t].f[k]; };
        int d0[QT];
#pragma unroll
        for (int t = 0; t < QT; ++t) d0[t] = pc[t] - (kb * 32 + 4 * kq);
        sm.load(0, 0, at);
#pragma unroll
        for (int g = 0; g < S::NG; ++g) {
            if (g + 1 < S::NG) sm.load((g + 1) & 1, g + 1, at);
            mmi_sched_barrier();
            sm.use(a.mask, qf, g & 1, g, kb * 32 + 4 * kq, d0);
        }
        if constexpr (NBUF == 1) __syncthreads();
        else cur ^= 1;
        stage(cur);
        __syncthreads();
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        float l = sm.l[t];
        l += mmi_shfl_xor(l, 16);
        l += mmi_shfl_xor(l, 32);
        const float inv = 1.0f / l;
        TlmCols o = c;
        o.c0 = c0[t];
#pragma unroll
        for (int d = 0; d < ND; ++d)
            if (d < a.nd) tlm_attn_store<Tr>(a, o, bl, kq, d, sm.acc[t][d] * inv);
    }
}

// the splits of one column tile -> output; one workgroup per tile, waves over the latent blocks
template <class Tr>
__global__ __launch_bounds__(256) void k_tlm_attn_combine(TlmAttnArgs a) {
    const int lane = (int)threadIdx.x & 63, wave = mmi_uniform((int)threadIdx.x >> 6), bl = lane & 15, kq = lane >> 4, tile = (int)blockIdx.x;
    const TlmCols c = tlm_find_tile(a, tile);
    const float* q = a.pml + (long)tile * a.nsplit * 32;
    float M = -1e30f, L = 0.f;
#pragma unroll 4
    for (int s = 0; s < a.nsplit; ++s) M = fmaxf(M, q[s * 32 + bl]);
#pragma unroll 4
    for (int s = 0; s < a.nsplit; ++s) L += q[s * 32 + 16 + bl] * exp2f(q[s * 32 + bl] - M);
    const float inv = 1.0f / L;
    for (int d = wave + 4 * (int)blockIdx.y; d < a.nd; d += 4 * (int)gridDim.y) {
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int s = 0; s < a.nsplit; ++s)
            v += *reinterpret_cast<const f32x4*>(a.po + ((((long)tile * a.nsplit + s) * a.nd + d) * 64 + lane) * 4) * exp2f(q[s * 32 + bl] - M);
        tlm_attn_store<Tr>(a, c, bl, kq, d, v * inv);
    }
}

// ------------------------------------------------------------------------------------------------
// minimal gated recurrence: S_t = (1 - z_t) S_(t-1) + z_t c_t, output S_t * g_t, from the fp32 gates the projection's epilogue stored.
// A step's sequences are cut into segments of at most TLM_SEG tokens.  The recurrence is linear in S, so a segment is the pair
// (A, B) with S_end = A S_begin + B: the first launch computes the pairs (only when some sequence has more than one segment), the
// second starts every segment from its predecessors' pairs.  State is [slot][2][width]: read one copy, write the other, so that a
// segment's write cannot be seen by another segment of the same sequence.
// ------------------------------------------------------------------------------------------------
constexpr int TLM_SEG = 32;
struct TlmSeg { int row0, n, slot, par, index, last, fresh, pad; };      // index: number of the segment in its sequence; fresh: position 0
struct TlmScanArgs {
    const float* zcg;             // [row][3][width]
    int width;                    // padded to 16
    const TlmSeg* seg;
    float* state;
    float* pair;                  // [segment][2][width]
    void* out; int out_ks;
};
__global__ __launch_bounds__(256) void k_tlm_scan_pairs(TlmScanArgs a) {
    const int c = (int)(blockIdx.x * blockDim.x + threadIdx.x);
    const TlmSeg s = a.seg[blockIdx.y];
    if (c >= a.width || s.last) return;
    const float* p = a.zcg + (long)s.row0 * 3 * a.width + c;
    float A = 1.f, B = 0.f;
    for (int i0 = 0; i0 < s.n; i0 += 8) {
        float z[8], u[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const long o = (long)(i0 + i < s.n ? i0 + i : s.n - 1) * 3 * a.width;
            z[i] = p[o];
            u[i] = p[o + a.width];
        }
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i0 + i < s.n) {
                A *= 1.0f - z[i];
                B = mmi_fma(1.0f - z[i], B, z[i] * u[i]);
            }
    }
    a.pair[(long)blockIdx.y * 2 * a.width + c] = A;
    a.pair[((long)blockIdx.y * 2 + 1) * a.width + c] = B;
}
template <class Tr>
__global__ __launch_bounds__(256) void k_tlm_scan(TlmScanArgs a) {
    const int c = (int)(blockIdx.x * blockDim.x + threadIdx.x);
    const TlmSeg s = a.seg[blockIdx.y];
    if (c >= a.width) return;
    const float* p = a.zcg + (long)s.row0 * 3 * a.width + c;
    typename Tr::elem* out = (typename Tr::elem*)a.out;
    float S = s.fresh ? 0.f : a.state[((long)s.slot * 2 + s.par) * a.width + c];
    const float* q = a.pair + (long)((int)blockIdx.y - s.index) * 2 * a.width + c;
    for (int i = 0; i < s.index; ++i) S = mmi_fma(q[(long)i * 2 * a.width], S, q[((long)i * 2 + 1) * a.width]);
    for (int i0 = 0; i0 < s.n; i0 += 8) {
        float z[8], u[8], g[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const long o = (long)(i0 + i < s.n ? i0 + i : s.n - 1) * 3 * a.width;
            z[i] = p[o];
            u[i] = p[o + a.width];
            g[i] = p[o + 2 * a.width];
        }
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i0 + i < s.n) {
                S = mmi_fma(1.0f - z[i], S, z[i] * u[i]);
                out[tlm_index<Tr>(s.row0 + i0 + i, c, a.out_ks)] = Tr::cvt(S * g[i]);
            }
    }
    if (s.last) a.state[((long)s.slot * 2 + (s.par ^ 1)) * a.width + c] = S;
}

// ------------------------------------------------------------------------------------------------
// sampling helpers
// ------------------------------------------------------------------------------------------------
// greedy: index of the largest logit, the lowest index on ties; out[map[row]] (map: row -> slot)
__global__ __launch_bounds__(256) void k_tlm_argmax(const float* __restrict__ logits, int V, const int* __restrict__ map, int* __restrict__ out,
                                                    int* __restrict__ last_tok) {
    MMI_SHARED float bv[256];
    MMI_SHARED int bi[256];
    const int tid = (int)threadIdx.x;
    const float* p = logits + (long)blockIdx.x * V;
    float best = -INFINITY;
    int at = 0;
    for (int i = tid; i < V; i += 256)
        if (p[i] > best) { best = p[i]; at = i; }
    bv[tid] = best;
    bi[tid] = at;
    __syncthreads();
    for (int s = 128; s > 0; s >>= 1) {
        if (tid < s && (bv[tid + s] > bv[tid] || (bv[tid + s] == bv[tid] && bi[tid + s] < bi[tid]))) {
            bv[tid] = bv[tid + s];
            bi[tid] = bi[tid + s];
        }
        __syncthreads();
    }
    if (tid == 0) {
        out[blockIdx.x] = bi[0];
        last_tok[map[blockIdx.x]] = bi[0];
    }
}
// fp32 logits -> the sampler's bf16 rows of ld columns (padding: -inf, never drawn)
__global__ void k_tlm_sample_rows(const float* __restrict__ logits, int V, uint16_t* __restrict__ dst, int ld, int n) {
    const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (long)n * ld) return;
    const int c = (int)(i % ld);
    dst[i] = c < V ? mmi_f32_to_bf16(logits[(i / ld) * V + c]) : (uint16_t)0xff80u;
}
__global__ void k_tlm_last_tok(const int* __restrict__ out, const int* __restrict__ map, int* __restrict__ last_tok, int n) {
    const int i = (int)(blockIdx.x * blockDim.x + threadIdx.x);
    if (i < n) last_tok[map[i]] = out[i];
}
