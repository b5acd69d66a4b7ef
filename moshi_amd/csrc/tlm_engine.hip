// Token language models behind the C ABI of include/moshi_tlm.h: decoder-only networks whose layers are described by mmi_tlm_cfg,
// stepped over mixed batches (prompt portions beside single tokens) from a paged cache and recurrent state slots.
//
//   step   = prepare (tokens, block tables, rotation tables) -> routing -> per layer run:
//              residual + norm(s) | mixer projections, feed-forward up | mixer core | mixer output, feed-forward down
//            -> residual + norm of the wanted rows -> head
//   The sublayers of a layer read norms of one input, so the mixer's input projection and the feed-forward's up projection are one
//   launch, and so are the mixer's output projection and the feed-forward's down projection (TlmJobs).
// Steps that only bring single tokens are captured into a hipGraph per shape (batch, wanted rows, attention split): everything that
// varies between two such steps is device memory uploaded in one copy.
#include "mmi_common.h"
#include "mmi_graph.h"
#include "../../include/moshi_tlm.h"
#include "lm_kernels.h"
#include "tlm_kernels.h"
#include "tlm_gqa.h"
#include "tlm_linear.h"

#include <math.h>
#include <algorithm>
#include <array>
#include <map>
#include <memory>
#include <tuple>
#include <type_traits>

int64_t mmi_copy_launch_log(const std::vector<std::string>& log, char* buf, int64_t cap);

namespace {

int round_up(int v, int m) { return (v + m - 1) / m * m; }

struct Mat {                       // one packed matrix, or `groups` of equal shape
    u32x4* wp = nullptr;
    int NT = 0, KS = 0;
    long gs = 0;                   // fragments x 64 per group
    long bytes() const { return gs * 16; }
};

struct Layer {
    mmi_tlm_layer c;
    float *norm = nullptr, *norm2 = nullptr, *ls1 = nullptr, *ls2 = nullptr;
    // minGRU
    Mat zcg, out;
    float* bias = nullptr;
    int wp = 0;
    // latent attention
    Mat in, uqn, uqr, uk, uv;
    float *qw = nullptr, *cw = nullptr;
    int qp = 0, kvp = 0, rp = 0, hp = 0, dim_p = 0, vdim_p = 0, lat_ks = 0, k_ks = 0, nd = 0, q_ks = 0, qn_ks = 0;
    int rope = -1, geo = -1;
    // grouped attention: `in` is [queries | keys | values]; k_ks, nd as above
    // channel delta: `in` is [q | k | v | beta], `lr` the low-rank halves of decay and gate, `a2` and `g2` the others; lightning: [q | k | v | gate]
    Mat lr, a2, g2;
    float *conv_w = nullptr, *decay = nullptr, *nw = nullptr;      // decay: (summand, factor) per column / powers of the constants
    int in_ld = 0, conv_c = 0, ra = 0, q0 = 0, k0 = 0, v0 = 0, b0 = 0;
    // feed-forward: experts, or one dense pair (gate and up rows alternate)
    Mat up, down;
    int route = -1;
    bool linear() const { return c.mixer == MMI_TLM_MIX_CHANNEL_DELTA || c.mixer == MMI_TLM_MIX_LIGHTNING; }
};

struct Run {                       // one execution of a layer: repeated layers share weights, not state
    int layer = 0;
    bool add_emb = false;
    int pass = -1;                 // first layer of a pass that starts with the projection of [x; embedding]
    void *kc = nullptr, *vc = nullptr;
    float *state = nullptr, *conv = nullptr;
};

struct Slot {
    bool live = false;
    int64_t pos = 0;
    int par = 0;                   // which copy of the recurrent state is current
    int64_t first_page = 0;        // pages before it have left every window
    std::vector<int> pages;        // pages[i] holds positions 64 (first_page + i) ..
    std::vector<int> kept;         // the sequence's first pages, once the windows have passed them but for the positions they keep
    int page(int64_t i) const { return i < first_page ? kept[(size_t)i] : pages[(size_t)(i - first_page)]; }
};

struct Staging {
    int* host = nullptr;
    hipEvent_t ev = nullptr;
    bool used = false;
};

// where the parts of a step's metadata sit in the uploaded block (ints)
struct Meta {
    int htok, pos, rslot, crow, prev, next, want, erow0, elen, epos0, eslot, tile0, seg, small, unit, chunk, upd, total;
};

struct Shape {                     // what a launch list depends on
    int T = 0, n_want = 0, n_entries = 0, n_seg = 0, nsplit = 1;
    bool pairs = false;            // some sequence spans several scan segments
    int n_small = 0, n_unit = 0, n_chunk = 0;      // sequences stepped token by token, sequences cut into chunks, their chunks
    std::vector<int> tiles;        // attention column tiles per head count
    std::vector<std::array<int, 2>> groups;        // column groups of 4 and of 8 tiles per head count
    std::vector<std::array<int, 3>> split;         // sequences of up to 64 columns: tiles; the others: groups of 4 and of 8 tiles
    Meta m;
    float* logits = nullptr;
    float* taps = nullptr;
};

}  // namespace

struct mmi_tlm {
    mmi_tlm_cfg cfg;
    std::vector<Layer> layers;
    std::vector<Run> runs;
    int device = 0;
    bool f32 = false;
    int kstep = 32, V = 8;
    int ld = 0, h_ks = 0;
    int max_slots = 0, max_pages = 0, max_T = 0;
    bool has_attn = false, has_latent = false, has_gru = false, has_linear = false;      // has_attn: some layer has a paged cache
    int64_t max_window = 0;        // 0: some layer sees every earlier position
    int keep_pages = 0;            // with windows: a sequence's first pages that are never released
    MmiArena wts, st, scratch;
    uint16_t *embed = nullptr, *bigram = nullptr, *pos_emb = nullptr;
    Mat loop_in;
    float* loop_step = nullptr;    // [times][ld]
    float* final_norm = nullptr;
    Mat head;
    std::vector<int> geo;          // distinct head counts
    std::vector<std::pair<double, int>> ropes;      // distinct (base, dims)
    std::vector<TlmRope> rope_host;
    TlmRope* rope_dev = nullptr;
    std::vector<TlmRouteLayer> route_host;
    TlmRouteLayer* route_dev = nullptr;
    int max_experts = 0, max_top = 0;
    long tile_ld = 0, list_ld = 0;
    // scratch
    float *x = nullptr, *mix = nullptr, *dn = nullptr, *zcg = nullptr, *lat = nullptr, *gate = nullptr, *pair = nullptr, *po = nullptr, *pml = nullptr;
    float *lin = nullptr, *qkv = nullptr, *dec = nullptr, *lgate = nullptr, *lo = nullptr, *cw = nullptr, *cq_g = nullptr, *ckt = nullptr, *cu0 = nullptr, *cp = nullptr,
          *cgend = nullptr;
    void *h2 = nullptr, *cat = nullptr, *lr = nullptr;
    int *brow = nullptr, *prev_tok = nullptr;
    void *h = nullptr, *y = nullptr, *cq = nullptr, *qn = nullptr, *q = nullptr, *ao = nullptr, *o = nullptr, *hid = nullptr;
    int *list = nullptr, *tiles = nullptr, *n_tiles = nullptr, *tok = nullptr, *meta = nullptr, *last_tok = nullptr, *block_table = nullptr;
    float* logits = nullptr;       // [max_slots][vocab] for captured steps
    uint16_t* samp_rows = nullptr; int samp_ld = 0;
    int* samp_map = nullptr; unsigned long long* samp_rng = nullptr; int* samp_zero = nullptr;
    uint64_t samp_count = 0;
    long split_elems = 0;          // partial-sum capacity of mix / dn / lat in rows
    // host state
    std::vector<Slot> slots;
    std::vector<int> free_pages;
    Staging staging[4];
    int stage_at = 0;
    size_t meta_cap = 0;
    float* taps = nullptr;
    bool graphs = true;
    hipStream_t cap_stream = nullptr;
    std::map<std::tuple<int, int, int>, std::unique_ptr<MmiProgram>> progs;
    std::vector<std::string> last_log;
    long weight_bytes = 0;
};

namespace {

constexpr int MAX_SPLIT = 8;
constexpr int ROWS_MAX = 64;       // up to here a step takes the weight-streaming kernel
constexpr int ATTN_TILE_GROUPS = 128;     // from this many column groups the attention stages keys through LDS
constexpr int PREFIXES = 6;        // prefix arrays over the sequences per head count: tiles, groups of 4, groups of 8, then those of `split`
constexpr int MAX_KEY_SPLIT = 16;
constexpr int MAX_PARTIALS = 512;  // (column tile, split) pairs of the attention

// ------------------------------------------------------------------------------------------------
// weights
// ------------------------------------------------------------------------------------------------
struct Loader {
    mmi_tlm* m;
    MmiWeights W;
    int* map = nullptr;            // device scratch for a row and a column map
    size_t map_cap = 0;
    ~Loader() { if (map) hipFree(map); }

    int find(const std::string& name, int dtype, std::initializer_list<int64_t> shape, const mmi_tensor_desc** out) {
        const mmi_tensor_desc* d = W.find(name);
        if (!d) return mmi_fail(MMI_ERR_MISSING_WEIGHT, "missing weight: " + name);
        if (d->dtype != dtype) return mmi_fail(MMI_ERR_UNSUPPORTED, "unexpected dtype of " + name);
        if (d->ndim != (int)shape.size()) return mmi_fail(MMI_ERR_SHAPE, "unexpected rank of " + name);
        int i = 0;
        for (int64_t s : shape) {
            if (d->shape[i] != s)
                return mmi_fail(MMI_ERR_SHAPE, "shape mismatch for " + name + ": dimension " + std::to_string(i) + " is " + std::to_string(d->shape[i]) +
                                                   ", expected " + std::to_string(s));
            ++i;
        }
        *out = d;
        return MMI_OK;
    }
    int upload(const std::vector<int>& a, const std::vector<int>& b) {
        const size_t n = a.size() + b.size();
        if (n > map_cap) {
            if (map) hipFree(map);
            map = nullptr;
            MMI_HIP_CHECK(hipMalloc((void**)&map, n * sizeof(int)));
            map_cap = n;
        }
        MMI_HIP_CHECK(hipDeviceSynchronize());
        MMI_HIP_CHECK(hipMemcpy(map, a.data(), a.size() * sizeof(int), hipMemcpyHostToDevice));
        if (!b.empty()) MMI_HIP_CHECK(hipMemcpy(map + a.size(), b.data(), b.size() * sizeof(int), hipMemcpyHostToDevice));
        return MMI_OK;
    }
    int alloc(Mat* mat, int groups, int NT, int KS) {
        mat->NT = NT;
        mat->KS = KS;
        mat->gs = (long)NT * KS * 64;
        MMI_HIP_CHECK(m->wts.alloc(&mat->wp, (size_t)groups * mat->gs));
        m->weight_bytes += groups * mat->bytes();
        return MMI_OK;
    }
    // tiles 0 .. rows/16 of the source (through the maps) become tiles t * tmul + toff of `dst`; the maps stay on the device until the
    // next upload, so packing many matrices of one shape uploads them once
    int pack(const mmi_tensor_desc* d, u32x4* dst, int rows, int cols, long sr, long sc, int tmul = 1, int toff = 0, long src_off = 0, int keep = 0) {
        const int NT = rows / 16, KS = cols / m->kstep;
        const long n = (long)NT * KS * 64 * m->V;
        const int blocks = (int)mmi_cdiv64(n, 256);
        const uint16_t* src = (const uint16_t*)d->data + src_off;
        if (m->f32) MMI_LAUNCH((k_tlm_pack<TlmF32>), blocks, 256, 0, (hipStream_t)0, src, sr, sc, map, map + rows, (float*)dst, NT, KS, tmul, toff, keep);
        else MMI_LAUNCH((k_tlm_pack<TlmBf16>), blocks, 256, 0, (hipStream_t)0, src, sr, sc, map, map + rows, (uint16_t*)dst, NT, KS, tmul, toff, keep);
        MMI_CHECK_LAUNCH();
        return MMI_OK;
    }
    int ident(int n, int padded_rows, int k, int padded_cols) {
        std::vector<int> a(padded_rows, -1), b(padded_cols, -1);
        for (int i = 0; i < n; ++i) a[i] = i;
        for (int i = 0; i < k; ++i) b[i] = i;
        return upload(a, b);
    }
    // plain [N][K] linear
    int linear(const std::string& name, int N, int K, Mat* mat) {
        const mmi_tensor_desc* d;
        int rc;
        const int rows = round_up(N, 16), cols = round_up(K, m->kstep);
        if ((rc = find(name, MMI_BF16, {N, K}, &d)) || (rc = alloc(mat, 1, rows / 16, cols / m->kstep)) || (rc = ident(N, rows, K, cols))) return rc;
        return pack(d, mat->wp, rows, cols, K, 1);
    }
    // a bf16 tensor's values on the host (small tensors)
    int host(const std::string& name, std::initializer_list<int64_t> shape, std::vector<float>* out) {
        const mmi_tensor_desc* d;
        int rc = find(name, MMI_BF16, shape, &d);
        if (rc) return rc;
        size_t n = 1;
        for (int64_t s : shape) n *= (size_t)s;
        std::vector<uint16_t> h(n);
        MMI_HIP_CHECK(hipMemcpy(h.data(), d->data, n * 2, hipMemcpyDeviceToHost));
        out->resize(n);
        for (size_t i = 0; i < n; ++i) (*out)[i] = mmi_bf16_to_f32(h[i]);
        return MMI_OK;
    }
    int to_device(const std::vector<float>& v, float** out) {
        MMI_HIP_CHECK(m->wts.alloc(out, v.size()));
        MMI_HIP_CHECK(hipMemcpy(*out, v.data(), v.size() * sizeof(float), hipMemcpyHostToDevice));
        return MMI_OK;
    }
    int table(const std::string& name, int64_t rows, int64_t cols, uint16_t** out) {
        const mmi_tensor_desc* d;
        int rc = find(name, MMI_BF16, {rows, cols}, &d);
        if (rc) return rc;
        MMI_HIP_CHECK(m->wts.alloc(out, (size_t)(rows * cols)));
        MMI_HIP_CHECK(hipMemcpy(*out, d->data, (size_t)(rows * cols) * 2, hipMemcpyDeviceToDevice));
        return MMI_OK;
    }
    // head by head linear [heads * n][K] -> tiles toff .. of `mat`, every head padded to np rows
    int heads(const std::string& name, int heads, int n, int np, int K, Mat* mat, int toff) {
        const mmi_tensor_desc* d;
        int rc;
        const int cols = mat->KS * m->kstep;
        std::vector<int> a(round_up(heads * np, 16), -1), b(cols, -1);
        for (int h = 0; h < heads; ++h)
            for (int i = 0; i < n; ++i) a[(size_t)h * np + i] = h * n + i;
        for (int i = 0; i < K; ++i) b[i] = i;
        if ((rc = find(name, MMI_BF16, {(int64_t)heads * n, K}, &d)) || (rc = upload(a, b))) return rc;
        return pack(d, mat->wp, (int)a.size(), cols, K, 1, 1, toff);
    }
    // output projection [N][heads * n] over heads padded to np
    int over_heads(const std::string& name, int N, int heads, int n, int np, Mat* mat) {
        const mmi_tensor_desc* d;
        int rc;
        const int rows = round_up(N, 16), cols = round_up(heads * np, m->kstep);
        std::vector<int> a(rows, -1), b(cols, -1);
        for (int i = 0; i < N; ++i) a[i] = i;
        for (int h = 0; h < heads; ++h)
            for (int j = 0; j < n; ++j) b[(size_t)h * np + j] = h * n + j;
        if ((rc = find(name, MMI_BF16, {N, (int64_t)heads * n}, &d)) || (rc = alloc(mat, 1, rows / 16, cols / m->kstep)) || (rc = upload(a, b))) return rc;
        return pack(d, mat->wp, rows, cols, (long)heads * n, 1);
    }
    int vec(const std::string& name, int n, int padded, float** out) {
        const mmi_tensor_desc* d;
        int rc = find(name, MMI_BF16, {n}, &d);
        if (rc) return rc;
        MMI_HIP_CHECK(m->wts.alloc(out, padded));
        return vec_into(d, n, padded, *out);
    }
    int vec_into(const mmi_tensor_desc* d, int n, int padded, float* out) {
        std::vector<int> a(padded, -1);
        for (int i = 0; i < n; ++i) a[i] = i;
        int rc = upload(a, {});
        if (rc) return rc;
        MMI_LAUNCH(k_tlm_vec, mmi_cdiv(padded, 256), 256, 0, (hipStream_t)0, (const uint16_t*)d->data, map, out, padded);
        MMI_CHECK_LAUNCH();
        return MMI_OK;
    }
};

int load_mingru(Loader& ld, Layer& L, const std::string& p) {
    mmi_tlm* m = ld.m;
    const int w = L.c.width, D = m->cfg.width;
    L.wp = round_up(w, 16);
    const int cols = round_up(D, m->kstep);
    int rc;
    if ((rc = ld.alloc(&L.zcg, 1, 3 * L.wp / 16, cols / m->kstep)) || (rc = ld.ident(w, L.wp, D, cols))) return rc;
    const char* parts[3] = {"z", "x", "g"};
    const mmi_tensor_desc* d;
    for (int k = 0; k < 3; ++k) {
        if ((rc = ld.find(p + ".mix." + parts[k], MMI_BF16, {w, D}, &d))) return rc;
        if ((rc = ld.pack(d, L.zcg.wp, L.wp, cols, D, 1, 3, k))) return rc;
    }
    MMI_HIP_CHECK(m->wts.alloc(&L.bias, (size_t)2 * L.wp));
    for (int k = 0; k < 2; ++k) {
        if ((rc = ld.find(p + ".mix." + parts[k] + ".b", MMI_BF16, {w}, &d)) || (rc = ld.vec_into(d, w, L.wp, L.bias + (size_t)k * L.wp))) return rc;
    }
    return ld.linear(p + ".mix.o", D, w, &L.out);
}

int load_latent_attention(Loader& ld, Layer& L, const std::string& p) {
    mmi_tlm* m = ld.m;
    const mmi_tlm_layer& c = L.c;
    const int D = m->cfg.width, H = c.heads, ks = m->kstep, hd = c.dim + c.rot_dim;
    L.qp = round_up(c.q_rank, 16);
    L.kvp = round_up(c.kv_rank, 16);
    L.rp = round_up(c.rot_dim, 16);
    L.hp = round_up(H, 16);
    L.dim_p = round_up(c.dim, ks);
    L.vdim_p = round_up(c.vdim, 16);
    L.lat_ks = round_up(c.kv_rank, ks) / ks;
    L.k_ks = L.lat_ks + round_up(c.rot_dim, ks) / ks;
    L.nd = L.kvp / 16;
    L.q_ks = round_up(c.q_rank, ks) / ks;
    L.qn_ks = H * L.dim_p / ks;
    auto turn = [&](int j) { return j / 2 + (j & 1) * (c.rot_dim / 2); };     // rotation partners side by side
    const mmi_tensor_desc* d;
    int rc;
    const std::string mx = p + ".mix.";
    // [query latent | latent | rotated key part | gates] of one input projection
    const int cols = round_up(D, ks);
    std::vector<int> cm(cols, -1);
    for (int i = 0; i < D; ++i) cm[i] = i;
    if ((rc = ld.alloc(&L.in, 1, (L.qp + L.kvp + L.rp + L.hp) / 16, cols / ks))) return rc;
    if ((rc = ld.find(mx + "dq", MMI_BF16, {c.q_rank, D}, &d)) || (rc = ld.ident(c.q_rank, L.qp, D, cols)) || (rc = ld.pack(d, L.in.wp, L.qp, cols, D, 1))) return rc;
    if ((rc = ld.find(mx + "dkv", MMI_BF16, {c.kv_rank + c.rot_dim, D}, &d)) || (rc = ld.ident(c.kv_rank, L.kvp, D, cols)) ||
        (rc = ld.pack(d, L.in.wp, L.kvp, cols, D, 1, 1, L.qp / 16)))
        return rc;
    if (L.rp) {
        std::vector<int> rm(L.rp, -1);
        for (int j = 0; j < c.rot_dim; ++j) rm[j] = c.kv_rank + turn(j);
        if ((rc = ld.upload(rm, cm)) || (rc = ld.pack(d, L.in.wp, L.rp, cols, D, 1, 1, (L.qp + L.kvp) / 16))) return rc;
    }
    if ((rc = ld.find(mx + "g", MMI_BF16, {H, D}, &d)) || (rc = ld.ident(H, L.hp, D, cols)) ||
        (rc = ld.pack(d, L.in.wp, L.hp, cols, D, 1, 1, (L.qp + L.kvp + L.rp) / 16)))
        return rc;
    if ((rc = ld.vec(mx + "dq.norm", c.q_rank, L.qp, &L.qw)) || (rc = ld.vec(mx + "dkv.norm", c.kv_rank, L.kvp, &L.cw))) return rc;
    // queries: un-rotated parts head by head, then rotated parts (one group per head)
    if ((rc = ld.find(mx + "uq", MMI_BF16, {(int64_t)H * hd, c.q_rank}, &d))) return rc;
    {
        const int qc = L.q_ks * ks;
        std::vector<int> rm((size_t)H * L.dim_p, -1), qm(qc, -1);
        for (int i = 0; i < c.q_rank; ++i) qm[i] = i;
        for (int h = 0; h < H; ++h)
            for (int j = 0; j < c.dim; ++j) rm[(size_t)h * L.dim_p + j] = h * hd + j;
        if ((rc = ld.alloc(&L.uqn, 1, (int)rm.size() / 16, L.q_ks)) || (rc = ld.upload(rm, qm)) || (rc = ld.pack(d, L.uqn.wp, (int)rm.size(), qc, c.q_rank, 1))) return rc;
        if (L.rp) {
            std::vector<int> rr((size_t)H * L.rp, -1);
            for (int h = 0; h < H; ++h)
                for (int j = 0; j < c.rot_dim; ++j) rr[(size_t)h * L.rp + j] = h * hd + c.dim + turn(j);
            if ((rc = ld.alloc(&L.uqr, H, L.rp / 16, L.q_ks)) || (rc = ld.upload(rr, qm)) || (rc = ld.pack(d, L.uqr.wp, (int)rr.size(), qc, c.q_rank, 1))) return rc;
        }
    }
    // key projection, transposed per head (it is applied to the query), and value projection per head
    if ((rc = ld.find(mx + "uk", MMI_BF16, {(int64_t)H * c.dim, c.kv_rank}, &d)) || (rc = ld.alloc(&L.uk, H, L.kvp / 16, L.dim_p / ks)) ||
        (rc = ld.ident(c.kv_rank, L.kvp, c.dim, L.dim_p)))
        return rc;
    for (int h = 0; h < H; ++h)
        if ((rc = ld.pack(d, L.uk.wp + h * L.uk.gs, L.kvp, L.dim_p, 1, c.kv_rank, 1, 0, (long)h * c.dim * c.kv_rank))) return rc;
    if ((rc = ld.find(mx + "uv", MMI_BF16, {(int64_t)H * c.vdim, c.kv_rank}, &d)) || (rc = ld.alloc(&L.uv, H, L.vdim_p / 16, L.lat_ks)) ||
        (rc = ld.ident(c.vdim, L.vdim_p, c.kv_rank, L.lat_ks * ks)))
        return rc;
    for (int h = 0; h < H; ++h)
        if ((rc = ld.pack(d, L.uv.wp + h * L.uv.gs, L.vdim_p, L.lat_ks * ks, c.kv_rank, 1, 1, 0, (long)h * c.vdim * c.kv_rank))) return rc;
    // output projection over the padded heads
    const int ok = round_up(H * L.vdim_p, ks), rows = round_up(D, 16);
    std::vector<int> rm(rows, -1), om(ok, -1);
    for (int i = 0; i < D; ++i) rm[i] = i;
    for (int h = 0; h < H; ++h)
        for (int j = 0; j < c.vdim; ++j) om[h * L.vdim_p + j] = h * c.vdim + j;
    if ((rc = ld.find(mx + "o", MMI_BF16, {D, (int64_t)H * c.vdim}, &d)) || (rc = ld.alloc(&L.out, 1, rows / 16, ok / ks)) || (rc = ld.upload(rm, om))) return rc;
    return ld.pack(d, L.out.wp, rows, ok, (long)H * c.vdim, 1);
}

int load_attention(Loader& ld, Layer& L, const std::string& p) {
    mmi_tlm* m = ld.m;
    const mmi_tlm_layer& c = L.c;
    const int D = m->cfg.width, H = c.heads, G = c.kv_heads, ks = m->kstep;
    L.dim_p = round_up(c.dim, ks);
    L.vdim_p = round_up(c.vdim, 16);
    L.k_ks = L.dim_p / ks;
    L.nd = L.vdim_p / 16;
    const std::string mx = p + ".mix.";
    int rc;
    if ((rc = ld.alloc(&L.in, 1, ((H + G) * L.dim_p + G * L.vdim_p) / 16, round_up(D, ks) / ks)) || (rc = ld.heads(mx + "q", H, c.dim, L.dim_p, D, &L.in, 0)) ||
        (rc = ld.heads(mx + "k", G, c.dim, L.dim_p, D, &L.in, H * L.dim_p / 16)) ||
        (rc = ld.heads(mx + "v", G, c.vdim, L.vdim_p, D, &L.in, (H + G) * L.dim_p / 16)))
        return rc;
    return ld.over_heads(mx + "o", D, H, c.vdim, L.vdim_p, &L.out);
}

// queries, keys, values of a mixer with a matrix state, and one more section of `extra` heads of `extra_n` columns
int load_linear_in(Loader& ld, Layer& L, const std::string& mx, int QH, const char* extra, int extra_heads, int extra_n) {
    mmi_tlm* m = ld.m;
    const mmi_tlm_layer& c = L.c;
    const int D = m->cfg.width, H = c.heads;
    L.dim_p = round_up(c.dim, 16);
    L.vdim_p = round_up(c.vdim, 16);
    L.q0 = 0;
    L.k0 = QH * L.dim_p;
    L.v0 = 2 * QH * L.dim_p;
    L.b0 = L.v0 + H * L.vdim_p;
    const int extra_p = extra_heads > 1 && extra_n > 1 ? round_up(extra_n, 16) : (extra_n > 1 ? L.vdim_p : 1);
    L.in_ld = L.b0 + round_up(extra_heads * extra_p, 16);
    int rc;
    if ((rc = ld.alloc(&L.in, 1, L.in_ld / 16, round_up(D, m->kstep) / m->kstep)) || (rc = ld.heads(mx + "q", QH, c.dim, L.dim_p, D, &L.in, 0)) ||
        (rc = ld.heads(mx + "k", QH, c.dim, L.dim_p, D, &L.in, L.k0 / 16)) || (rc = ld.heads(mx + "v", H, c.vdim, L.vdim_p, D, &L.in, L.v0 / 16)) ||
        (rc = ld.heads(mx + extra, extra_heads, extra_n, extra_p, D, &L.in, L.b0 / 16)))
        return rc;
    return ld.over_heads(mx + "o", D, H, c.vdim, L.vdim_p, &L.out);
}

int load_channel_delta(Loader& ld, Layer& L, const std::string& p) {
    mmi_tlm* m = ld.m;
    const mmi_tlm_layer& c = L.c;
    const int D = m->cfg.width, H = c.heads, G = c.kv_heads, ks = m->kstep;
    const std::string mx = p + ".mix.";
    int rc;
    if ((rc = load_linear_in(ld, L, mx, G, "b", H, 1))) return rc;
    L.conv_c = L.b0;
    const char* parts[3] = {"q", "k", "v"};
    std::vector<float> src, w((size_t)c.conv * L.conv_c, 0.f);
    for (int k = 0; k < 3; ++k) {
        const int nh = k == 2 ? H : G, n = k == 2 ? c.vdim : c.dim, np = k == 2 ? L.vdim_p : L.dim_p, c0 = k == 0 ? L.q0 : (k == 1 ? L.k0 : L.v0);
        if ((rc = ld.host(mx + parts[k] + ".conv", {(int64_t)nh * n, c.conv}, &src))) return rc;
        for (int h = 0; h < nh; ++h)
            for (int i = 0; i < n; ++i)
                for (int j = 0; j < c.conv; ++j) w[(size_t)j * L.conv_c + c0 + h * np + i] = src[((size_t)h * n + i) * c.conv + j];
    }
    if ((rc = ld.to_device(w, &L.conv_w))) return rc;
    // decay: exp(-factor softplus(x + summand)), factor = exp(A_log) of the head
    std::vector<float> alog, bias;
    if ((rc = ld.host(mx + "A_log", {H}, &alog)) || (rc = ld.host(mx + "dt_bias", {(int64_t)H * c.dim}, &bias))) return rc;
    const int dcols = H * L.dim_p;
    std::vector<float> dec((size_t)2 * dcols, 0.f);
    for (int h = 0; h < H; ++h)
        for (int i = 0; i < L.dim_p; ++i) {
            dec[(size_t)h * L.dim_p + i] = i < c.dim ? bias[(size_t)h * c.dim + i] : 0.f;
            dec[(size_t)dcols + h * L.dim_p + i] = (float)exp((double)alog[h]);
        }
    if ((rc = ld.to_device(dec, &L.decay)) || (rc = ld.vec(mx + "norm", c.vdim, L.vdim_p, &L.nw))) return rc;
    // low-rank halves: both read the layer's norm, so they are one matrix
    L.ra = round_up(c.decay_rank, ks);
    const int rg = round_up(c.gate_rank, ks), cols = round_up(D, ks) / ks;
    if ((rc = ld.alloc(&L.lr, 1, (L.ra + rg) / 16, cols)) || (rc = ld.heads(mx + "a1", 1, c.decay_rank, L.ra, D, &L.lr, 0)) ||
        (rc = ld.heads(mx + "g1", 1, c.gate_rank, rg, D, &L.lr, L.ra / 16)) || (rc = ld.alloc(&L.a2, 1, dcols / 16, L.ra / ks)) ||
        (rc = ld.heads(mx + "a2", H, c.dim, L.dim_p, c.decay_rank, &L.a2, 0)) || (rc = ld.alloc(&L.g2, 1, H * L.vdim_p / 16, rg / ks)))
        return rc;
    return ld.heads(mx + "g2", H, c.vdim, L.vdim_p, c.gate_rank, &L.g2, 0);
}

int load_lightning(Loader& ld, Layer& L, const std::string& p) {
    const mmi_tlm_layer& c = L.c;
    const int H = c.heads;
    const std::string mx = p + ".mix.";
    int rc;
    if ((rc = load_linear_in(ld, L, mx, H, "g", H, c.vdim))) return rc;
    std::vector<float> w, wp((size_t)H * L.vdim_p, 0.f), pw((size_t)H * (TLM_CHUNK + 1));
    if ((rc = ld.host(mx + "norm", {(int64_t)H * c.vdim}, &w))) return rc;
    for (int h = 0; h < H; ++h) {
        for (int i = 0; i < c.vdim; ++i) wp[(size_t)h * L.vdim_p + i] = w[(size_t)h * c.vdim + i];
        for (int i = 0; i <= TLM_CHUNK; ++i) pw[(size_t)h * (TLM_CHUNK + 1) + i] = (float)pow(c.decay[h], i);
    }
    if ((rc = ld.to_device(wp, &L.nw))) return rc;
    return ld.to_device(pw, &L.decay);
}

int load_dense_glu(Loader& ld, Layer& L, const std::string& p) {
    mmi_tlm* m = ld.m;
    const int D = m->cfg.width, F = L.c.ff, rows = round_up(2 * F, 16), cols = round_up(D, m->kstep);
    const mmi_tensor_desc* d;
    int rc;
    if ((rc = ld.alloc(&L.up, 1, rows / 16, cols / m->kstep))) return rc;
    std::vector<int> cm(cols, -1);
    for (int i = 0; i < D; ++i) cm[i] = i;
    for (int k = 0; k < 2; ++k) {                         // gate rows (the others zero), then the up rows between them
        std::vector<int> rm(rows, -1);
        for (int i = 0; i < F; ++i) rm[2 * i + k] = i;
        if ((rc = ld.find(p + (k ? ".mlp.up" : ".mlp.gate"), MMI_BF16, {F, D}, &d)) || (rc = ld.upload(rm, cm)) ||
            (rc = ld.pack(d, L.up.wp, rows, cols, D, 1, 1, 0, 0, k)))
            return rc;
    }
    return ld.linear(p + ".mlp.down", D, F, &L.down);
}

int load_moe(Loader& ld, Layer& L, const std::string& p) {
    mmi_tlm* m = ld.m;
    const mmi_tlm_layer& c = L.c;
    const int D = m->cfg.width, E = c.experts, rows_u = round_up(c.ff, 16), cols_u = round_up(D, m->kstep), rows_d = round_up(D, 16), cols_d = round_up(c.ff, m->kstep);
    const mmi_tensor_desc* d;
    int rc;
    if ((rc = ld.alloc(&L.up, E, rows_u / 16, cols_u / m->kstep)) || (rc = ld.alloc(&L.down, E, rows_d / 16, cols_d / m->kstep))) return rc;
    if ((rc = ld.ident(c.ff, rows_u, D, cols_u))) return rc;
    for (int e = 0; e < E; ++e)
        if ((rc = ld.find(p + ".mlp.e" + std::to_string(e) + ".up", MMI_BF16, {c.ff, D}, &d)) || (rc = ld.pack(d, L.up.wp + e * L.up.gs, rows_u, cols_u, D, 1))) return rc;
    if ((rc = ld.ident(D, rows_d, c.ff, cols_d))) return rc;
    for (int e = 0; e < E; ++e)
        if ((rc = ld.find(p + ".mlp.e" + std::to_string(e) + ".down", MMI_BF16, {D, c.ff}, &d)) || (rc = ld.pack(d, L.down.wp + e * L.down.gs, rows_d, cols_d, c.ff, 1))) return rc;
    if ((rc = ld.find(p + ".mlp.table", MMI_I32, {m->cfg.vocab, c.top}, &d))) return rc;
    const size_t n = (size_t)m->cfg.vocab * c.top;
    std::vector<int> t(n);
    MMI_HIP_CHECK(hipMemcpy(t.data(), d->data, n * sizeof(int), hipMemcpyDeviceToHost));
    for (size_t i = 0; i < n; ++i)
        if (t[i] < 0 || t[i] >= E) return mmi_fail(MMI_ERR_INVALID, p + ".mlp.table names an expert that does not exist");
    int* dev = nullptr;
    MMI_HIP_CHECK(m->wts.alloc(&dev, n));
    MMI_HIP_CHECK(hipMemcpy(dev, d->data, n * sizeof(int), hipMemcpyDeviceToDevice));
    L.route = (int)m->route_host.size();
    m->route_host.push_back(TlmRouteLayer{dev, E, c.top});
    m->max_experts = std::max(m->max_experts, E);
    m->max_top = std::max(m->max_top, c.top);
    return MMI_OK;
}

int check_cfg(const mmi_tlm_cfg& c) {
    if (c.vocab < 1 || c.width < 1 || c.n_layers < 1 || !c.layers) return mmi_fail(MMI_ERR_INVALID, "token LM: empty configuration");
    if (c.dtype != MMI_BF16 && c.dtype != MMI_F32) return mmi_fail(MMI_ERR_UNSUPPORTED, "token LM: dtype must be bf16 or fp32");
    if (c.norm_groups < 1 || c.width % c.norm_groups) return mmi_fail(MMI_ERR_INVALID, "token LM: width must be a multiple of the norm groups");
    if (c.width > 8192) return mmi_fail(MMI_ERR_UNSUPPORTED, "token LM: width above 8192");
    if (c.loop_start < 0 || c.loop_stop < c.loop_start || c.loop_stop > c.n_layers || (c.loop_stop > c.loop_start && c.loop_times < 1))
        return mmi_fail(MMI_ERR_INVALID, "token LM: bad layer repetition");
    if (c.loop_inject != MMI_TLM_LOOP_ADD && c.loop_inject != MMI_TLM_LOOP_PROJECT) return mmi_fail(MMI_ERR_UNSUPPORTED, "token LM: unknown start of a pass");
    if (c.norms < 1 || c.norms > 2) return mmi_fail(MMI_ERR_INVALID, "token LM: one or two norms per layer");
    if (c.bigram_buckets < 0 || c.max_positions < 0) return mmi_fail(MMI_ERR_INVALID, "token LM: embedding sizes");
    for (int i = 0; i < c.n_layers; ++i) {
        const mmi_tlm_layer& l = c.layers[i];
        const std::string at = "token LM, layer " + std::to_string(i) + ": ";
        if (l.mixer == MMI_TLM_MIX_MINGRU) {
            if (l.width < 1) return mmi_fail(MMI_ERR_INVALID, at + "minGRU width");
        } else if (l.mixer == MMI_TLM_MIX_LATENT_ATTENTION) {
            if (l.heads < 1 || l.dim < 1 || l.vdim < 1 || l.q_rank < 1 || l.kv_rank < 1 || l.rot_dim < 0 || l.rot_dim % 2 || l.window < 0)
                return mmi_fail(MMI_ERR_INVALID, at + "latent attention sizes");
            if (l.kv_rank > 512) return mmi_fail(MMI_ERR_UNSUPPORTED, at + "kv_rank above 512");
            if (l.rot_dim > 128) return mmi_fail(MMI_ERR_UNSUPPORTED, at + "rot_dim above 128");
            if (round_up(l.q_rank, 16) + round_up(l.kv_rank, 16) + round_up(l.rot_dim, 16) + round_up(l.heads, 16) > 8192)
                return mmi_fail(MMI_ERR_UNSUPPORTED, at + "query latent above the kernel's row buffer");
        } else if (l.mixer == MMI_TLM_MIX_ATTENTION || l.mixer == MMI_TLM_MIX_CHANNEL_DELTA || l.mixer == MMI_TLM_MIX_LIGHTNING) {
            const bool shared = l.mixer != MMI_TLM_MIX_LIGHTNING;
            if (l.heads < 1 || l.dim < 1 || l.vdim < 1 || (shared && (l.kv_heads < 1 || l.heads % l.kv_heads))) return mmi_fail(MMI_ERR_INVALID, at + "head sizes");
            if (l.dim > 256 || l.vdim > 256) return mmi_fail(MMI_ERR_UNSUPPORTED, at + "heads above 256 dimensions");
            if (l.heads > 65535) return mmi_fail(MMI_ERR_UNSUPPORTED, at + "more than 65535 heads");
            if (l.mixer == MMI_TLM_MIX_ATTENTION && (l.window < 0 || l.keep_first < 0)) return mmi_fail(MMI_ERR_INVALID, at + "attention window");
            if (l.mixer == MMI_TLM_MIX_CHANNEL_DELTA && (l.conv < 1 || l.decay_rank < 1 || l.gate_rank < 1)) return mmi_fail(MMI_ERR_INVALID, at + "delta rule sizes");
            if (l.mixer == MMI_TLM_MIX_LIGHTNING && !l.decay) return mmi_fail(MMI_ERR_INVALID, at + "no decay");
        } else {
            return mmi_fail(MMI_ERR_UNSUPPORTED, at + "unknown mixer");
        }
        if (l.mlp == MMI_TLM_MLP_MOE) {
            if (l.experts < 1 || l.top < 1 || l.top > l.experts || l.ff < 1) return mmi_fail(MMI_ERR_INVALID, at + "expert sizes");
            if (l.experts > 4096) return mmi_fail(MMI_ERR_UNSUPPORTED, at + "more than 4096 experts");
            if (l.act != MMI_TLM_ACT_RELU2 || l.router != MMI_TLM_ROUTE_TOKEN_TABLE) return mmi_fail(MMI_ERR_UNSUPPORTED, at + "unknown expert activation or router");
        } else if (l.mlp == MMI_TLM_MLP_DENSE) {
            if (l.ff < 1 || !(l.limit > 0.f)) return mmi_fail(MMI_ERR_INVALID, at + "feed-forward sizes");
            if (l.act != MMI_TLM_ACT_CLAMPED_SWIGLU) return mmi_fail(MMI_ERR_UNSUPPORTED, at + "unknown feed-forward activation");
        } else if (l.mlp != MMI_TLM_MLP_NONE) {
            return mmi_fail(MMI_ERR_UNSUPPORTED, at + "unknown feed-forward");
        }
    }
    return MMI_OK;
}

// ------------------------------------------------------------------------------------------------
// buffers
// ------------------------------------------------------------------------------------------------
int alloc_packed(mmi_tlm* m, void** p, long rows, int ks) {
    const size_t n = (size_t)((rows + 15) / 16) * ks * 64;
    u32x4* q = nullptr;
    MMI_HIP_CHECK(m->scratch.alloc(&q, n));
    MMI_HIP_CHECK(hipMemset(q, 0, n * 16));              // padding columns are read (times zero weights): keep them finite
    *p = q;
    return MMI_OK;
}
int alloc_f32(mmi_tlm* m, float** p, size_t n) {
    MMI_HIP_CHECK(m->scratch.alloc(p, n));
    MMI_HIP_CHECK(hipMemset(*p, 0, std::max<size_t>(n, 1) * sizeof(float)));
    return MMI_OK;
}

int table_ld(const mmi_tlm* m) { return m->keep_pages + std::max(1, m->max_pages); }      // block-table entries per slot

int alloc_buffers(mmi_tlm* m) {
    const mmi_tlm_cfg& c = m->cfg;
    const int T = m->max_T;
    int rc;
    m->split_elems = std::max((long)T, (long)MAX_SPLIT * ROWS_MAX);
    int gru_w = 0, y_ks = 0, lat_ld = 0, cq_ks = 0, qn_ks = 0, o_ks = 0, hid_ks = 0, gate_ld = 0, nd = 0;
    long q_elems = 0, ao_elems = 0;
    long lin_ld = 0, conv_c = 0, dec_ld = 0, lgate_ld = 0, lo_ld = 0, heads = 0, hd = 0, hv = 0;
    int lr_ks = 0;
    for (const Layer& L : m->layers) {
        if (L.c.mixer == MMI_TLM_MIX_MINGRU) {
            gru_w = std::max(gru_w, L.wp);
            y_ks = std::max(y_ks, L.out.KS);
        } else if (L.c.mixer == MMI_TLM_MIX_ATTENTION) {
            q_elems = std::max(q_elems, (long)((T * (long)L.c.heads + 15) / 16) * L.k_ks);
            o_ks = std::max(o_ks, L.out.KS);
            nd = std::max(nd, L.nd);
        } else if (L.linear()) {
            lin_ld = std::max(lin_ld, (long)L.in_ld);
            conv_c = std::max(conv_c, (long)L.conv_c);
            heads = std::max(heads, (long)L.c.heads);
            hd = std::max(hd, (long)L.c.heads * L.dim_p);
            hv = std::max(hv, (long)L.c.heads * L.vdim_p);
            o_ks = std::max(o_ks, L.out.KS);
            if (L.c.mixer == MMI_TLM_MIX_CHANNEL_DELTA) {
                lr_ks = std::max(lr_ks, L.lr.NT * 16 / m->kstep);
                dec_ld = std::max(dec_ld, (long)L.c.heads * L.dim_p);
                lgate_ld = std::max(lgate_ld, (long)L.c.heads * L.vdim_p);
            }
            lo_ld = std::max(lo_ld, (long)L.c.heads * L.vdim_p);
        } else {
            lat_ld = std::max(lat_ld, L.qp + L.kvp + L.rp + L.hp);
            cq_ks = std::max(cq_ks, L.q_ks);
            qn_ks = std::max(qn_ks, L.qn_ks);
            q_elems = std::max(q_elems, (long)((T * (long)L.c.heads + 15) / 16) * L.k_ks);
            ao_elems = std::max(ao_elems, (long)round_up(T, 16) / 16 * L.c.heads * L.lat_ks);
            o_ks = std::max(o_ks, L.out.KS);
            gate_ld = std::max(gate_ld, L.c.heads);
            nd = std::max(nd, L.nd);
        }
        if (L.c.mlp != MMI_TLM_MLP_NONE) hid_ks = std::max(hid_ks, L.down.KS);
    }
    if ((rc = alloc_f32(m, &m->x, (size_t)T * m->ld)) || (rc = alloc_packed(m, &m->h, std::max(T, m->max_slots), m->h_ks)) ||
        (rc = alloc_f32(m, &m->mix, (size_t)m->split_elems * m->ld)))
        return rc;
    if (m->has_gru) {
        const int n_seg = T / TLM_SEG + m->max_slots + 1;
        if ((rc = alloc_f32(m, &m->zcg, (size_t)T * 3 * gru_w)) || (rc = alloc_packed(m, &m->y, T, y_ks)) || (rc = alloc_f32(m, &m->pair, (size_t)n_seg * 2 * gru_w))) return rc;
    }
    if (c.norms == 2 && (rc = alloc_packed(m, &m->h2, std::max(T, m->max_slots), m->h_ks))) return rc;
    if (m->loop_in.wp && (rc = alloc_packed(m, &m->cat, T, 2 * m->h_ks))) return rc;
    if (m->has_linear) {
        const size_t n_chunk = (size_t)T / TLM_CHUNK + std::min(m->max_slots, T / (TLM_SMALL + 1)) + 1;      // only sequences above TLM_SMALL tokens have any
        if ((rc = alloc_f32(m, &m->lin, (size_t)T * lin_ld)) || (rc = alloc_f32(m, &m->qkv, (size_t)T * conv_c)) || (rc = alloc_f32(m, &m->dec, (size_t)T * dec_ld)) ||
            (rc = alloc_f32(m, &m->lgate, (size_t)T * lgate_ld)) || (rc = alloc_f32(m, &m->lo, (size_t)T * lo_ld)) || (rc = alloc_packed(m, &m->lr, T, std::max(1, lr_ks))) ||
            (rc = alloc_f32(m, &m->cw, conv_c ? n_chunk * TLM_CHUNK * hd : 1)) || (rc = alloc_f32(m, &m->cq_g, n_chunk * TLM_CHUNK * hd)) ||
            (rc = alloc_f32(m, &m->ckt, n_chunk * TLM_CHUNK * hd)) || (rc = alloc_f32(m, &m->cu0, conv_c ? n_chunk * TLM_CHUNK * hv : 1)) ||
            (rc = alloc_f32(m, &m->cp, n_chunk * TLM_CHUNK * TLM_CHUNK * heads)) || (rc = alloc_f32(m, &m->cgend, n_chunk * hd)))
            return rc;
    }
    if (m->has_attn && !m->has_latent) {
        if ((rc = alloc_packed(m, &m->q, q_elems * 16, 1)) || (rc = alloc_f32(m, &m->po, (size_t)MAX_PARTIALS * nd * 256)) || (rc = alloc_f32(m, &m->pml, (size_t)MAX_PARTIALS * 32)))
            return rc;
    }
    if (!m->has_latent && (m->has_attn || m->has_linear) && (rc = alloc_packed(m, &m->o, T, o_ks))) return rc;
    if (c.bigram_buckets > 0) {
        MMI_HIP_CHECK(m->scratch.alloc(&m->brow, T));
        MMI_HIP_CHECK(m->scratch.alloc(&m->prev_tok, 2 * (size_t)m->max_slots));
        MMI_HIP_CHECK(hipMemset(m->prev_tok, 0, 2 * (size_t)m->max_slots * sizeof(int)));
    }
    if (m->has_latent) {
        if ((rc = alloc_f32(m, &m->lat, (size_t)m->split_elems * lat_ld)) || (rc = alloc_packed(m, &m->cq, T, cq_ks)) || (rc = alloc_packed(m, &m->qn, T, qn_ks)) ||
            (rc = alloc_packed(m, &m->q, q_elems * 16, 1)) || (rc = alloc_packed(m, &m->ao, ao_elems * 16, 1)) || (rc = alloc_packed(m, &m->o, T, o_ks)) ||
            (rc = alloc_f32(m, &m->gate, (size_t)T * gate_ld)) || (rc = alloc_f32(m, &m->po, (size_t)MAX_PARTIALS * nd * 256)) ||
            (rc = alloc_f32(m, &m->pml, (size_t)MAX_PARTIALS * 32)))
            return rc;
        for (TlmRope& r : m->rope_host)
            if ((rc = alloc_f32(m, &r.out, (size_t)T * r.ld * 2))) return rc;
    }
    if (m->route_host.empty() && hid_ks) {
        if ((rc = alloc_packed(m, &m->hid, T, hid_ks)) || (rc = alloc_f32(m, &m->dn, (size_t)std::max((long)T, (long)MAX_SPLIT * ROWS_MAX) * m->ld))) return rc;
    }
    if (!m->route_host.empty()) {
        const size_t nl = m->route_host.size();
        m->list_ld = (long)T * m->max_top;
        m->tile_ld = (long)T * m->max_top / 16 + m->max_experts + 1;
        if ((rc = alloc_packed(m, &m->hid, (long)T * m->max_top, hid_ks)) ||
            (rc = alloc_f32(m, &m->dn, (size_t)std::max((long)T, (long)MAX_SPLIT * ROWS_MAX) * m->max_top * m->ld)))
            return rc;
        MMI_HIP_CHECK(m->scratch.alloc(&m->list, nl * m->list_ld));
        MMI_HIP_CHECK(m->scratch.alloc(&m->tiles, nl * m->tile_ld * 3));
        MMI_HIP_CHECK(m->scratch.alloc(&m->n_tiles, nl));
        MMI_HIP_CHECK(m->scratch.alloc(&m->route_dev, nl));
        MMI_HIP_CHECK(hipMemcpy(m->route_dev, m->route_host.data(), nl * sizeof(TlmRouteLayer), hipMemcpyHostToDevice));
    }
    MMI_HIP_CHECK(m->scratch.alloc(&m->rope_dev, std::max<size_t>(1, m->rope_host.size())));
    if (!m->rope_host.empty()) MMI_HIP_CHECK(hipMemcpy(m->rope_dev, m->rope_host.data(), m->rope_host.size() * sizeof(TlmRope), hipMemcpyHostToDevice));
    MMI_HIP_CHECK(m->scratch.alloc(&m->tok, T));
    MMI_HIP_CHECK(hipMemset(m->tok, 0, (size_t)T * sizeof(int)));
    MMI_HIP_CHECK(m->scratch.alloc(&m->last_tok, m->max_slots));
    MMI_HIP_CHECK(hipMemset(m->last_tok, 0, (size_t)m->max_slots * sizeof(int)));
    const size_t n_table = (size_t)m->max_slots * table_ld(m) + 1;
    MMI_HIP_CHECK(m->scratch.alloc(&m->block_table, n_table));
    MMI_HIP_CHECK(hipMemset(m->block_table, 0, n_table * sizeof(int)));
    if ((rc = alloc_f32(m, &m->logits, (size_t)m->max_slots * c.vocab))) return rc;
    m->samp_ld = round_up(c.vocab, 8);
    MMI_HIP_CHECK(m->scratch.alloc(&m->samp_rows, (size_t)m->max_slots * m->samp_ld));
    MMI_HIP_CHECK(m->scratch.alloc(&m->samp_map, 4 * (size_t)m->max_slots));
    MMI_HIP_CHECK(m->scratch.alloc(&m->samp_rng, 8));
    MMI_HIP_CHECK(m->scratch.alloc(&m->samp_zero, 1));
    MMI_HIP_CHECK(hipMemset(m->samp_zero, 0, sizeof(int)));
    // metadata: 6 ints per token + wanted rows, per-entry arrays, tile prefixes, segments, sequences and chunks, block-table updates
    m->meta_cap = 128 + (size_t)7 * T + 20 * (size_t)m->max_slots + 8 * ((size_t)T / TLM_CHUNK + m->max_slots + 1) + PREFIXES * m->geo.size() * ((size_t)m->max_slots + 1) + 8 * ((size_t)T / TLM_SEG + m->max_slots + 1) +
                  2 * ((size_t)T / TLM_PAGE + 2 * (size_t)m->max_slots + 2);
    MMI_HIP_CHECK(m->scratch.alloc(&m->meta, m->meta_cap));
    for (Staging& s : m->staging) {
        MMI_HIP_CHECK(hipHostMalloc((void**)&s.host, m->meta_cap * sizeof(int), 0));
        MMI_HIP_CHECK(hipEventCreateWithFlags(&s.ev, hipEventDisableTiming));
    }
    return MMI_OK;
}

int alloc_state(mmi_tlm* m) {
    for (Run& r : m->runs) {
        const Layer& L = m->layers[r.layer];
        if (L.c.mixer == MMI_TLM_MIX_MINGRU) {
            const size_t n = (size_t)m->max_slots * 2 * L.wp;
            MMI_HIP_CHECK(m->st.alloc(&r.state, n));
            MMI_HIP_CHECK(hipMemset(r.state, 0, n * sizeof(float)));
        } else if (L.linear()) {
            const size_t n = (size_t)m->max_slots * L.c.heads * L.dim_p * L.vdim_p, nc = (size_t)m->max_slots * 2 * std::max(1, L.c.conv - 1) * std::max(1, L.conv_c);
            MMI_HIP_CHECK(m->st.alloc(&r.state, n));
            MMI_HIP_CHECK(hipMemset(r.state, 0, n * sizeof(float)));
            if (L.conv_c) {
                MMI_HIP_CHECK(m->st.alloc(&r.conv, nc));
                MMI_HIP_CHECK(hipMemset(r.conv, 0, nc * sizeof(float)));
            }
        } else if (L.c.mixer == MMI_TLM_MIX_ATTENTION) {
            const size_t nk = (size_t)m->max_pages * L.c.kv_heads * 4 * L.k_ks * 64, nv = (size_t)m->max_pages * L.c.kv_heads * (TLM_PAGE / m->kstep) * L.nd * 64;
            u32x4 *k = nullptr, *v = nullptr;
            MMI_HIP_CHECK(m->st.alloc(&k, nk));
            MMI_HIP_CHECK(hipMemset(k, 0, nk * 16));      // (as below)
            MMI_HIP_CHECK(m->st.alloc(&v, nv));
            MMI_HIP_CHECK(hipMemset(v, 0, nv * 16));
            r.kc = k;
            r.vc = v;
        } else {
            const size_t nk = (size_t)m->max_pages * 4 * L.k_ks * 64;
            u32x4* k = nullptr;
            MMI_HIP_CHECK(m->st.alloc(&k, nk));
            MMI_HIP_CHECK(hipMemset(k, 0, nk * 16));      // masked keys of a block are multiplied by zero weights: never-written rows must be finite
            r.kc = k;
        }
    }
    return MMI_OK;
}

// ------------------------------------------------------------------------------------------------
// launch list
// ------------------------------------------------------------------------------------------------
struct Plan { bool rows; int mt, fm; };      // weight-streaming kernel with mt row tiles, or the tiled kernel with 32 fm rows per block
Plan plan_rows(int T) {
    Plan p{T <= ROWS_MAX, 1, 2};
    p.mt = T <= 16 ? 1 : (T <= 32 ? 2 : 4);
    p.fm = T >= 1024 ? 4 : 2;
    return p;
}
int plan_tile(const Plan& p) { return p.rows ? 16 * p.mt : 32 * p.fm; }

TlmJob base_job(const Mat& w, const void* x, int xks) {
    TlmJob j;
    memset(&j, 0, sizeof(j));
    j.wp = w.wp;
    j.wgs = w.gs;
    j.xp = (const u32x4*)x;
    j.xks = xks;
    j.KS = w.KS;
    j.NT = w.NT;
    j.groups = 1;
    j.ksplit = 1;
    j.in_mul = 1;
    j.out_mul = 1;
    j.scale = 1.f;
    return j;
}
TlmJob dense_job(const Mat& w, const void* x, int xks, int rows) {
    TlmJob j = base_job(w, x, xks);
    j.rows = rows;
    return j;
}
TlmJob routed_job(mmi_tlm* m, const Layer& L, const Mat& w, const void* x, int xks, int in_div, int T, const Plan& p) {
    TlmJob j = base_job(w, x, xks);
    j.list = m->list + (long)L.route * m->list_ld;
    j.tiles = m->tiles + (long)L.route * m->tile_ld * 3;
    j.n_tiles = m->n_tiles + L.route;
    j.in_div = in_div;
    const int pairs = T * L.c.top;
    j.rblocks = std::min(pairs, std::min(L.c.experts, pairs) + pairs / plan_tile(p));      // every expert's run ends in at most one partial tile
    return j;
}
int rows_ntw(const Plan& p);
// K split so that a product with few n-tiles still covers the chip; the consumer sums the fp32 partials
int split_for(const Plan& p, const Mat& w, int blocks) {
    if (!p.rows) return 1;
    int s = 1;
    while (s < MAX_SPLIT && blocks * s < 384 * rows_ntw(p) && w.KS / (2 * s) >= 8) s *= 2;
    return s;
}

int rows_ntw(const Plan& p) { return p.mt; }                // n-tiles per workgroup of the weight-streaming kernel
template <class Tr>
int launch_jobs_t(hipStream_t s, const Plan& p, TlmJobs& J) {
    // the tiled kernel takes 256 features at a time where that still covers the chip
    int fn = p.fm;
    for (int pass = 0; pass < 2; ++pass) {
        long total = 0;
        if (!p.rows && p.fm == 4 && pass == 0) fn = 8;
        for (int i = 0; i < J.n; ++i) {
            TlmJob& j = J.j[i];
            if (!j.list) j.rblocks = mmi_cdiv(j.rows, plan_tile(p));
            j.blocks = (p.rows ? mmi_cdiv(j.NT, rows_ntw(p)) : mmi_cdiv(j.NT, 2 * fn)) * (j.list ? 1 : j.groups) * j.ksplit * j.rblocks;
            total += j.blocks;
        }
        if (fn == 8 && total < 256) {
            fn = 4;
            continue;
        }
        const int grid = (int)total;
        if (p.rows) {
            if (p.mt == 1) MMI_LAUNCH((k_tlm_gemm_rows<Tr, 1, 1, 8, 4>), grid, 512, 0, s, J);
            else if (p.mt == 2) MMI_LAUNCH((k_tlm_gemm_rows<Tr, 2, 2, 8, 2>), grid, 512, 0, s, J);
            else MMI_LAUNCH((k_tlm_gemm_rows<Tr, 4, 4, 4, 2>), grid, 256, 0, s, J);
        } else if (fn == 8) {
            MMI_LAUNCH((k_tlm_gemm_tile<Tr, 8, 4, 1>), grid, 256, 0, s, J);
        } else if (p.fm == 4) {
            MMI_LAUNCH((k_tlm_gemm_tile<Tr, 4, 4, 2>), grid, 256, 0, s, J);
        } else {
            MMI_LAUNCH((k_tlm_gemm_tile<Tr, 2, 2, 2>), grid, 256, 0, s, J);
        }
        break;
    }
    MMI_CHECK_LAUNCH();
    return MMI_OK;
}
int launch_jobs(mmi_tlm* m, hipStream_t s, const Plan& p, TlmJobs J) {
    return m->f32 ? launch_jobs_t<TlmF32>(s, p, J) : launch_jobs_t<TlmBf16>(s, p, J);
}

// the instantiation for a layer's latent blocks and rotated k-steps
template <class Tr, class F>
int attn_dispatch(int nd, int rk, F f) {
    constexpr int R1 = 32 / Tr::KSTEP, R2 = 64 / Tr::KSTEP, R4 = 128 / Tr::KSTEP;
#define TLM_ND(ND_)                                                                                                  \
    if (nd <= ND_) {                                                                                                 \
        if (rk <= R1) return f(std::integral_constant<int, ND_>(), std::integral_constant<int, R1>());               \
        if (rk <= R2) return f(std::integral_constant<int, ND_>(), std::integral_constant<int, R2>());               \
        return f(std::integral_constant<int, ND_>(), std::integral_constant<int, R4>());                             \
    }
    TLM_ND(4) TLM_ND(8) TLM_ND(16) TLM_ND(32)
#undef TLM_ND
    return mmi_fail(MMI_ERR_UNSUPPORTED, "latent too wide");
}
int attn_group_tiles(int nd, bool f32) { return nd <= (f32 ? 8 : 16) ? 8 : 4; }      // column tiles a workgroup of k_tlm_attn_tile takes (TlmAttnTile::QT)

template <class Tr>
int launch_attn_t(hipStream_t s, const TlmAttnArgs& a, bool tiled) {
    const int rk = a.q_ks - a.out_ks;
    return attn_dispatch<Tr>(a.nd, rk, [&](auto nd, auto rks) {
        constexpr int ND = decltype(nd)::value, RK = decltype(rks)::value;
        if constexpr (Tr::V == 8 || ND <= 16) if (tiled) {
            constexpr size_t smem = TlmAttnTile<Tr, ND, RK>::smem();
            static_assert(smem <= 160 * 1024, "LDS of a CU");
            if (smem > 64 * 1024) {
                static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&k_tlm_attn_tile<Tr, ND, RK>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
                MMI_HIP_CHECK(attr);
            }
            MMI_LAUNCH((k_tlm_attn_tile<Tr, ND, RK>), a.n_tiles, 256, smem, s, a);
            MMI_CHECK_LAUNCH();
            return (int)MMI_OK;
        }
        MMI_LAUNCH((k_tlm_attn<Tr, ND, RK>), dim3(round_up(a.n_tiles, 8), a.nsplit), 256, 0, s, a);
        if (a.nsplit > 1) MMI_LAUNCH((k_tlm_attn_combine<Tr>), dim3(a.n_tiles, mmi_cdiv(a.nd, 8)), 256, 0, s, a);
        MMI_CHECK_LAUNCH();
        return (int)MMI_OK;
    });
}

template <class Tr, int D>
int launch_gqa_d(hipStream_t s, const TlmGqaArgs& a, bool tiled) {
    if (tiled) {
        constexpr size_t smem = TlmGqaTile<Tr, D>::smem();
        static_assert(smem <= 160 * 1024, "LDS of a CU");
        if (smem > 64 * 1024) {
            static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&k_tlm_gqa_tile<Tr, D>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
            MMI_HIP_CHECK(attr);
        }
        MMI_LAUNCH((k_tlm_gqa_tile<Tr, D>), dim3(a.n_tiles, a.kv_heads), 256, smem, s, a);
    } else {
        MMI_LAUNCH((k_tlm_gqa<Tr, D>), dim3(a.n_tiles, a.kv_heads, a.nsplit), 256, 0, s, a);
        if (a.nsplit > 1) MMI_LAUNCH((k_tlm_gqa_combine<Tr>), dim3(a.n_tiles, a.kv_heads, mmi_cdiv(a.nd, 4)), 256, 0, s, a);
    }
    MMI_CHECK_LAUNCH();
    return MMI_OK;
}
int gqa_bound(const Layer& L, int kstep) {               // the kernels' bound on both head sizes
    const int d = std::max(L.k_ks * kstep, L.nd * 16);
    return d <= 64 ? 64 : (d <= 128 ? 128 : 256);
}
template <class Tr>
int launch_gqa_t(hipStream_t s, const TlmGqaArgs& a, int bound, bool tiled) {
    if (bound == 64) return launch_gqa_d<Tr, 64>(s, a, tiled);
    if (bound == 128) return launch_gqa_d<Tr, 128>(s, a, tiled);
    return launch_gqa_d<Tr, 256>(s, a, tiled);
}

struct Carry {                    // what the next residual launch has to add
    const float* mix = nullptr; int mix_p = 1; const float* ls1 = nullptr;
    const float* dn = nullptr; int dn_p = 1, top = 1; const float* ls2 = nullptr;
    const float* vec = nullptr; bool replace = false;      // (mix is the whole new residual, plus vec)
};
struct Norms {                    // what it leaves behind: one or two normalised operands, or (raw) the residual itself as an operand
    const float* w = nullptr; void* out = nullptr;
    const float* w2 = nullptr; void* out2 = nullptr;
    void* raw = nullptr;
};

void add_resid(mmi_tlm* m, MmiProgram& P, const Shape& sh, const Carry& c, int emb_mode, float* tap, const Norms& o, const int* rows, int n) {
    TlmResidArgs a;
    memset(&a, 0, sizeof(a));
    a.x = m->x;
    a.width = m->cfg.width;
    a.ld = m->ld;
    a.mix = c.mix;
    a.mix_p = c.mix_p;
    a.mix_ps = (long)sh.T * m->ld;
    a.ls1 = c.ls1;
    a.dn = c.dn;
    a.dn_p = c.dn_p;
    a.top = c.top;
    a.dn_ps = (long)sh.T * c.top * m->ld;
    a.ls2 = c.ls2;
    a.replace = c.replace;
    a.vec = c.vec;
    a.emb.table = m->embed;
    a.emb.tok = m->tok;
    a.emb.scale = m->cfg.embed_scale;
    a.emb.bigram = m->bigram;
    a.emb.brow = m->brow;
    a.emb.pos = m->pos_emb;
    a.emb.at = m->meta + sh.m.pos;
    a.emb_mode = emb_mode;
    a.tap = tap;
    a.w = o.w;
    a.w2 = o.w2;
    a.out2 = o.out2;
    a.raw = o.raw;
    a.raw_ks = 2 * m->h_ks;
    if (emb_mode == TLM_EMB_SET) a.emb_out = m->cat;
    a.emb_k0 = m->h_ks * m->kstep;
    a.groups = m->cfg.norm_groups;
    a.eps = m->cfg.norm_eps;
    a.out = o.out;
    a.KS = m->h_ks;
    a.rows = rows;
    const int block = n <= 256 ? std::min(1024, std::max(256, round_up(m->ld / 4, 64))) : 256;     // few rows: one vector per thread
    const size_t smem = ((size_t)m->ld + 2 * (size_t)m->cfg.norm_groups + block / 64 + 8) * sizeof(float);
    const bool f32 = m->f32;
    P.add([=](hipStream_t s) {
        if (f32) MMI_LAUNCH((k_tlm_resid_norm<TlmF32>), n, block, smem, s, a);
        else MMI_LAUNCH((k_tlm_resid_norm<TlmBf16>), n, block, smem, s, a);
        MMI_CHECK_LAUNCH();
        return (int)MMI_OK;
    });
}
void add_jobs(mmi_tlm* m, MmiProgram& P, const Plan& p, const TlmJobs& J, long bytes) {
    P.add([=](hipStream_t s) { return launch_jobs(m, s, p, J); }, bytes);
}

// mixer cores: fill `first` with the product(s) that read the norm, queue everything up to the output projection's operand, and
// return the output projection
struct MixerOut { const Mat* w; const void* x; int xks; };

MixerOut build_mingru(mmi_tlm* m, MmiProgram& P, const Shape& sh, const Layer& L, const Run& r, TlmJobs first, const Plan& p, const std::string& site) {
    const int T = sh.T;
    TlmJob j = dense_job(L.zcg, m->h, m->h_ks, T);
    j.epi = TLM_EPI_GRU;
    j.out = m->zcg;
    j.out_ld = L.wp;
    j.bias = L.bias;
    first.j[first.n++] = j;
    P.site(site + "in");
    add_jobs(m, P, p, first, L.zcg.bytes());
    TlmScanArgs a;
    memset(&a, 0, sizeof(a));
    a.zcg = m->zcg;
    a.width = L.wp;
    a.seg = (const TlmSeg*)(m->meta + sh.m.seg);
    a.state = r.state;
    a.pair = m->pair;
    a.out = m->y;
    a.out_ks = L.out.KS;
    const bool f32 = m->f32, pairs = sh.pairs;
    const int n_seg = sh.n_seg, block = L.wp >= 256 ? 256 : 64;
    P.site(site + "scan");
    P.add([=](hipStream_t s) {
        const dim3 grid(mmi_cdiv(a.width, block), n_seg);
        if (pairs) MMI_LAUNCH(k_tlm_scan_pairs, grid, block, 0, s, a);
        if (f32) MMI_LAUNCH((k_tlm_scan<TlmF32>), grid, block, 0, s, a);
        else MMI_LAUNCH((k_tlm_scan<TlmBf16>), grid, block, 0, s, a);
        MMI_CHECK_LAUNCH();
        return (int)MMI_OK;
    });
    return MixerOut{&L.out, m->y, L.out.KS};
}

MixerOut build_latent_attention(mmi_tlm* m, MmiProgram& P, const Shape& sh, const Layer& L, const Run& r, TlmJobs first, const Plan& p, const std::string& site) {
    const int T = sh.T, H = L.c.heads;
    const bool f32 = m->f32;
    const int ld = L.qp + L.kvp + L.rp + L.hp;
    TlmJob j = dense_job(L.in, m->h, m->h_ks, T);
    j.epi = TLM_EPI_F32;
    j.out = m->lat;
    j.out_ld = ld;
    j.out_ps = (long)T * ld;
    j.ksplit = split_for(p, L.in, L.in.NT);
    const int in_p = j.ksplit;
    first.j[first.n++] = j;
    P.site(site + "in");
    add_jobs(m, P, p, first, L.in.bytes());

    TlmLatentArgs a;
    memset(&a, 0, sizeof(a));
    a.in = m->lat;
    a.in_p = in_p;
    a.in_ps = (long)T * ld;
    a.ld = ld;
    a.q_rank = L.c.q_rank;
    a.kv_rank = L.c.kv_rank;
    a.rot = L.c.rot_dim;
    a.heads = H;
    a.qp = L.qp;
    a.kvp = L.kvp;
    a.rp = L.rp;
    a.qw = L.qw;
    a.cw = L.cw;
    a.eps = m->cfg.norm_eps;
    const float* rope = L.rope >= 0 ? m->rope_host[L.rope].out : nullptr;
    const int rope_ld = L.rope >= 0 ? m->rope_host[L.rope].ld : 0;
    a.rope = rope;
    a.rope_ld = rope_ld;
    a.crow = m->meta + sh.m.crow;
    a.q = m->cq;
    a.q_ks = L.q_ks;
    a.kc = r.kc;
    a.k_ks = L.k_ks;
    a.rot_k0 = L.lat_ks * m->kstep;
    a.gate = m->gate;
    a.gate_ld = H;
    P.site(site + "latent");
    P.add([=](hipStream_t s) {
        if (f32) MMI_LAUNCH((k_tlm_latent<TlmF32>), T, 256, (size_t)ld * sizeof(float), s, a);
        else MMI_LAUNCH((k_tlm_latent<TlmBf16>), T, 256, (size_t)ld * sizeof(float), s, a);
        MMI_CHECK_LAUNCH();
        return (int)MMI_OK;
    });

    TlmJobs Q;
    memset(&Q, 0, sizeof(Q));
    TlmJob& jn = Q.j[Q.n++];
    jn = dense_job(L.uqn, m->cq, L.q_ks, T);
    jn.epi = TLM_EPI_PACK;
    jn.out = m->qn;
    jn.out_ld = L.qn_ks;
    if (L.rp) {
        TlmJob& jr = Q.j[Q.n++];
        jr = dense_job(L.uqr, m->cq, L.q_ks, T);
        jr.groups = H;
        jr.epi = TLM_EPI_ROPE;
        jr.out = m->q;
        jr.out_ld = L.k_ks;
        jr.out_mul = H;
        jr.out_gadd = 1;
        jr.out_k0 = L.lat_ks * m->kstep;
        jr.rope = rope;
        jr.rope_ld = rope_ld;
    }
    P.site(site + "q");
    add_jobs(m, P, p, Q, L.uqn.bytes() + H * L.uqr.bytes());

    memset(&Q, 0, sizeof(Q));
    TlmJob& jk = Q.j[Q.n++];
    jk = dense_job(L.uk, m->qn, L.qn_ks, T);
    jk.groups = H;
    jk.xkg = L.dim_p / m->kstep;
    jk.epi = TLM_EPI_PACK;
    jk.out = m->q;
    jk.out_ld = L.k_ks;
    jk.out_mul = H;
    jk.out_gadd = 1;
    P.site(site + "absorb");
    add_jobs(m, P, p, Q, H * L.uk.bytes());

    TlmAttnArgs t;
    memset(&t, 0, sizeof(t));
    t.q = m->q;
    t.kc = r.kc;
    t.out = m->ao;
    t.out_rows = round_up(T, 16);
    t.heads = H;
    t.q_ks = L.k_ks;
    t.nd = L.nd;
    t.out_ks = L.lat_ks;
    t.mask = TlmMask{L.c.window, 0, L.c.scale * 1.44269504088896340736f};
    t.n_entries = sh.n_entries;
    const bool wide = attn_group_tiles(L.nd, f32) == 8;
    const bool tiled = sh.groups[L.geo][wide] >= ATTN_TILE_GROUPS && !(f32 && L.nd > 16);     // fp32 with a wide latent: the operands do not fit the registers
    const int kind = tiled ? (wide ? 2 : 1) : 0;       // which of the three prefix arrays
    t.n_tiles = tiled ? sh.groups[L.geo][kind - 1] : sh.tiles[L.geo];
    t.nsplit = tiled ? 1 : std::max(1, std::min(sh.nsplit, (L.nd > 16 ? 256 : MAX_PARTIALS) / std::max(1, t.n_tiles)));     // (a wide latent: one workgroup per CU)
    t.tile0 = m->meta + sh.m.tile0 + (PREFIXES * L.geo + kind) * (sh.n_entries + 1);
    t.erow0 = m->meta + sh.m.erow0;
    t.elen = m->meta + sh.m.elen;
    t.epos0 = m->meta + sh.m.epos0;
    t.eslot = m->meta + sh.m.eslot;
    t.pages = TlmPages{m->block_table, table_ld(m), m->keep_pages};
    t.po = m->po;
    t.pml = m->pml;
    P.site(site + "attn");
    P.add([=](hipStream_t s) { return f32 ? launch_attn_t<TlmF32>(s, t, tiled) : launch_attn_t<TlmBf16>(s, t, tiled); });

    memset(&Q, 0, sizeof(Q));
    TlmJob& jv = Q.j[Q.n++];
    jv = dense_job(L.uv, m->ao, L.lat_ks, T);
    jv.groups = H;
    jv.in_gadd = t.out_rows;
    jv.epi = TLM_EPI_PACK;
    jv.out = m->o;
    jv.out_ld = L.out.KS;
    jv.out_kg = L.vdim_p;
    jv.gate = m->gate;
    jv.gate_ld = H;
    P.site(site + "value");
    add_jobs(m, P, p, Q, H * L.uv.bytes());
    return MixerOut{&L.out, m->o, L.out.KS};
}

MixerOut build_attention(mmi_tlm* m, MmiProgram& P, const Shape& sh, const Layer& L, const Run& r, TlmJobs first, const Plan& p, const std::string& site) {
    const int T = sh.T, H = L.c.heads, G = L.c.kv_heads;
    const bool f32 = m->f32;
    TlmJob j = dense_job(L.in, m->h, m->h_ks, T);
    j.epi = TLM_EPI_QKV;
    j.out = m->q;
    j.out_ld = L.k_ks;
    j.qkv = TlmQkv{r.kc, r.vc, m->meta + sh.m.crow, H * L.dim_p / 16, G * L.dim_p / 16, L.dim_p / 16, L.nd, H, G};
    first.j[first.n++] = j;
    P.site(site + "in");
    add_jobs(m, P, p, first, L.in.bytes());

    TlmGqaArgs t;
    memset(&t, 0, sizeof(t));
    t.q = m->q;
    t.kc = r.kc;
    t.vc = r.vc;
    t.out = m->o;
    t.out_ks = L.out.KS;
    t.heads = H;
    t.kv_heads = G;
    t.rep = H / G;
    t.q_ks = L.k_ks;
    t.nd = L.nd;
    t.mask = TlmMask{L.c.window, L.c.window > 0 ? L.c.keep_first : 0, L.c.scale * 1.44269504088896340736f};
    t.sink = L.c.sink;
    t.n_entries = sh.n_entries;
    const int bound = gqa_bound(L, m->kstep);
    const bool wide = !(f32 && bound == 256);            // columns per workgroup of k_tlm_gqa_tile (TlmGqaTile::QT)
    const std::array<int, 3>& sp = sh.split[L.geo];
    // long portions through the kernel that stages keys, short ones (single tokens) through the other, if there are enough of the former
    const bool tiled = sp[1 + wide] * G >= ATTN_TILE_GROUPS / 2;
    auto part = [&](TlmGqaArgs& x, int kind, int n, bool split) {
        x.tile0 = m->meta + sh.m.tile0 + (PREFIXES * L.geo + kind) * (sh.n_entries + 1);
        x.n_tiles = n;
        x.nsplit = split ? std::max(1, std::min(sh.nsplit, MAX_PARTIALS / std::max(1, n * G))) : 1;
    };
    t.erow0 = m->meta + sh.m.erow0;
    t.elen = m->meta + sh.m.elen;
    t.epos0 = m->meta + sh.m.epos0;
    t.eslot = m->meta + sh.m.eslot;
    t.pages = TlmPages{m->block_table, table_ld(m), m->keep_pages};
    t.po = m->po;
    t.pml = m->pml;
    auto launch = [&](const TlmGqaArgs& x, bool staged) {
        P.add([=](hipStream_t s) { return f32 ? launch_gqa_t<TlmF32>(s, x, bound, staged) : launch_gqa_t<TlmBf16>(s, x, bound, staged); });
    };
    P.site(site + "attn");
    if (tiled) {
        TlmGqaArgs u = t;
        part(u, wide ? 5 : 4, sp[1 + wide], false);
        launch(u, true);
        part(t, 3, sp[0], true);
    } else {
        part(t, 0, sh.tiles[L.geo], true);
    }
    if (t.n_tiles) launch(t, false);
    return MixerOut{&L.out, m->o, L.out.KS};
}

template <class Tr, bool DELTA>
int launch_state_step(hipStream_t s, const TlmLinArgs& a, int n) {
    const int cgp = tlm_step_groups(a.vdim_p);
    int block = 64;                                      // rows of S per thread: 4, in larger workgroups 8, at the largest sizes 16
    while (block < 256 && mmi_cdiv(a.dim_p, block / cgp) > 4) block *= 2;
    while (block < 512 && mmi_cdiv(a.dim_p, block / cgp) > 8) block *= 2;
    while (mmi_cdiv(a.dim_p, block / cgp) > 16) block *= 2;
    const int parts = block / cgp, rows = mmi_cdiv(a.dim_p, parts);
    const int rt = rows <= 4 && block <= 256 ? 4 : (rows <= 8 && block <= 512 ? 8 : 16);
    const size_t smem = (size_t)(3 * parts * rt + a.vdim_p + 2 * parts * a.vdim_p) * sizeof(float);
    if (rt == 4) MMI_LAUNCH((k_tlm_state_step<Tr, DELTA, 4, 256>), dim3(n, a.heads), block, smem, s, a, cgp);
    else if (rt == 8) MMI_LAUNCH((k_tlm_state_step<Tr, DELTA, 8, 512>), dim3(n, a.heads), block, smem, s, a, cgp);
    else MMI_LAUNCH((k_tlm_state_step<Tr, DELTA, 16, 1024>), dim3(n, a.heads), block, smem, s, a, cgp);
    MMI_CHECK_LAUNCH();
    return MMI_OK;
}
template <bool DELTA>
int launch_chunk_scan(hipStream_t s, const TlmLinArgs& a, int n_unit) {
    const int grid = 8 * mmi_cdiv(n_unit * a.heads, 8) * (a.vdim_p / 16), nd = a.dim_p / 16;
    if (nd <= 4) MMI_LAUNCH((k_tlm_chunk_scan<DELTA, 1>), grid, 256, 0, s, a, n_unit);
    else if (nd <= 8) MMI_LAUNCH((k_tlm_chunk_scan<DELTA, 2>), grid, 256, 0, s, a, n_unit);
    else MMI_LAUNCH((k_tlm_chunk_scan<DELTA, 4>), grid, 256, 0, s, a, n_unit);
    MMI_CHECK_LAUNCH();
    return MMI_OK;
}

// the mixers that carry a matrix per head (tlm_linear.h)
MixerOut build_linear(mmi_tlm* m, MmiProgram& P, const Shape& sh, const Layer& L, const Run& r, TlmJobs first, const Plan& p, const std::string& site) {
    const int T = sh.T, H = L.c.heads;
    const bool f32 = m->f32, delta = L.c.mixer == MMI_TLM_MIX_CHANNEL_DELTA;
    TlmJob j = dense_job(L.in, m->h, m->h_ks, T);
    j.epi = delta ? TLM_EPI_F32 : TLM_EPI_SILU;
    j.act_nt = L.b0 / 16;
    j.out = m->lin;
    j.out_ld = L.in_ld;
    first.j[first.n++] = j;
    const int lr_ks = L.lr.NT * 16 / m->kstep;
    if (delta) {
        j = dense_job(L.lr, m->h, m->h_ks, T);
        j.epi = TLM_EPI_PACK;
        j.out = m->lr;
        j.out_ld = lr_ks;
        first.j[first.n++] = j;
    }
    P.site(site + "in");
    add_jobs(m, P, p, first, L.in.bytes() + L.lr.bytes());

    TlmLinArgs a;
    memset(&a, 0, sizeof(a));
    a.in = m->lin;
    a.in_ld = L.in_ld;
    a.q0 = L.q0;
    a.k0 = L.k0;
    a.v0 = L.v0;
    a.b0 = L.b0;
    a.heads = H;
    a.kv_heads = delta ? L.c.kv_heads : H;
    a.dim = L.c.dim;
    a.vdim = L.c.vdim;
    a.dim_p = L.dim_p;
    a.vdim_p = L.vdim_p;
    a.q_scale = delta ? (float)(1.0 / sqrt((double)L.c.dim)) : 1.f;
    a.eps = m->cfg.norm_eps;
    a.conv_w = L.conv_w;
    a.conv_state = r.conv;
    a.conv_c = L.conv_c;
    a.taps = L.c.conv;
    a.decay = delta ? m->dec : L.decay;
    a.decay_c = L.decay;
    a.gate = delta ? m->lgate : m->lin + L.b0;
    a.gate_ld = delta ? H * L.vdim_p : L.in_ld;
    a.nw = L.nw;
    a.state = r.state;
    a.small = (const TlmUnit*)(m->meta + sh.m.small);
    a.unit = (const TlmUnit*)(m->meta + sh.m.unit);
    a.chunk = (const TlmSeg*)(m->meta + sh.m.chunk);
    a.qkv = m->qkv;
    a.w = m->cw;
    a.qg = m->cq_g;
    a.kt = m->ckt;
    a.u0 = m->cu0;
    a.p = m->cp;
    a.gend = m->cgend;
    a.o = m->lo;
    a.out = m->o;
    a.out_ks = L.out.KS;
    if (delta) {
        TlmJobs Q;
        memset(&Q, 0, sizeof(Q));
        TlmJob& ja = Q.j[Q.n++];
        ja = dense_job(L.a2, m->lr, lr_ks, T);
        ja.epi = TLM_EPI_F32;
        ja.out = m->dec;
        ja.out_ld = H * L.dim_p;
        TlmJob& jg = Q.j[Q.n++];
        jg = dense_job(L.g2, (const u32x4*)m->lr + (long)(L.ra / m->kstep) * 64, lr_ks, T);
        jg.epi = TLM_EPI_F32;
        jg.out = m->lgate;
        jg.out_ld = H * L.vdim_p;
        P.site(site + "lowrank");
        add_jobs(m, P, p, Q, L.a2.bytes() + L.g2.bytes());
    }
    const int n_small = sh.n_small, n_unit = sh.n_unit, n_chunk = sh.n_chunk;
    if (n_small) {
        P.site(site + "step");
        P.add([=](hipStream_t s) {
            if (f32) return delta ? launch_state_step<TlmF32, true>(s, a, n_small) : launch_state_step<TlmF32, false>(s, a, n_small);
            return delta ? launch_state_step<TlmBf16, true>(s, a, n_small) : launch_state_step<TlmBf16, false>(s, a, n_small);
        });
    }
    if (n_chunk) {
        if (delta) {
            P.site(site + "conv");
            P.add([=](hipStream_t s) {
                MMI_LAUNCH(k_tlm_conv, dim3(n_chunk, 2 * a.kv_heads + a.heads), 256, 0, s, a, tlm_step_groups(a.dim_p), tlm_step_groups(a.vdim_p));
                MMI_CHECK_LAUNCH();
                return (int)MMI_OK;
            });
        }
        P.site(site + "chunk");
        P.add([=](hipStream_t s) {
            if (delta) {
                const size_t smem = tlm_chunk_delta_smem();
                static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&k_tlm_chunk_delta), hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
                MMI_HIP_CHECK(attr);
                MMI_LAUNCH(k_tlm_chunk_delta, dim3(n_chunk, a.heads), 256, smem, s, a);
            } else {
                MMI_LAUNCH(k_tlm_chunk_lightning, dim3(n_chunk, a.heads), 256, 0, s, a);
            }
            MMI_CHECK_LAUNCH();
            return (int)MMI_OK;
        });
        P.site(site + "scan");
        P.add([=](hipStream_t s) { return delta ? launch_chunk_scan<true>(s, a, n_unit) : launch_chunk_scan<false>(s, a, n_unit); });
    }
    if (!delta || n_chunk) {                             // (the delta rule's norm is per head: single tokens have had theirs)
        const TlmSeg* chunk = delta ? a.chunk : nullptr;
        const int rows = delta ? n_chunk * TLM_CHUNK : T;
        P.site(site + "gate");
        P.add([=](hipStream_t s) {
            const size_t smem = (size_t)(a.heads + 4) * sizeof(float);
            if (f32) MMI_LAUNCH((k_tlm_gated_norm<TlmF32>), rows, 256, smem, s, a, delta ? 1 : 0, chunk);
            else MMI_LAUNCH((k_tlm_gated_norm<TlmBf16>), rows, 256, smem, s, a, delta ? 1 : 0, chunk);
            MMI_CHECK_LAUNCH();
            return (int)MMI_OK;
        });
    }
    return MixerOut{&L.out, m->o, L.out.KS};
}

const char* mixer_site(int mixer) {
    switch (mixer) {
        case MMI_TLM_MIX_MINGRU: return "gru.";
        case MMI_TLM_MIX_LATENT_ATTENTION: return "mla.";
        case MMI_TLM_MIX_ATTENTION: return "gqa.";
        case MMI_TLM_MIX_CHANNEL_DELTA: return "delta.";
        default: return "light.";
    }
}

void build_program(mmi_tlm* m, MmiProgram& P, const Shape& sh) {
    const int T = sh.T;
    const Plan p = plan_rows(T);
    TlmPrepArgs a;
    memset(&a, 0, sizeof(a));
    a.T = T;
    a.n_ropes = (int)m->rope_host.size();
    a.n_updates = m->meta;
    a.htok = m->meta + sh.m.htok;
    a.pos = m->meta + sh.m.pos;
    a.rslot = m->meta + sh.m.rslot;
    a.last_tok = m->last_tok;
    a.tok = m->tok;
    a.updates = m->meta + sh.m.upd;
    a.block_table = m->block_table;
    a.rope = m->rope_dev;
    a.buckets = m->cfg.bigram_buckets;
    a.mul_prev = (long)m->cfg.bigram_mul_prev;
    a.mul_cur = (long)m->cfg.bigram_mul_cur;
    a.prev = m->meta + sh.m.prev;
    a.next = m->meta + sh.m.next;
    a.prev_tok = m->prev_tok;
    a.brow = m->brow;
    P.site("prepare");
    P.add([=](hipStream_t s) {
        MMI_LAUNCH(k_tlm_prepare, std::min(512, mmi_cdiv(T * 16, 256) + 1), 256, 0, s, a);
        MMI_CHECK_LAUNCH();
        return (int)MMI_OK;
    });
    if (!m->route_host.empty()) {
        TlmRouteArgs ra;
        memset(&ra, 0, sizeof(ra));
        ra.layers = m->route_dev;
        ra.tok = m->tok;
        ra.T = T;
        ra.tile = plan_tile(p);
        ra.list = m->list;
        ra.list_ld = m->list_ld;
        ra.tiles = m->tiles;
        ra.tile_ld = m->tile_ld;
        ra.n_tiles = m->n_tiles;
        const int nl = (int)m->route_host.size(), block = T * m->max_top <= 256 ? 256 : 1024;
        const size_t smem = (size_t)2 * m->max_experts * sizeof(unsigned);
        P.site("route");
        P.add([=](hipStream_t s) {
            MMI_LAUNCH(k_tlm_route, nl, block, smem, s, ra);
            MMI_CHECK_LAUNCH();
            return (int)MMI_OK;
        });
    }
    Carry c;
    const size_t tap_ld = (size_t)T * m->ld;
    for (size_t i = 0; i < m->runs.size(); ++i) {
        const Run& r = m->runs[i];
        const Layer& L = m->layers[r.layer];
        const std::string site = mixer_site(L.c.mixer);
        int emb = i == 0 ? TLM_EMB_SET : (r.add_emb ? TLM_EMB_ADD : TLM_EMB_NONE);
        float* tap = sh.taps && i ? sh.taps + (i - 1) * tap_ld : nullptr;
        if (r.pass >= 0) {                               // x <- loop.in [x; embedding] + loop.step[pass]
            P.site("loop.x");
            Norms raw;
            raw.raw = m->cat;
            add_resid(m, P, sh, c, emb, tap, raw, nullptr, T);
            TlmJobs J;
            memset(&J, 0, sizeof(J));
            TlmJob& j = J.j[J.n++];
            j = dense_job(m->loop_in, m->cat, 2 * m->h_ks, T);
            j.ksplit = split_for(p, m->loop_in, j.NT);
            j.epi = TLM_EPI_F32;
            j.out = m->mix;
            j.out_ld = m->ld;
            j.out_ps = (long)T * m->ld;
            c = Carry();
            c.mix = m->mix;
            c.mix_p = j.ksplit;
            c.replace = true;
            c.vec = m->loop_step + (size_t)r.pass * m->ld;
            P.site("loop.in");
            add_jobs(m, P, p, J, m->loop_in.bytes());
            emb = TLM_EMB_NONE;
            tap = nullptr;
        }
        const bool moe = L.c.mlp == MMI_TLM_MLP_MOE, dense = L.c.mlp == MMI_TLM_MLP_DENSE;
        Norms nm;
        nm.w = L.norm;
        nm.out = m->h;
        void* hf = m->h;                                 // what the feed-forward reads
        if (L.norm2) {
            nm.w2 = L.norm2;
            nm.out2 = hf = m->h2;
        }
        P.site(site + "norm");
        add_resid(m, P, sh, c, emb, tap, nm, nullptr, T);
        TlmJobs first;
        memset(&first, 0, sizeof(first));
        if (moe) {
            TlmJob& j = first.j[first.n++];
            j = routed_job(m, L, L.up, hf, m->h_ks, L.c.top, T, p);
            j.epi = TLM_EPI_PACK;
            j.act = TLM_ACT_RELU2;
            j.out = m->hid;
            j.out_ld = L.down.KS;
        } else if (dense) {
            TlmJob& j = first.j[first.n++];
            j = dense_job(L.up, hf, m->h_ks, T);
            j.epi = TLM_EPI_GLU;
            j.scale = L.c.limit;
            j.out = m->hid;
            j.out_ld = L.down.KS;
        }
        MixerOut mo;
        if (L.c.mixer == MMI_TLM_MIX_MINGRU) mo = build_mingru(m, P, sh, L, r, first, p, site);
        else if (L.c.mixer == MMI_TLM_MIX_LATENT_ATTENTION) mo = build_latent_attention(m, P, sh, L, r, first, p, site);
        else if (L.c.mixer == MMI_TLM_MIX_ATTENTION) mo = build_attention(m, P, sh, L, r, first, p, site);
        else mo = build_linear(m, P, sh, L, r, first, p, site);
        TlmJobs J;
        memset(&J, 0, sizeof(J));
        c = Carry();
        if (moe || dense) {
            TlmJob& j = J.j[J.n++];
            c.top = moe ? L.c.top : 1;
            j = moe ? routed_job(m, L, L.down, m->hid, L.down.KS, 1, T, p) : dense_job(L.down, m->hid, L.down.KS, T);
            j.ksplit = split_for(p, L.down, j.NT * (moe ? j.rblocks : 1));
            j.epi = TLM_EPI_F32;
            j.out = m->dn;
            j.out_ld = m->ld;
            j.out_ps = (long)T * c.top * m->ld;
            c.dn = m->dn;
            c.dn_p = j.ksplit;
            c.ls2 = L.ls2;
        }
        TlmJob& j = J.j[J.n++];
        j = dense_job(*mo.w, mo.x, mo.xks, T);
        j.ksplit = split_for(p, *mo.w, j.NT);
        j.epi = TLM_EPI_F32;
        j.out = m->mix;
        j.out_ld = m->ld;
        j.out_ps = (long)T * m->ld;
        c.mix = m->mix;
        c.mix_p = j.ksplit;
        c.ls1 = L.ls1;
        P.site(site + "out");
        add_jobs(m, P, p, J, mo.w->bytes() + (dense ? L.down.bytes() : 0));
    }
    if (sh.taps) {
        P.site("taps");
        add_resid(m, P, sh, c, TLM_EMB_NONE, sh.taps + (m->runs.size() - 1) * tap_ld, Norms(), nullptr, T);
        c = Carry();                                                     // (the residual has been written back)
    }
    if (sh.n_want > 0) {
        P.site("final_norm");
        Norms nm;
        nm.w = m->final_norm;
        nm.out = m->h;
        add_resid(m, P, sh, c, TLM_EMB_NONE, nullptr, nm, m->meta + sh.m.want, sh.n_want);
        const Plan hp = plan_rows(sh.n_want);
        TlmJobs J;
        memset(&J, 0, sizeof(J));
        TlmJob& j = J.j[J.n++];
        j = dense_job(m->head, m->h, m->h_ks, sh.n_want);
        j.epi = TLM_EPI_LOGITS;
        j.out = sh.logits;
        j.out_ld = m->cfg.vocab;
        j.n_valid = m->cfg.vocab;
        j.scale = m->cfg.logit_scale;
        P.site("head");
        add_jobs(m, P, hp, J, m->head.bytes());
    }
}

// ------------------------------------------------------------------------------------------------
// cache manager
// ------------------------------------------------------------------------------------------------
int64_t pages_for(const mmi_tlm* m, const Slot* s, int64_t n) {
    if (!m->has_attn) return 0;
    const int64_t pos = s ? s->pos : 0;
    const int64_t have = s ? s->first_page + (int64_t)s->pages.size() : 0;
    return std::max<int64_t>(0, (pos + n + TLM_PAGE - 1) / TLM_PAGE - have);
}
void release_behind_window(mmi_tlm* m, Slot& s) {
    if (!m->has_attn || m->max_window <= 0) return;
    const int64_t first_seen = s.pos - m->max_window + 1;               // the oldest position the next token can see
    while (!s.pages.empty() && (s.first_page + 1) * TLM_PAGE <= first_seen) {
        if (s.first_page < m->keep_pages) s.kept.push_back(s.pages.front());
        else m->free_pages.push_back(s.pages.front());
        s.pages.erase(s.pages.begin());
        ++s.first_page;
    }
}
void release_slot(mmi_tlm* m, Slot& s) {
    for (int p : s.kept) m->free_pages.push_back(p);
    for (int p : s.pages) m->free_pages.push_back(p);
    s = Slot();
}

void destroy(mmi_tlm* m) {
    hipDeviceSynchronize();
    for (auto& p : m->progs) p.second->clear();
    for (Staging& s : m->staging) {
        if (s.host) hipHostFree(s.host);
        if (s.ev) hipEventDestroy(s.ev);
    }
    if (m->cap_stream) hipStreamDestroy(m->cap_stream);
    m->wts.release();
    m->st.release();
    m->scratch.release();
    delete m;
}

int create_impl(mmi_tlm* m, const mmi_tensor_desc* weights, int n_weights) {
    const mmi_tlm_cfg& c = m->cfg;
    MMI_HIP_CHECK(hipGetDevice(&m->device));
    m->f32 = c.dtype == MMI_F32;
    m->kstep = m->f32 ? TlmF32::KSTEP : TlmBf16::KSTEP;
    m->V = m->f32 ? TlmF32::V : TlmBf16::V;
    m->ld = round_up(c.width, 16);
    m->h_ks = round_up(c.width, m->kstep) / m->kstep;
    Loader ld;
    ld.m = m;
    ld.W = MmiWeights{weights, n_weights};
    int rc;
    if ((rc = ld.table("embed", c.vocab, c.width, &m->embed)) || (c.bigram_buckets > 0 && (rc = ld.table("bigram", (int64_t)c.bigram_buckets + 1, c.width, &m->bigram))) ||
        (c.max_positions > 0 && (rc = ld.table("pos", c.max_positions, c.width, &m->pos_emb))) || (rc = ld.vec("final.norm", c.width, m->ld, &m->final_norm)) ||
        (rc = ld.linear(c.tied_head ? "embed" : "head", c.vocab, c.width, &m->head)))
        return rc;
    const bool project = c.loop_inject == MMI_TLM_LOOP_PROJECT && c.loop_stop > c.loop_start;
    if (project) {
        const mmi_tensor_desc* d;
        const int rows = m->ld, half = m->h_ks * m->kstep;      // columns of x, then of the embedding, each padded to whole k-steps
        std::vector<int> rm(rows, -1), cm(2 * half, -1);
        for (int i = 0; i < c.width; ++i) {
            rm[i] = cm[i] = i;
            cm[half + i] = c.width + i;
        }
        if ((rc = ld.find("loop.in", MMI_BF16, {c.width, 2 * (int64_t)c.width}, &d)) || (rc = ld.alloc(&m->loop_in, 1, rows / 16, 2 * m->h_ks)) || (rc = ld.upload(rm, cm)) ||
            (rc = ld.pack(d, m->loop_in.wp, rows, 2 * half, 2 * c.width, 1)))
            return rc;
        std::vector<float> v, vp((size_t)c.loop_times * m->ld, 0.f);
        if ((rc = ld.host("loop.step", {c.loop_times, c.width}, &v))) return rc;
        for (int t = 0; t < c.loop_times; ++t)
            for (int i = 0; i < c.width; ++i) vp[(size_t)t * m->ld + i] = v[(size_t)t * c.width + i];
        if ((rc = ld.to_device(vp, &m->loop_step))) return rc;
    }
    int keep = 0;
    bool unlimited = false;
    for (int i = 0; i < c.n_layers; ++i) {
        m->layers.emplace_back();
        Layer& L = m->layers.back();
        L.c = c.layers[i];
        const std::string p = "l" + std::to_string(i);
        if ((rc = ld.vec(p + ".norm1", c.width, m->ld, &L.norm)) || (c.norms == 2 && L.c.mlp != MMI_TLM_MLP_NONE && (rc = ld.vec(p + ".norm2", c.width, m->ld, &L.norm2))) ||
            (c.layer_scales && (rc = ld.vec(p + ".ls1", c.width, m->ld, &L.ls1))))
            return rc;
        auto cached = [&](int columns, int window) {     // a layer with a paged cache, `columns` attention columns per token
            m->has_attn = true;
            if (window <= 0) unlimited = true;
            m->max_window = std::max<int64_t>(m->max_window, window);
            L.geo = (int)(std::find(m->geo.begin(), m->geo.end(), columns) - m->geo.begin());
            if (L.geo == (int)m->geo.size()) m->geo.push_back(columns);
        };
        if (L.c.mixer == MMI_TLM_MIX_MINGRU) {
            m->has_gru = true;
            if ((rc = load_mingru(ld, L, p))) return rc;
        } else if (L.c.mixer == MMI_TLM_MIX_ATTENTION) {
            cached(L.c.heads / L.c.kv_heads, L.c.window);
            if (L.c.window > 0) keep = std::max(keep, L.c.keep_first);
            if ((rc = load_attention(ld, L, p))) return rc;
        } else if (L.linear()) {
            m->has_linear = true;
            if ((rc = L.c.mixer == MMI_TLM_MIX_CHANNEL_DELTA ? load_channel_delta(ld, L, p) : load_lightning(ld, L, p))) return rc;
        } else {
            m->has_latent = true;
            cached(L.c.heads, L.c.window);
            if ((rc = load_latent_attention(ld, L, p))) return rc;
            if (L.c.rot_dim > 0) {
                const std::pair<double, int> key(L.c.rot_base, L.c.rot_dim);
                L.rope = (int)(std::find(m->ropes.begin(), m->ropes.end(), key) - m->ropes.begin());
                if (L.rope == (int)m->ropes.size()) {
                    m->ropes.push_back(key);
                    const int half = L.c.rot_dim / 2;
                    std::vector<float> f(half);
                    for (int k = 0; k < half; ++k) f[k] = (float)pow(L.c.rot_base, -2.0 * k / L.c.rot_dim);
                    float* dev = nullptr;
                    MMI_HIP_CHECK(m->wts.alloc(&dev, half));
                    MMI_HIP_CHECK(hipMemcpy(dev, f.data(), half * sizeof(float), hipMemcpyHostToDevice));
                    m->rope_host.push_back(TlmRope{dev, half, L.rp / 2, nullptr});
                }
            }
        }
        if (L.c.mlp != MMI_TLM_MLP_NONE) {
            if ((c.layer_scales && (rc = ld.vec(p + ".ls2", c.width, m->ld, &L.ls2))) ||
                (rc = L.c.mlp == MMI_TLM_MLP_MOE ? load_moe(ld, L, p) : load_dense_glu(ld, L, p)))
                return rc;
        }
    }
    if (unlimited) m->max_window = 0;
    if (m->max_window > 0) m->keep_pages = mmi_cdiv(keep, TLM_PAGE);
    const int times = c.loop_stop > c.loop_start ? c.loop_times : 1;
    const int start = c.loop_stop > c.loop_start ? c.loop_start : c.n_layers, stop = c.loop_stop > c.loop_start ? c.loop_stop : c.n_layers;
    auto run = [&](int layer, bool add, int pass) {
        Run r;
        r.layer = layer;
        r.add_emb = add;
        r.pass = pass;
        m->runs.push_back(r);
    };
    for (int i = 0; i < start; ++i) run(i, false, -1);
    for (int t = 0; t < times; ++t)
        for (int i = start; i < stop; ++i) run(i, !project && t > 0 && i == start, project && i == start ? t : -1);
    for (int i = stop; i < c.n_layers; ++i) run(i, false, -1);
    m->slots.resize(m->max_slots);
    for (int i = m->max_pages - 1; i >= 0; --i) m->free_pages.push_back(i);
    if ((rc = alloc_state(m)) || (rc = alloc_buffers(m))) return rc;
    m->graphs = mmi_graphs_enabled();
    if (m->graphs) MMI_HIP_CHECK(hipStreamCreateWithFlags(&m->cap_stream, hipStreamNonBlocking));
    MMI_HIP_CHECK(hipDeviceSynchronize());
    return MMI_OK;
}

}  // namespace

extern "C" int mmi_tlm_create(const mmi_tlm_cfg* cfg, const mmi_tensor_desc* weights, int32_t n_weights, int32_t max_slots, int64_t max_tokens,
                              int32_t max_step_tokens, mmi_tlm** out) {
    if (!cfg || !weights || !out || max_slots < 1 || max_slots > 4096 || max_tokens < 1 || max_step_tokens < 1)
        return mmi_fail(MMI_ERR_INVALID, "mmi_tlm_create: bad arguments");
    int rc = check_cfg(*cfg);
    if (rc) return rc;
    mmi_tlm* m = new mmi_tlm();
    m->cfg = *cfg;
    m->max_slots = max_slots;
    m->max_pages = (int)mmi_cdiv64(max_tokens, TLM_PAGE);
    m->max_T = max_step_tokens;
    rc = create_impl(m, weights, n_weights);
    m->cfg.layers = nullptr;                         // the caller's array; the engine keeps its own copies
    if (rc) {
        destroy(m);
        return rc;
    }
    *out = m;
    return MMI_OK;
}

extern "C" void mmi_tlm_destroy(mmi_tlm* m) {
    if (!m) return;
    MmiDeviceGuard g(m->device);
    destroy(m);
}

extern "C" int mmi_tlm_open(mmi_tlm* m, int32_t* slot) {
    if (!m || !slot) return mmi_fail(MMI_ERR_INVALID, "mmi_tlm_open: null argument");
    for (size_t i = 0; i < m->slots.size(); ++i)
        if (!m->slots[i].live) {
            m->slots[i] = Slot();
            m->slots[i].live = true;
            *slot = (int32_t)i;
            return MMI_OK;
        }
    return mmi_fail(MMI_ERR_BUSY, "every sequence slot is taken");
}

extern "C" int mmi_tlm_close(mmi_tlm* m, int32_t slot) {
    if (!m || slot < 0 || slot >= m->max_slots || !m->slots[slot].live) return mmi_fail(MMI_ERR_NO_CHANNEL, "no open sequence in this slot");
    release_slot(m, m->slots[slot]);
    return MMI_OK;
}

extern "C" int64_t mmi_tlm_pages_needed(const mmi_tlm* m, int32_t slot, int64_t n) {
    if (!m || slot >= m->max_slots) return -1;
    return pages_for(m, slot < 0 ? nullptr : &m->slots[slot], n);
}

extern "C" int64_t mmi_tlm_info(const mmi_tlm* m, int32_t which, int32_t slot) {
    if (!m) return -1;
    const bool ok = slot >= 0 && slot < m->max_slots && m->slots[slot].live;
    switch (which) {
        case MMI_TLM_PAGE_TOKENS: return TLM_PAGE;
        case MMI_TLM_TOTAL_PAGES: return m->max_pages;
        case MMI_TLM_FREE_PAGES: return (int64_t)m->free_pages.size();
        case MMI_TLM_FREE_SLOTS: {
            int64_t n = 0;
            for (const Slot& s : m->slots) n += !s.live;
            return n;
        }
        case MMI_TLM_POSITION: return ok ? m->slots[slot].pos : -1;
        case MMI_TLM_HELD_PAGES: return ok ? (int64_t)(m->slots[slot].pages.size() + m->slots[slot].kept.size()) : -1;
        case MMI_TLM_WEIGHT_BYTES: return m->weight_bytes;
        case MMI_TLM_LAYER_RUNS: return (int64_t)m->runs.size();
        case MMI_TLM_GRAPHS: return (int64_t)m->progs.size();
    }
    return -1;
}

extern "C" int mmi_tlm_set_taps(mmi_tlm* m, float* taps) {
    if (!m) return mmi_fail(MMI_ERR_INVALID, "mmi_tlm_set_taps: null handle");
    if (taps && m->cfg.width != m->ld) return mmi_fail(MMI_ERR_UNSUPPORTED, "taps need a width that is a multiple of 16");
    m->taps = taps;
    return MMI_OK;
}

extern "C" int64_t mmi_tlm_launch_list(const mmi_tlm* m, char* buf, int64_t cap) { return m ? mmi_copy_launch_log(m->last_log, buf, cap) : -1; }

extern "C" int mmi_tlm_step(mmi_tlm* m, int32_t n_entries, const int32_t* slots, const int32_t* counts, const int32_t* tokens, int32_t n_want,
                            const int32_t* want, float* logits, mmi_stream stream) {
    if (!m || n_entries < 0 || n_want < 0 || (n_entries && (!slots || !counts || !tokens)) || (n_want && (!want || !logits)))
        return mmi_fail(MMI_ERR_INVALID, "mmi_tlm_step: bad arguments");
    if (n_entries == 0) return MMI_OK;
    MmiDeviceGuard guard(m->device);
    hipStream_t s = (hipStream_t)stream;
    // ---- validate, nothing changed yet
    if (n_entries > m->max_slots) return mmi_fail(MMI_ERR_SHAPE, "more entries than slots");
    std::vector<char> seen(m->max_slots, 0);
    int64_t T64 = 0, need = 0;
    for (int e = 0; e < n_entries; ++e) {
        if (slots[e] < 0 || slots[e] >= m->max_slots || !m->slots[slots[e]].live) return mmi_fail(MMI_ERR_NO_CHANNEL, "no open sequence in this slot");
        if (seen[slots[e]]++) return mmi_fail(MMI_ERR_INVALID, "a slot appears twice in one step");
        if (counts[e] < 1) return mmi_fail(MMI_ERR_INVALID, "an entry brings no token");
        T64 += counts[e];
        if (m->slots[slots[e]].pos + counts[e] > (int64_t)1 << 24) return mmi_fail(MMI_ERR_SHAPE, "position above 2^24");
        if (m->cfg.max_positions > 0 && m->slots[slots[e]].pos + counts[e] > m->cfg.max_positions) return mmi_fail(MMI_ERR_SHAPE, "position past the model's last");
        need += pages_for(m, &m->slots[slots[e]], counts[e]);
    }
    if (T64 > m->max_T) return mmi_fail(MMI_ERR_SHAPE, "the step brings more tokens than max_step_tokens");
    const int T = (int)T64;
    for (int i = 0; i < T; ++i)
        if (tokens[i] < -1 || tokens[i] >= m->cfg.vocab) return mmi_fail(MMI_ERR_INVALID, "token outside the vocabulary");
    for (int i = 0; i < n_want; ++i)
        if (want[i] < 0 || want[i] >= T || (i && want[i] <= want[i - 1])) return mmi_fail(MMI_ERR_INVALID, "wanted rows must ascend within the step");
    if (need > (int64_t)m->free_pages.size()) return mmi_fail(MMI_ERR_BUSY, "the cache pool has too few free pages");

    // ---- metadata block
    Shape sh;
    sh.T = T;
    sh.n_want = n_want;
    sh.n_entries = n_entries;
    for (int e = 0; e < n_entries; ++e) {
        const int n = mmi_cdiv(counts[e], TLM_SEG);
        sh.n_seg += n;
        sh.pairs |= n > 1;
        if (counts[e] <= TLM_SMALL) ++sh.n_small;
        else {
            ++sh.n_unit;
            sh.n_chunk += mmi_cdiv(counts[e], TLM_CHUNK);
        }
    }
    Meta& M = sh.m;
    int at = 16;
    auto take = [&](int n) {
        const int o = at;
        at += round_up(n, 4);
        return o;
    };
    M.htok = take(T);
    M.pos = take(T);
    M.rslot = take(T);
    M.crow = take(T);
    M.prev = take(T);
    M.next = take(T);
    M.want = take(n_want);
    M.erow0 = take(n_entries);
    M.elen = take(n_entries);
    M.epos0 = take(n_entries);
    M.eslot = take(n_entries);
    M.tile0 = take(PREFIXES * (int)m->geo.size() * (n_entries + 1));
    M.seg = take(8 * sh.n_seg);
    M.small = take(8 * sh.n_small);
    M.unit = take(8 * sh.n_unit);
    M.chunk = take(8 * sh.n_chunk);
    M.upd = at;
    M.total = at + 2 * (int)need;
    if ((size_t)M.total > m->meta_cap) return mmi_fail(MMI_ERR_SHAPE, "step metadata above its buffer");
    Staging& st = m->staging[m->stage_at];
    m->stage_at = (m->stage_at + 1) & 3;
    if (st.used) MMI_HIP_CHECK(hipEventSynchronize(st.ev));
    int* b = st.host;
    memset(b, 0, 16 * sizeof(int));
    int upd = 0, row = 0, seg = 0;
    int64_t blocks = 0;
    TlmSeg *sg = (TlmSeg*)(b + M.seg), *ck = (TlmSeg*)(b + M.chunk);
    TlmUnit *small = (TlmUnit*)(b + M.small), *unit = (TlmUnit*)(b + M.unit);
    int n_ck = 0;
    sh.tiles.assign(m->geo.size(), 0);
    sh.groups.assign(m->geo.size(), {0, 0});
    sh.split.assign(m->geo.size(), {0, 0, 0});
    for (int e = 0; e < n_entries; ++e) {
        Slot& S = m->slots[slots[e]];
        for (int64_t n = pages_for(m, &S, counts[e]); n > 0; --n) {
            const int page = m->free_pages.back();
            m->free_pages.pop_back();
            const int64_t at_page = S.first_page + (int64_t)S.pages.size();
            const int64_t idx = (int64_t)slots[e] * table_ld(m) + (at_page < m->keep_pages ? at_page : m->keep_pages + (at_page - m->keep_pages) % std::max(1, m->max_pages));
            S.pages.push_back(page);
            b[M.upd + 2 * upd] = (int)idx;
            b[M.upd + 2 * upd + 1] = page;
            ++upd;
        }
        b[M.erow0 + e] = row;
        b[M.elen + e] = counts[e];
        b[M.epos0 + e] = (int)S.pos;
        b[M.eslot + e] = slots[e];
        for (size_t g = 0; g < m->geo.size(); ++g) {
            int* t = b + M.tile0 + PREFIXES * (int)g * (n_entries + 1) + e;
            const int n = mmi_cdiv(counts[e] * m->geo[g], 16);
            t[0] = sh.tiles[g];
            t[n_entries + 1] = sh.groups[g][0];
            t[2 * (n_entries + 1)] = sh.groups[g][1];
            sh.tiles[g] += n;
            sh.groups[g][0] += mmi_cdiv(n, 4);
            sh.groups[g][1] += mmi_cdiv(n, 8);
            std::array<int, 3>& sp = sh.split[g];
            for (int k = 0; k < 3; ++k) t[(3 + k) * (n_entries + 1)] = sp[k];
            if (n <= 4) sp[0] += n;
            else {
                sp[1] += mmi_cdiv(n, 4);
                sp[2] += mmi_cdiv(n, 8);
            }
        }
        for (int o = 0, k = 0; o < counts[e]; o += TLM_SEG, ++k) {
            const int n = std::min(TLM_SEG, counts[e] - o);
            sg[seg++] = TlmSeg{row + o, n, slots[e], S.par, k, o + n == counts[e] ? 1 : 0, S.pos == 0 ? 1 : 0, 0};
        }
        if (counts[e] <= TLM_SMALL) {
            *small++ = TlmUnit{row, counts[e], slots[e], S.par, S.pos == 0 ? 1 : 0, 0, 0, 0};
        } else {
            *unit++ = TlmUnit{row, counts[e], slots[e], S.par, S.pos == 0 ? 1 : 0, n_ck, mmi_cdiv(counts[e], TLM_CHUNK), 0};
            for (int o = 0, k = 0; o < counts[e]; o += TLM_CHUNK, ++k) {
                const int n = std::min(TLM_CHUNK, counts[e] - o);
                ck[n_ck++] = TlmSeg{row + o, n, slots[e], S.par, k, o + n == counts[e] ? 1 : 0, S.pos == 0 ? 1 : 0, 0};
            }
        }
        for (int i = 0; i < counts[e]; ++i, ++row) {
            const int64_t pos = S.pos + i;
            b[M.prev + row] = pos == 0 ? -1 : (i > 0 ? -2 : slots[e] * 2 + S.par);
            b[M.next + row] = i + 1 == counts[e] ? slots[e] * 2 + (S.par ^ 1) : -1;
            b[M.htok + row] = tokens[row];
            b[M.pos + row] = (int)pos;
            b[M.rslot + row] = slots[e];
            b[M.crow + row] = m->has_attn ? S.page(pos / TLM_PAGE) * TLM_PAGE + (int)(pos % TLM_PAGE) : 0;
        }
        int64_t span = S.pos + counts[e];
        if (m->max_window > 0) span = std::min<int64_t>(span, m->max_window + counts[e] + m->keep_pages * TLM_PAGE);
        blocks = std::max(blocks, span / 32 + 1);
        S.pos += counts[e];
        S.par ^= 1;
    }
    for (int i = 0; i < n_want; ++i) b[M.want + i] = want[i];
    b[0] = upd;
    // few column tiles and long contexts: split the keys over workgroups, at least 4 blocks of 32 keys each
    int tiles_max = 1;
    for (int t : sh.tiles) tiles_max = std::max(tiles_max, t);
    while (sh.nsplit < MAX_KEY_SPLIT && tiles_max * sh.nsplit * 2 <= MAX_PARTIALS && blocks / (sh.nsplit * 2) >= 4) sh.nsplit *= 2;
    MMI_HIP_CHECK(hipMemcpyAsync(m->meta, b, (size_t)M.total * sizeof(int), hipMemcpyHostToDevice, s));
    MMI_HIP_CHECK(hipEventRecord(st.ev, s));
    st.used = true;

    // ---- launches
    int rc = MMI_OK;
    sh.taps = m->taps;
    const bool decode = T == n_entries && T <= ROWS_MAX && !m->taps;
    if (decode) {
        sh.logits = m->logits;
        auto& prog = m->progs[std::make_tuple(T, n_want, sh.nsplit)];
        if (!prog) {
            prog.reset(new MmiProgram());
            build_program(m, *prog, sh);
        }
        rc = prog->run(s, m->graphs, m->cap_stream);
        m->last_log = prog->launch_log();
        if (!rc && n_want && logits != m->logits)
            MMI_HIP_CHECK(hipMemcpyAsync(logits, m->logits, (size_t)n_want * m->cfg.vocab * sizeof(float), hipMemcpyDeviceToDevice, s));
    } else {
        sh.logits = logits;
        MmiProgram P;
        build_program(m, P, sh);
        rc = P.run_eager(s);
        m->last_log = P.launch_log();
    }
    for (int e = 0; e < n_entries; ++e) release_behind_window(m, m->slots[slots[e]]);
    return rc;
}

extern "C" int mmi_tlm_sample(mmi_tlm* m, int32_t n, const float* logits, const int32_t* slots, const float* temp, const int32_t* top_k, uint64_t seed,
                              int32_t* out, mmi_stream stream) {
    if (!m || n < 1 || n > m->max_slots || !logits || !slots || !temp || !top_k || !out) return mmi_fail(MMI_ERR_INVALID, "mmi_tlm_sample: bad arguments");
    MmiDeviceGuard guard(m->device);
    hipStream_t s = (hipStream_t)stream;
    const int V = m->cfg.vocab;
    for (int i = 0; i < n; ++i) {
        if (slots[i] < 0 || slots[i] >= m->max_slots) return mmi_fail(MMI_ERR_INVALID, "slot out of range");
        if (temp[i] > 0.f && m->samp_ld > 32768) return mmi_fail(MMI_ERR_UNSUPPORTED, "sampling needs a vocabulary of at most 32768 entries (greedy does not)");
    }
    Staging& st = m->staging[m->stage_at];
    m->stage_at = (m->stage_at + 1) & 3;
    if (st.used) MMI_HIP_CHECK(hipEventSynchronize(st.ev));
    memcpy(st.host, slots, (size_t)n * sizeof(int));
    unsigned long long rng[2] = {seed, m->samp_count++};
    memcpy(st.host + round_up(n, 2), rng, sizeof(rng));
    MMI_HIP_CHECK(hipMemcpyAsync(m->samp_map, st.host, (size_t)n * sizeof(int), hipMemcpyHostToDevice, s));
    MMI_HIP_CHECK(hipMemcpyAsync(m->samp_rng, st.host + round_up(n, 2), sizeof(rng), hipMemcpyHostToDevice, s));
    MMI_HIP_CHECK(hipEventRecord(st.ev, s));
    st.used = true;
    for (int i = 0; i < n;) {                        // runs of rows with the same parameters
        int k = i + 1;
        while (k < n && (temp[i] <= 0.f ? temp[k] <= 0.f : (temp[k] == temp[i] && top_k[k] == top_k[i]))) ++k;
        const int rows = k - i;
        if (temp[i] <= 0.f) {
            MMI_LAUNCH(k_tlm_argmax, rows, 256, 0, s, logits + (size_t)i * V, V, m->samp_map + i, out + i, m->last_tok);
        } else {
            const int ld = m->samp_ld;
            uint16_t* r = m->samp_rows + (size_t)i * ld;
            MMI_LAUNCH(k_tlm_sample_rows, (int)mmi_cdiv64((int64_t)rows * ld, 256), 256, 0, s, logits + (size_t)i * V, V, r, ld, rows);
            SampleArgs a;
            memset(&a, 0, sizeof(a));
            a.logits = r;
            a.ld = ld;
            a.V = ld;
            a.k = top_k[i] >= V || top_k[i] < 0 ? 0 : top_k[i];
            a.temp = temp[i];
            a.use_sampling = 1;
            a.use_noise = m->samp_zero;
            a.rng = m->samp_rng;
            a.site = i;
            a.out = out + i;
            a.out_stride = 1;
            a.B = rows;
            a.use_forced = m->samp_zero;
            if (ld <= 2048) MMI_LAUNCH((k_sample<256, 8, true>), rows, 256, 0, s, a);
            else if (ld <= 8192) MMI_LAUNCH((k_sample<1024, 8, true>), rows, 1024, 0, s, a);
            else MMI_LAUNCH((k_sample<1024, 32, true>), rows, 1024, 0, s, a);
            MMI_LAUNCH(k_tlm_last_tok, mmi_cdiv(rows, 64), 64, 0, s, out + i, m->samp_map + i, m->last_tok, rows);
        }
        MMI_CHECK_LAUNCH();
        i = k;
    }
    return MMI_OK;
}
