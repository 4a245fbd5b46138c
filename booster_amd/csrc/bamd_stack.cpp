// bamd_stack.cpp — host runtime of configured layer stacks (bamd_stack.h): configuration, weights (safetensors -> packed matrices on the device), per-sequence
// state (pages of latents or of keys and values, recurrent and convolution states, previous inputs), the scheduler that cuts a batch into passes, and the passes themselves.
//
// A context holds n_seq sequences over one pool of 64-position pages.  State that a pass both reads and replaces (previous inputs, convolution inputs) is double
// buffered per sequence; the recurrent state is owned by one block and updated in place.  A pass runs either decoding rows (one token per sequence; replayed as a
// hipGraph) or prompt portions (rows of all sequences behind one another).  Positions cannot be taken back: a recurrent state has no past.
#include "bamd_runtime.h"
#include "bamd_arch.h"
#include "bamd_dense.h"
#include "bamd_json.h"
#include "bamd_safetensors.h"
#include "bamd_stack.h"

#include <algorithm>
#include <fstream>
#include <iterator>
#include <map>
#include <math.h>
#include <string.h>

void bamd_launch_pack(const uint16_t * src, const int32_t * row_off, const int32_t * col_off, int row_tiles, int k_tiles, uint16_t * dst, int step, int ld, hipStream_t s);

namespace {
// BAMD_STAGE_GRAPH=0: decoding rows are enqueued kernel by kernel instead of as a captured hipGraph (as bamd_stage_step of the GGUF pipeline)
const bool g_graph = [] { const char * e = getenv("BAMD_STAGE_GRAPH"); return !(e && e[0] == '0'); }();
int up(int v, int m) { return (v + m - 1) / m * m; }
int ld_of(const bamd_dense & w) { return 16 * w.row_tiles; }      // floats per row of its output
int fail(const std::string & m) { return bamd_fail(m); }

// ---- loading -----------------------------------------------------------------------------------------------------------------------------------------
struct Loader {
    SafeTensors file; bamd_model * m; hipStream_t s = nullptr; int act = 0;
    void * staging = nullptr; size_t staging_bytes = 0; int32_t * maps = nullptr; size_t maps_n = 0;
    ~Loader() { if (staging) hipFree(staging); if (maps) hipFree(maps); if (s) hipStreamDestroy(s); }

    const SafeTensor * get(const std::string & name, std::vector<int64_t> shape) {
        const SafeTensor * t = file.find(name);
        if (!t) { fail("missing tensor " + name); return nullptr; }
        if (t->shape != shape && !(shape.empty() && t->count() == 1)) { std::string w; for (int64_t d : shape) w += (w.empty() ? "" : ", ") + std::to_string(d); fail("tensor " + name + ": expected shape [" + w + "]"); return nullptr; }
        if (t->dtype != "BF16" && t->dtype != "F32") { fail("tensor " + name + ": type " + t->dtype + " not supported (BF16, F32)"); return nullptr; }
        return t;
    }
    // 32-bit values of a tensor
    int values(const std::string & name, std::vector<int64_t> shape, std::vector<float> & h) {
        const SafeTensor * t = get(name, shape);
        if (!t) return 1;
        h.resize((size_t) t->count());
        for (size_t i = 0; i < h.size(); ++i) {
            if (t->dtype == "F32") memcpy(&h[i], t->data + 4 * i, 4);
            else { uint16_t u; memcpy(&u, t->data + 2 * i, 2); const uint32_t w = (uint32_t) u << 16; memcpy(&h[i], &w, 4); }
        }
        return 0;
    }
    template <typename U> int upload(const std::vector<U> & h, U ** out) {
        if (dev_alloc(m->allocs, (void **) out, std::max<size_t>(h.size(), 1) * sizeof(U))) return 1;
        HIPC(hipMemcpy(*out, h.data(), h.size() * sizeof(U), hipMemcpyHostToDevice));
        return 0;
    }
    // 32-bit vector on the device, times a constant; by: times another tensor of the same shape
    int vec(const std::string & name, std::vector<int64_t> shape, float ** out, float scale = 1.f, const std::string & by = "") {
        std::vector<float> h, w;
        if (values(name, shape, h) || (!by.empty() && values(by, shape, w))) return 1;
        for (size_t i = 0; i < h.size(); ++i) h[i] *= w.empty() ? scale : w[i] * scale;
        return upload(h, out);
    }
    // size of a tensor's dimension that no configuration entry names (0: no such tensor)
    int dim(const std::string & name, size_t at) { const SafeTensor * t = file.find(name); return t && at < t->shape.size() && t->shape[at] > 0 && t->shape[at] < (1 << 28) ? (int) t->shape[at] : 0; }
    int raw(const std::string & name, std::vector<int64_t> shape, uint16_t ** out) {
        const SafeTensor * t = matrix(name, shape);
        if (!t) return 1;
        if (dev_alloc(m->allocs, (void **) out, t->nbytes)) return 1;
        HIPC(hipMemcpy(*out, t->data, t->nbytes, hipMemcpyHostToDevice));
        return 0;
    }
    const SafeTensor * matrix(const std::string & name, std::vector<int64_t> shape) {
        const SafeTensor * t = get(name, shape);
        if (t && t->dtype != "BF16") { fail("tensor " + name + ": matrices are BF16"); return nullptr; }
        if (t && t->count() > 0x7fffffffll) { fail("tensor " + name + ": more than 2^31 values"); return nullptr; }
        return t;
    }
    // rows / columns of the packed matrix taken from the tensor's values at row[i] + col[j] (-1: zero); step: row tiles go to every step-th one, ld: column blocks of the whole matrix
    int pack(const SafeTensor * t, const std::vector<int32_t> & row, const std::vector<int32_t> & col, uint16_t * dst, int step = 1, int ld = 0) {
        const int rt = up((int) row.size(), 16) / 16, kt = up((int) col.size(), 32) / 32;
        if (t->nbytes > staging_bytes) {
            if (staging) HIPC(hipFree(staging));
            staging = nullptr; HIPC(hipMalloc(&staging, t->nbytes)); staging_bytes = t->nbytes;
        }
        const size_t n = (size_t) rt * 16 + (size_t) kt * 32;
        if (n > maps_n) { if (maps) HIPC(hipFree(maps)); maps = nullptr; HIPC(hipMalloc((void **) &maps, n * 4)); maps_n = n; }
        std::vector<int32_t> h(n, -1);
        std::copy(row.begin(), row.end(), h.begin());
        std::copy(col.begin(), col.end(), h.begin() + (size_t) rt * 16);
        HIPC(hipMemcpyAsync(staging, t->data, t->nbytes, hipMemcpyHostToDevice, s));
        HIPC(hipMemcpyAsync(maps, h.data(), n * 4, hipMemcpyHostToDevice, s));
        bamd_launch_pack((const uint16_t *) staging, maps, maps + (size_t) rt * 16, rt, kt, dst, step, ld ? ld : kt, s);
        HIPC(hipGetLastError());
        HIPC(hipStreamSynchronize(s));
        m->weight_bytes += (int64_t) t->nbytes;
        return 0;
    }
    int alloc(bamd_dense & d, int rows, int K) {
        d.rows = rows; d.K = up(K, 32); d.row_tiles = up(rows, 16) / 16; d.k_tiles = d.K / 32; d.bytes = (size_t) up(rows, 16) * d.K * 2;
        return dev_alloc(m->allocs, (void **) &d.w, d.bytes);
    }
    static std::vector<int32_t> steps(int n, int by) { std::vector<int32_t> v((size_t) n); for (int i = 0; i < n; ++i) v[(size_t) i] = i * by; return v; }
    // n groups of `size`, each padded to `padded`
    static std::vector<int32_t> grouped(int n, int size, int padded, int by) {
        std::vector<int32_t> v((size_t) n * padded, -1);
        for (int g = 0; g < n; ++g) for (int i = 0; i < size; ++i) v[(size_t) g * padded + i] = (g * size + i) * by;
        return v;
    }
    int plain(const std::string & name, int rows, int K, bamd_dense & d) {
        const SafeTensor * t = matrix(name, { rows, K });
        return !t || alloc(d, rows, K) || pack(t, steps(rows, K), steps(K, 1), const_cast<uint16_t *>(d.w));
    }
};
struct Conf {                                      // required entries of a JSON object
    const Json * j; std::string where;
    int num(const char * key, double & v) const {
        const Json * e = j ? j->get(key) : nullptr;
        if (!e || e->kind != Json::NUM) return fail("config.json: " + where + key + " missing");
        v = e->num;
        return 0;
    }
    int f32(const char * key, float & v) const { double d; if (num(key, d)) return 1; v = (float) d; return 0; }
    int size(const char * key, int & v, int lo = 1, int hi = 1 << 28) const {
        double d;
        if (num(key, d)) return 1;
        if (d != floor(d) || d < lo || d > hi) return fail("config.json: " + where + key + " out of range");
        v = (int) d;
        return 0;
    }
};

// ---- model --------------------------------------------------------------------------------------------------------------------------------------------
struct Ctx; struct Pass;
struct MixState { float * a = nullptr, * b = nullptr; void * cache = nullptr, * cache2 = nullptr; std::vector<MixState> sub; };       // of one layer in one context
struct Operand { int pre = BAMD_PRE_ROWS; bamd_group_norm_args grp; const void * x = nullptr; int ldx = 0; };   // what the output projection reads

struct Mixer {
    bamd_dense in, out;
    virtual ~Mixer() {}
    virtual int load(Loader & l, const Conf & c, const std::string & p, int E, float eps, const bamd_stack_design & d) = 0;
    virtual int state(Ctx & c, MixState & st) = 0;
    virtual int run(Pass & p, MixState & st, Operand & o) = 0;       // p.y holds the input projection's rows
    virtual int f32_cols() const { return 0; }                       // columns of the f32 scratch row it wants
    virtual int latents() const { return 0; }
    virtual int prompt_rows(int) const { return 0; }                 // query rows per tile of a prompt (0: no attention)
    virtual int scan_blocks() const { return 0; }                    // blocks of one segment of a prompt's scan (0: no segments)
    virtual void partials(int, size_t &, size_t &) const {}          // floats of the decoding shares' sums and of their maxima, for so many rows
    virtual double step_bytes(int len) const = 0;                    // state bytes of one decoded token
};
struct Layer { std::unique_ptr<Mixer> mix; float * norm1 = nullptr, * norm2 = nullptr, * pre1 = nullptr, * pre2 = nullptr, * shift = nullptr, * act = nullptr; bool mlp = false; bamd_dense up, down; int F = 0; float limit = 0; };      // norm: of a sublayer's output (scale included), pre: of its input

struct Stack : bamd_arch_runtime {
    bamd_stack_design d; bamd_model * m = nullptr;
    int act = 0, E = 0, V = 0, L = 0, max_pos = 0; float eps = 0, scale = 1;
    uint16_t * embd = nullptr, * pos = nullptr; float * norm_f = nullptr; bamd_dense head;
    std::vector<Layer> layers; std::string vocab;
    size_t el() const { return act == BAMD_ACT_F32 ? 4 : 2; }

    int load(bamd_model * m, const bamd_load_args & a, const bamd_stack_design & design);
    int context_init(bamd_context * c) override;
    void context_free(bamd_context * c) override;
    void clear(bamd_context * c) override;
    int seq_len(bamd_context * c, int seq) override;
    int seq_free(bamd_context * c, int seq) override;
    int decode_batch(bamd_context * c, const bamd_batch_entry * e, int n, float * logits, bool wait) override;
    int generate(bamd_context * c, const int32_t * seqs, int n_seqs, int n_steps, const int32_t * first, int32_t * out, float * ms) override;
    int stage(bamd_context * c, const int32_t * tokens, const void * token_dev, int n, int n_past, const void * hidden_in, void * hidden_out, bool want_logits, hipStream_t s) override;
    int argmax_to(bamd_context * c, int32_t * token_dev, hipStream_t s) override;
    int profile_kinds(bamd_context * c, int pos, int * launches, double * ms, double * bytes) override;
    const char * vocab_path() override { return vocab.c_str(); }
};

struct Seq { int len = 0, par = 0; std::vector<int32_t> pages; };
struct Timer {                                     // per-launch HIP events (profile_kinds)
    std::vector<hipEvent_t> ev; std::vector<int> kind; std::vector<double> bytes;
    ~Timer() { for (auto e : ev) hipEventDestroy(e); }
};
#define STACK_CTX 8192                             /* positions of a context that asks for none, where the model sets no bound */
#define STACK_ROWS 2048                            /* token rows of one pass */
#define SEG_MIN 64                                 /* tokens of the shortest scan segment */
#define PAIR_ROWS 4                                /* decoding rows up to which two branches share their launches */
#define SEG_BLOCKS 768                             /* blocks a scan wants */
struct Ctx {
    bamd_context * c = nullptr; Stack * st = nullptr;
    std::vector<Seq> seqs; std::vector<int32_t> free_pages; int max_pages = 0; bool pages_dirty = true;
    std::vector<MixState> mix; std::vector<float *> prev;
    int rows_cap = 0, splits_cap = 0;
    float * xa = nullptr, * xb = nullptr, * y = nullptr, * y2 = nullptr, * y3 = nullptr; void * h = nullptr;
    int ldy = 0, ldy2 = 0, ldy3 = 0, ldh = 0;
    void * qp = nullptr; float * part_o = nullptr, * part_ml = nullptr;
    void * kc = nullptr, * kk = nullptr, * kv = nullptr; size_t kc_n = 0, kk_n = 0, kv_n = 0;      // unpacked latents / keys / values of a prompt pass
    float * filtered = nullptr, * steps = nullptr; size_t filtered_n = 0, steps_n = 0;             // filtered channels, step sizes and decays of a prompt pass
    float * alpha = nullptr, * seg_state = nullptr, * seg_decay = nullptr; size_t alpha_n = 0, seg_state_n = 0, seg_decay_n = 0;      // decays and segment states of a prompt pass
    unsigned long long * keys = nullptr; int32_t * step = nullptr, * gen_out = nullptr; int gen_cap = 0;
    // step descriptors: entries | row_entry | tokens | want | query tiles | key blocks | scan segments, one device block per pass, filled from a ring of pinned blocks
    struct Layout { size_t ent, row, tok, want, tile, kblk, seg, total; int tiles, kblks, segs; } lay;
    unsigned char * dev = nullptr; int32_t * pages = nullptr;
    static constexpr int RING = 4;
    unsigned char * host[RING] = {}; int32_t * pages_host[RING] = {}; hipEvent_t ev[RING] = {}; int ring = 0;
    std::map<int, hipGraphExec_t> graphs;          // rows * 2 + greedy
};
struct Pass {                                      // one pass through the layers
    Ctx & c; Stack & st; hipStream_t s; bamd_batch_dev b; bool decode = false;
    int n_tiles = 0, k_rows = 0, max_n = 1, n_segs = 0; float * x; float * xo; const float * pend = nullptr; int ldp = 0; const float * pend_g = nullptr;
    Timer * tm = nullptr;
    void begin(int kind, double bytes) { if (!tm) return; hipEvent_t e; hipEventCreate(&e); hipEventRecord(e, s); tm->ev.push_back(e); tm->kind.push_back(kind); tm->bytes.push_back(bytes); }
    void end() { if (!tm) return; hipEvent_t e; hipEventCreate(&e); hipEventRecord(e, s); tm->ev.push_back(e); }

    bamd_residual_args residual(const float * mu, float * prev, const float * gi) {
        bamd_residual_args a; memset(&a, 0, sizeof a);
        a.norm = st.d.norm == STACK_NORM_SANDWICH ? BAMD_NORM_LAYER : BAMD_NORM_RMS; a.gi = gi;
        a.x = x; a.y = pend; a.ldy = ldp; a.g = pend_g; a.eps = st.eps; a.mu = mu; a.prev = prev; a.xo = xo; a.h = c.h; a.E = st.E; a.ldh = up(st.E, 32);
        return a;
    }
    void advanced(const float * y, int ld, const float * g) { std::swap(x, xo); pend = y; ldp = ld; pend_g = g; }
    // a product whose operand rows exist; small row counts stream the weights once
    int product(const bamd_dense & w, const void * in, int ldx, float * out, int ldo, int kind) {
        begin(kind, (double) w.bytes);
        const int rc = b.rows <= BAMD_MV_ROWS ? bamd_launch_dense_mv(st.act, w, BAMD_PRE_ROWS, b, nullptr, in, ldx, b.rows, out, ldo, s)
                                              : bamd_launch_dense_gemm(st.act, w, in, ldx, b.rows, out, ldo, BAMD_OUT_F32, s);
        end();
        return rc ? fail("dense product: unsupported shape") : 0;
    }
    bool fused(const bamd_dense & w) const { return b.rows == 1 && decode && bamd_dense_mv_lds(st.act, w.K) <= BAMD_MV_LDS; }
    int product_pre(const bamd_dense & w, int pre, const bamd_pre_args & p, float * out, int ldo, int kind) {
        if (fused(w)) {
            begin(kind, (double) w.bytes);
            const int rc = bamd_launch_dense_mv(st.act, w, pre, b, &p, nullptr, 0, 1, out, ldo, s);
            end();
            return rc ? fail("dense product: unsupported shape") : 0;
        }
        begin(2, 0);
        int ldx = 0;
        if (pre == BAMD_PRE_RESIDUAL) { bamd_launch_residual_rows(st.act, b, p.res, s); ldx = p.res.ldh; }
        else if (pre == BAMD_PRE_GLU) { bamd_launch_glu_rows(st.act, b.rows, p.glu, s); ldx = p.glu.ldh; }
        else if (pre == BAMD_PRE_POLY) { bamd_launch_poly_rows(st.act, b.rows, p.poly, s); ldx = p.poly.ldh; }
        else { bamd_launch_group_norm_rows(st.act, b.rows, p.grp, s); ldx = p.grp.ldh; }
        end();
        return product(w, c.h, ldx, out, ldo, kind);
    }
    int layers();
    int head(const int32_t * want, int n, float * logits);
};

// ---- mixers -------------------------------------------------------------------------------------------------------------------------------------------
struct Mamba2 : Mixer {
    int H = 0, P = 0, N = 0, G = 0, taps = 0, ng = 0, inner = 0, ch = 0; float eps = 0;
    float * conv = nullptr, * conv_b = nullptr, * dt_bias = nullptr, * A_log = nullptr, * D = nullptr, * norm = nullptr;
    int load(Loader & l, const Conf & c, const std::string & p, int E, float e, const bamd_stack_design &) override {
        eps = e;
        if (c.size("heads", H) || c.size("vdim", P) || c.size("state", N, 1, 256) || c.size("groups", G) || c.size("conv", taps, 1, 1024) || c.size("norm_groups", ng, 1, 512)) return 1;
        inner = H * P; ch = inner + 2 * G * N;
        if (H % G || inner % ng) return fail("config.json: " + c.where + "heads is no multiple of groups, or heads * vdim none of norm_groups");
        return l.plain(p + "in", inner + ch + H, E, in) || l.plain(p + "o", E, inner, out) || l.vec(p + "conv", { ch, taps }, &conv) || l.vec(p + "conv.b", { ch }, &conv_b) ||
               l.vec(p + "dt_bias", { H }, &dt_bias) || l.vec(p + "A_log", { H }, &A_log) || l.vec(p + "D", { H }, &D) || l.vec(p + "norm", { inner }, &norm);
    }
    int f32_cols() const override { return inner; }
    double step_bytes(int) const override { return 8.0 * H * N * P; }
    int state(Ctx & c, MixState & st) override;
    int run(Pass & p, MixState & st, Operand & o) override;
};
struct LatentAttention : Mixer {
    int H = 0, d = 0, dv = 0, R = 0, D = 0, Rp = 0, g_off = 0; float scale = 0, eps = 0; bool gated = false;
    float * c_norm = nullptr, * sink = nullptr; bamd_dense uk, uv; uint16_t * ukT = nullptr;
    int load(Loader & l, const Conf & c, const std::string & p, int E, float e, const bamd_stack_design & dz) override {
        eps = e; gated = dz.latent_gate;
        if (c.size("heads", H) || c.size("dim", d, 1, 256) || c.size("vdim", dv, 1, 256) || c.size("kv_rank", R, 1, 1024) || c.f32("scale", scale)) return 1;
        for (D = 32; D < std::max(d, dv); D *= 2) {}
        Rp = up(R, 32);
        if (Rp > bamd_latent_max_rank(l.act)) return fail("config.json: " + c.where + "kv_rank above " + std::to_string(bamd_latent_max_rank(l.act)) + " has no decoding kernel");
        // [q, each head padded to D | latent | gates]
        const SafeTensor * tq = l.matrix(p + "q", { H * d, E }), * tc = l.matrix(p + "dkv", { R, E }), * tg = gated ? l.matrix(p + "g", { H, E }) : nullptr;
        const SafeTensor * tk = l.matrix(p + "uk", { H * d, R }), * tv = l.matrix(p + "uv", { H * dv, R }), * to = l.matrix(p + "o", { E, H * dv });
        if (!tq || !tc || (gated && !tg) || !tk || !tv || !to) return 1;
        g_off = H * D + up(R, 16);
        if (l.alloc(in, g_off + (gated ? H : 0), E)) return 1;
        uint16_t * w = const_cast<uint16_t *>(in.w);
        const size_t row = (size_t) in.K;
        if (l.pack(tq, Loader::grouped(H, d, D, E), Loader::steps(E, 1), w) || l.pack(tc, Loader::steps(R, E), Loader::steps(E, 1), w + (size_t) H * D * row) ||
            (gated && l.pack(tg, Loader::steps(H, E), Loader::steps(E, 1), w + (size_t) g_off * row))) return 1;
        if (l.alloc(uk, H * D, R) || l.pack(tk, Loader::grouped(H, d, D, R), Loader::steps(R, 1), const_cast<uint16_t *>(uk.w))) return 1;
        if (l.alloc(uv, H * D, R) || l.pack(tv, Loader::grouped(H, dv, D, R), Loader::steps(R, 1), const_cast<uint16_t *>(uv.w))) return 1;
        if (l.alloc(out, E, H * D) || l.pack(to, Loader::steps(E, H * dv), Loader::grouped(H, dv, D, 1), const_cast<uint16_t *>(out.w))) return 1;
        // per head the transpose of its key rows: [Rp][D]
        if (dev_alloc(l.m->allocs, (void **) &ukT, (size_t) H * Rp * D * 2)) return 1;
        std::vector<int32_t> rows = Loader::steps(R, 1); rows.resize((size_t) Rp, -1);
        const int64_t wb = l.m->weight_bytes;
        for (int hd = 0; hd < H; ++hd) {
            std::vector<int32_t> cols((size_t) D, -1);
            for (int i = 0; i < d; ++i) cols[(size_t) i] = (hd * d + i) * R;
            if (l.pack(tk, rows, cols, ukT + (size_t) hd * Rp * D)) return 1;
        }
        l.m->weight_bytes = wb;
        return l.vec(p + "dkv.norm", { R }, &c_norm) || (dz.latent_sink && l.vec(p + "sink", { H }, &sink));
    }
    int latents() const override { return Rp; }
    int prompt_rows(int act) const override { return bamd_latent_prompt_rows(act, D); }
    double step_bytes(int len) const override { return (double) len * R * 2; }
    int state(Ctx & c, MixState & st) override;
    int run(Pass & p, MixState & st, Operand & o) override;
};
// ---- branches: mixers that share one input projection and one output projection (their results are summed there) ------------------------------------------
struct Part { const SafeTensor * t; std::vector<int32_t> rows, cols; int at; };       // of a packed matrix, at its row / column `at`
struct Branch {
    int in0 = 0, in_rows = 0, out0 = 0, out_cols = 0; float out_scale = 1;            // rows of the input projection, columns of the output projection
    virtual ~Branch() {}
    // in0, out0, out_scale are set; sets in_rows (a multiple of 16) and out_cols (of 32)
    virtual int load(Loader & l, const Conf & c, const std::string & p, int E, float eps, const bamd_stack_design & d, std::vector<Part> & in, std::vector<Part> & out) = 0;
    virtual int state(Ctx & c, MixState & st) = 0;
    virtual int run(Pass & p, MixState & st, int ld, int ldo) = 0;                    // p.c.y: rows of the input projection -> p.c.h: operand of the output projection
    virtual double step_bytes(int len) const = 0;
    virtual int f32_cols() const { return 0; }
    virtual int prompt_rows(int) const { return 0; }
    virtual int scan_blocks() const { return 0; }
    virtual void partials(int, size_t &, size_t &) const {}
};
// the bias of every distance up to `top` (and everything farther) from a table [rows][heads]: one row per distance in the first half, logarithmic steps in the second
std::vector<float> expand_bias(const std::vector<float> & rel, int rows, int heads, int top) {
    std::vector<float> h((size_t) heads * (top + 1));
    const int half = rows / 2;
    for (int n = 0; n <= top; ++n) {
        // (a step that falls on a whole distance belongs to it, whatever the logarithms round to)
        const int k = n < half ? n : std::min(rows - 1, half + (int) floor(log((double) n / half) / log((double) top / half) * (rows - half) + 1e-9));
        for (int i = 0; i < heads; ++i) h[(size_t) i * (top + 1) + n] = rel[(size_t) k * heads + i];
    }
    return h;
}
int kv_splits(const bamd_kv_args & a, int rows, int max_pages) {
    const int groups = std::max(1, rows * bamd_kv_groups(a)), span = bamd_kv_span(a, max_pages);
    return std::max(1, std::min({ (2 * span + 1 + 3) / 4, std::max(1, 1024 / groups), 64 }));    // four waves per share, half a page each; the row's own key is one more
}
struct KvAttention : Branch {
    bamd_kv_args a; int vdim = 0;
    KvAttention() { memset((void *) &a, 0, sizeof a); }
    int load(Loader & l, const Conf & c, const std::string & p, int E, float eps, const bamd_stack_design & d, std::vector<Part> & in, std::vector<Part> & out) override {
        int H, G;
        if (c.size("heads", H) || c.size("kv_heads", G) || c.size("dim", a.dim, 1, 256) || c.size("vdim", vdim, 1, 256) || c.f32("scale", a.scale) || (d.kv_cap && c.f32("softcap", a.cap))) return 1;
        if (H % G) return fail("config.json: " + c.where + "heads is no multiple of kv_heads");
        if (d.kv_cap && !(a.cap > 0)) return fail("config.json: " + c.where + "softcap out of range");
        a.heads = H; a.kv_heads = G; a.eps = eps; a.unit = d.kv_unit; a.gated = d.kv_gate; a.out_scale = out_scale; a.out_off = out0;
        a.window = 0x3fffffff; a.keep = 0;
        const Json * mask = c.j->get("mask");
        if (mask && mask->kind == Json::OBJ) {
            const Conf mc{ mask, c.where + "mask." };
            if (mc.size("size", a.window) || mc.size("keep_first", a.keep, 0)) return 1;
        }
        for (a.D = 32; a.D < std::max(a.dim, vdim); a.D *= 2) {}
        const int D = a.D;
        if (d.kv_bias) {
            const int B = l.dim(p + "rel", 0);
            std::vector<float> rel; float * dev;
            if (c.size("bias_max", a.bias_top, 1, 1 << 24) || l.values(p + "rel", { B, H }, rel)) return 1;
            if (a.bias_top <= B / 2 || B < 2) return fail("config.json: " + c.where + "bias_max is not above half of the bias table's rows");
            if (l.upload(expand_bias(rel, B, H, a.bias_top), &dev)) return 1;
            a.bias = dev;
        }
        // [q, each head padded to D | k | v | gates]
        const SafeTensor * tq = l.matrix(p + "q", { H * a.dim, E }), * tk = l.matrix(p + "k", { G * a.dim, E }), * tv = l.matrix(p + "v", { G * vdim, E }), * to = l.matrix(p + "o", { E, H * vdim });
        const SafeTensor * tg = d.kv_gate ? l.matrix(p + "g", { H, E }) : nullptr;
        if (!tq || !tk || !tv || !to || (d.kv_gate && !tg)) return 1;
        const std::vector<int32_t> cols = Loader::steps(E, 1);
        a.q_off = in0; a.k_off = a.q_off + H * D; a.v_off = a.k_off + G * D; a.g_off = a.v_off + G * D;
        in.push_back({ tq, Loader::grouped(H, a.dim, D, E), cols, a.q_off }); in.push_back({ tk, Loader::grouped(G, a.dim, D, E), cols, a.k_off }); in.push_back({ tv, Loader::grouped(G, vdim, D, E), cols, a.v_off });
        if (tg) in.push_back({ tg, Loader::steps(H, E), cols, a.g_off });
        out.push_back({ to, Loader::steps(E, H * vdim), Loader::grouped(H, vdim, D, 1), out0 });
        in_rows = a.g_off + (tg ? up(H, 16) : 0) - in0; out_cols = H * D;
        return 0;
    }
    double step_bytes(int len) const override { return (double) std::min<long>(len, (long) a.window + a.keep) * a.kv_heads * (a.dim + vdim) * 2; }
    int prompt_rows(int act) const override { return bamd_kv_prompt_rows(act, a.D); }
    void partials(int rows, size_t & po, size_t & pm) const override {
        const size_t cells = std::max<size_t>(1024, (size_t) rows * bamd_kv_groups(a));       // rows x groups x splits never exceeds this (kv_splits)
        po = std::max(po, cells * 16 * a.D); pm = std::max(pm, cells * 32);
    }
    int state(Ctx & c, MixState & st) override;
    int run(Pass & p, MixState & st, int ld, int ldo) override;
    bamd_kv_args args(Pass & p, MixState & st, int ld, int ldo) const;
};
struct GatedLinear : Branch {
    bamd_gla_args a; int N = 0;
    GatedLinear() { memset((void *) &a, 0, sizeof a); }
    int load(Loader & l, const Conf & c, const std::string & p, int E, float eps, const bamd_stack_design & d, std::vector<Part> & in, std::vector<Part> & out) override {
        int H; float tau;
        if (c.size("heads", H) || c.size("dim", N, 1, 256) || c.size("vdim", a.P) || c.f32("tau", tau)) return 1;
        if (!(tau > 0)) return fail("config.json: " + c.where + "tau out of range");
        const int P = a.P, R = l.dim(p + "a1", 0);
        if (R > 1024) return fail("tensor " + p + "a1: rank above 1024");
        a.heads = H; a.Np = up(N, 4); a.Pp = up(P, 4); a.rank = R; a.inv_tau = 1.f / tau; a.q_scale = (float) (1.0 / sqrt((double) N)); a.eps = eps; a.out_off = out0;
        const SafeTensor * tq = l.matrix(p + "q", { H * N, E }), * tk = l.matrix(p + "k", { H * N, E }), * tv = l.matrix(p + "v", { H * P, E }), * tg = d.gla_gate ? l.matrix(p + "g", { H * P, E }) : nullptr;
        const SafeTensor * t1 = l.matrix(p + "a1", { R, E }), * t2 = l.matrix(p + "a2", { H * N, R }), * to = l.matrix(p + "o", { E, H * P });
        if (!tq || !tk || !tv || (d.gla_gate && !tg) || !t1 || !t2 || !to) return 1;
        // [q | k | v | gate, heads padded to four | the decays' low rank]
        const std::vector<int32_t> cols = Loader::steps(E, 1);
        a.q_off = in0; a.k_off = a.q_off + up(H * a.Np, 16); a.v_off = a.k_off + up(H * a.Np, 16); a.g_off = a.v_off + up(H * a.Pp, 16); a.t_off = a.g_off + (tg ? up(H * a.Pp, 16) : 0);
        in.push_back({ tq, Loader::grouped(H, N, a.Np, E), cols, a.q_off }); in.push_back({ tk, Loader::grouped(H, N, a.Np, E), cols, a.k_off }); in.push_back({ tv, Loader::grouped(H, P, a.Pp, E), cols, a.v_off });
        if (tg) in.push_back({ tg, Loader::grouped(H, P, a.Pp, E), cols, a.g_off }); else a.g_off = -1;
        in.push_back({ t1, Loader::steps(R, E), cols, a.t_off });
        in_rows = a.t_off + up(R, 16) - in0; out_cols = up(H * a.Pp, 32);
        a.out_cols = out_cols;
        std::vector<int32_t> oc = Loader::grouped(H, P, a.Pp, 1); oc.resize((size_t) out_cols, -1);
        out.push_back({ to, Loader::steps(E, H * P), oc, out0 });
        // second factor of the decays, transposed: neighbouring channels are neighbours
        std::vector<uint16_t> w((size_t) R * H * a.Np, 0); std::vector<float> bias, pb((size_t) H * a.Np, 0.f), nm;
        for (int i = 0; i < H * N; ++i) for (int r = 0; r < R; ++r) memcpy(&w[(size_t) r * H * a.Np + (size_t) (i / N) * a.Np + i % N], t2->data + ((size_t) i * R + r) * 2, 2);
        if (l.values(p + "a2.b", { H * N }, bias) || l.values(p + "norm", { P }, nm)) return 1;
        for (int i = 0; i < H * N; ++i) pb[(size_t) (i / N) * a.Np + i % N] = bias[(size_t) i];
        for (float & v : nm) v *= out_scale;
        nm.resize((size_t) a.Pp, 0.f);
        uint16_t * dw; float * db, * dn;
        if (l.upload(w, &dw) || l.upload(pb, &db) || l.upload(nm, &dn)) return 1;
        a.a2 = dw; a.a2b = db; a.norm = dn;
        l.m->weight_bytes += (int64_t) t2->nbytes;
        return 0;
    }
    double step_bytes(int) const override { return 8.0 * a.heads * N * a.P; }
    int f32_cols() const override { return a.heads * a.Pp; }
    int scan_blocks() const override { return bamd_gla_blocks(a.heads, a.Pp); }
    int state(Ctx & c, MixState & st) override;
    int run(Pass & p, MixState & st, int ld, int ldo) override;
    bamd_gla_args args(Pass & p, MixState & st, int ld, int ldo) const;
};
// several branches over one input, their outputs summed with a scale each
struct Parallel : Mixer {
    std::vector<std::unique_ptr<Branch>> br;
    int load(Loader & l, const Conf & c, const std::string & p, int E, float eps, const bamd_stack_design & d) override {
        std::vector<Part> pi, po;
        const char * sides[2] = { "left", "right" };
        br.emplace_back(new KvAttention()); br.emplace_back(new GatedLinear());
        int ni = 0, no = 0;
        for (int i = 0; i < 2; ++i) {
            const std::string side = sides[i];
            Branch & b = *br[(size_t) i];
            const Json * j = c.j ? c.j->get(side) : nullptr;
            if (!j || j->kind != Json::OBJ) return fail("config.json: " + c.where + side + " missing");
            b.in0 = ni; b.out0 = no;
            if (c.f32((side + "_scale").c_str(), b.out_scale) || b.load(l, Conf{ j, c.where + side + "." }, p + side + ".", E, eps, d, pi, po)) return 1;
            ni += b.in_rows; no += b.out_cols;
        }
        if (l.alloc(in, ni, E) || l.alloc(out, E, no)) return 1;
        for (const Part & q : pi) if (l.pack(q.t, q.rows, q.cols, const_cast<uint16_t *>(in.w) + (size_t) q.at * in.K)) return 1;
        for (const Part & q : po) if (l.pack(q.t, q.rows, q.cols, const_cast<uint16_t *>(out.w) + (size_t) (q.at / 32) * 512, 1, out.k_tiles)) return 1;
        return 0;
    }
    int state(Ctx & c, MixState & st) override {
        st.sub.resize(br.size());
        for (size_t i = 0; i < br.size(); ++i) if (br[i]->state(c, st.sub[i])) return 1;
        return 0;
    }
    int run(Pass & p, MixState & st, Operand & o) override;
    double step_bytes(int len) const override { double t = 0; for (auto & b : br) t += b->step_bytes(len); return t; }
    int f32_cols() const override { int n = 0; for (auto & b : br) n = std::max(n, b->f32_cols()); return n; }
    int prompt_rows(int act) const override { int n = 0; for (auto & b : br) if (const int q = b->prompt_rows(act)) n = n ? std::min(n, q) : q; return n; }
    int scan_blocks() const override { int n = 0; for (auto & b : br) n = std::max(n, b->scan_blocks()); return n; }
    void partials(int rows, size_t & po, size_t & pm) const override { for (auto & b : br) b->partials(rows, po, pm); }
};
std::unique_ptr<Mixer> make_mixer(const std::string & type, const bamd_stack_design & d) {
    const std::string all = std::string(" ") + d.mixers + " ";
    if (all.find(" " + type + " ") == std::string::npos) return nullptr;
    if (type == "mamba2") return std::unique_ptr<Mixer>(new Mamba2());
    if (type == "latent_attention") return std::unique_ptr<Mixer>(new LatentAttention());
    if (type == "parallel") return std::unique_ptr<Mixer>(new Parallel());
    return nullptr;
}

int Stack::load(bamd_model * model, const bamd_load_args & a, const bamd_stack_design & design) {
    m = model; d = design;
    const std::string dir = a.path;
    std::ifstream f(dir + "/config.json", std::ios::binary);
    const std::string text((std::istreambuf_iterator<char>(f)), std::istreambuf_iterator<char>());
    Json j; std::string err;
    if (!Json::parse(text.data(), text.data() + text.size(), j, err)) return fail(dir + "/config.json: " + err);
    const Conf top{ &j, "" };
    const Json * ls = j.get("layers");
    if (top.size("vocab", V) || top.size("width", E) || (d.scaled_embedding && Conf{ j.get("embedding"), "embedding." }.f32("scale", scale)) || Conf{ j.get("norm"), "norm." }.f32("eps", eps)) return 1;
    if (d.learned_positions && top.size("max_positions", max_pos)) return 1;
    if (!ls || ls->kind != Json::ARR || ls->arr.empty()) return fail("config.json: layers missing");
    L = (int) ls->arr.size();
    int lf = a.layer_first, ll = a.layer_last;
    if (ll < 0 || ll > L) ll = L;
    if (lf < 0 || lf > ll) return fail("bad layer range");
    m->E = E; m->V = V; m->L = L; m->eps = eps; m->n_ctx_train = d.learned_positions ? max_pos : STACK_CTX; m->layer_first = lf; m->layer_last = ll; m->with_embd = a.with_embd != 0; m->with_output = a.with_output != 0;
    if (a.dtype != BAMD_DTYPE_DEFAULT && a.dtype != BAMD_DTYPE_BF16 && a.dtype != BAMD_DTYPE_F32) return fail("unknown dtype");
    act = a.dtype == BAMD_DTYPE_F32 ? BAMD_ACT_F32 : BAMD_ACT_BF16;
    { std::ifstream v(dir + "/tokenizer.gguf"); if (v) vocab = dir + "/tokenizer.gguf"; }

    Loader l; l.m = m; l.act = act;
    if (!l.file.open(dir + "/model.safetensors", err)) return fail(err);
    const int ndev = bamd_device_count();
    if (ndev <= 0) return fail("no HIP device available: libbooster_amd has no CPU fallback");
    if (a.device < 0 || a.device >= ndev) return fail("bad device index");
    HIPC(hipSetDevice(a.device));
    m->device = a.device;
    { hipDeviceProp_t p; HIPC(hipGetDeviceProperties(&p, a.device)); m->n_cu = p.multiProcessorCount > 0 ? p.multiProcessorCount : 256; }
    HIPC(hipStreamCreate(&l.s));
    if (m->with_embd && (l.raw("embed", { V, E }, &embd) || (d.learned_positions && l.raw("pos", { max_pos, E }, &pos)))) return 1;
    const bool sandwich = d.norm == STACK_NORM_SANDWICH;
    const std::vector<int64_t> gain = sandwich ? std::vector<int64_t>{ E } : std::vector<int64_t>{};      // shape of a norm's gain
    float logit_scale = 1.f;                                     // enters with the last norm's gain
    if (d.tied_head && top.f32("logit_scale", logit_scale)) return 1;
    if (m->with_output && (l.vec("final.norm", gain, &norm_f, logit_scale) || l.plain(d.tied_head ? "embed" : "head", V, E, head))) return 1;
    layers.resize((size_t) (ll - lf));
    for (int il = lf; il < ll; ++il) {
        Layer & ly = layers[(size_t) (il - lf)];
        const Json & cj = ls->arr[(size_t) il];
        const std::string p = "l" + std::to_string(il) + ".", where = "layers[" + std::to_string(il) + "].";
        const Json * type = cj.get("type"), * mlp = cj.get("mlp");
        if (!type || type->kind != Json::STR) return fail("config.json: " + where + "type missing");
        ly.mix = make_mixer(type->str, d);
        if (!ly.mix) return fail("config.json: " + where + "type \"" + type->str + "\" is not one of this architecture's mixers (" + d.mixers + ")");
        if (ly.mix->load(l, Conf{ cj.get("mixer"), where + "mixer." }, p + "mix.", E, eps, d)) return 1;
        if (sandwich ? l.vec(p + "norm1", gain, &ly.pre1) || l.vec(p + "norm1b", gain, &ly.norm1, 1.f, p + "ls1") : l.vec(p + "norm1", gain, &ly.norm1)) return 1;
        if ((d.token_shift && l.vec(p + "shift", { E }, &ly.shift))) return 1;
        ly.mlp = mlp && mlp->kind == Json::OBJ;
        if (ly.mlp) {
            const Json * kind = mlp->get("kind");
            if (!kind || kind->str != "dense") return fail("config.json: " + where + "mlp.kind is not \"dense\"");
            if (Conf{ mlp, where + "mlp." }.size("ff", ly.F)) return 1;
            if (sandwich ? l.vec(p + "norm2", gain, &ly.pre2) || l.vec(p + "norm2b", gain, &ly.norm2, 1.f, p + "ls2") : l.vec(p + "norm2", gain, &ly.norm2)) return 1;
            if (l.plain(p + "mlp.down", E, ly.F, ly.down)) return 1;
            if (d.mlp_act == STACK_ACT_CLAMPED_GLU) {
                // gate and up rows in turn, sixteen of each: one wave holds both halves of its outputs
                const SafeTensor * tg = l.matrix(p + "mlp.gate", { ly.F, E }), * tu = l.matrix(p + "mlp.up", { ly.F, E });
                if (!tg || !tu || Conf{ mlp, where + "mlp." }.f32("limit", ly.limit) || l.alloc(ly.up, 2 * ly.down.K, E)) return 1;
                std::vector<int32_t> rows = Loader::steps(ly.F, E); rows.resize((size_t) ly.down.K, -1);
                uint16_t * w = const_cast<uint16_t *>(ly.up.w);
                if (l.pack(tg, rows, Loader::steps(E, 1), w, 2) || l.pack(tu, rows, Loader::steps(E, 1), w + (size_t) 16 * ly.up.K, 2)) return 1;
            } else if (l.plain(p + "mlp.up", ly.F, E, ly.up) || l.vec(p + "mlp.act", { 4 }, &ly.act)) return 1;
        }
    }
    return 0;
}

// ---- context ------------------------------------------------------------------------------------------------------------------------------------------
int Mamba2::state(Ctx & c, MixState & st) {
    const size_t hist = (size_t) 2 * c.c->n_seq * (taps - 1) * ch, S = (size_t) c.c->n_seq * H * N * P;
    return dev_alloc(c.c->allocs, (void **) &st.a, std::max<size_t>(hist, 1) * 4) || dev_alloc(c.c->allocs, (void **) &st.b, S * 4);
}
int LatentAttention::state(Ctx & c, MixState & st) {
    const size_t n_pages = c.free_pages.size();
    return dev_alloc(c.c->allocs, &st.cache, n_pages * BAMD_PAGE * Rp * c.st->el());
}
int KvAttention::state(Ctx & c, MixState & st) {
    const size_t n = (size_t) c.free_pages.size() * a.kv_heads * BAMD_PAGE * a.D * c.st->el();
    return dev_alloc(c.c->allocs, &st.cache, n) || dev_alloc(c.c->allocs, &st.cache2, n);
}
int GatedLinear::state(Ctx & c, MixState & st) { return dev_alloc(c.c->allocs, (void **) &st.b, (size_t) c.c->n_seq * a.heads * a.Np * a.Pp * 4); }
Ctx & ctx_of(bamd_context * c) { return *(Ctx *) c->arch_state; }

int Stack::context_init(bamd_context * bc) {
    Ctx * cp = new Ctx();
    bc->arch_state = cp;
    Ctx & c = *cp;
    c.c = bc; c.st = this;
    const int S = bc->n_seq, n_ctx = bc->n_ctx;
    c.seqs.resize((size_t) S);
    c.max_pages = (n_ctx + BAMD_PAGE - 1) / BAMD_PAGE;
    for (int i = c.max_pages + S - 1; i > 0; --i) c.free_pages.push_back(i - 1);        // n_ctx positions fit however they are spread over the sequences
    c.rows_cap = std::max(S, std::min(STACK_ROWS, up(n_ctx, 64)));
    c.ldh = up(E, 32); c.ldy2 = up(E, 16);
    size_t qp = 0, po = 0, pm = 0;
    const int brows = std::min(S, c.rows_cap);
    for (Layer & ly : layers) {
        Mixer & mx = *ly.mix;
        c.ldy = std::max({ c.ldy, ld_of(mx.in), ly.mlp ? ld_of(ly.up) : 0 });
        c.ldh = std::max({ c.ldh, mx.out.K, mx.in.K, ly.mlp ? ly.down.K : 0 });
        c.ldy3 = std::max(c.ldy3, up(mx.f32_cols(), 16));
        if (auto * la = dynamic_cast<LatentAttention *>(&mx)) {
            const size_t hg = (size_t) (la->H + 15) / 16, cells = 512 + (size_t) brows * hg;     // rows x head groups x splits never exceeds this (splits_for)
            qp = std::max(qp, (size_t) brows * hg * 16 * la->Rp); po = std::max(po, cells * 16 * la->Rp); pm = std::max(pm, cells * 32);
        }
        mx.partials(brows, po, pm);
    }
    const size_t R = (size_t) c.rows_cap;
    if (dev_alloc(bc->allocs, (void **) &c.xa, R * E * 4) || dev_alloc(bc->allocs, (void **) &c.xb, R * E * 4) || dev_alloc(bc->allocs, (void **) &c.y, R * std::max(c.ldy, 16) * 4) ||
        dev_alloc(bc->allocs, (void **) &c.y2, R * c.ldy2 * 4) || dev_alloc(bc->allocs, (void **) &c.y3, R * std::max(c.ldy3, 16) * 4) || dev_alloc(bc->allocs, &c.h, R * c.ldh * el())) return 1;
    if (qp && dev_alloc(bc->allocs, &c.qp, qp * el())) return 1;
    if (po && (dev_alloc(bc->allocs, (void **) &c.part_o, po * 4) || dev_alloc(bc->allocs, (void **) &c.part_ml, pm * 4))) return 1;
    if (qp) HIPC(hipMemset(c.qp, 0, qp * el()));                  // rows of absent heads stay zero
    c.mix.resize(layers.size()); c.prev.resize(layers.size());
    for (size_t i = 0; i < layers.size(); ++i) {
        if (layers[i].mix->state(c, c.mix[i])) return 1;
        if (d.token_shift && dev_alloc(bc->allocs, (void **) &c.prev[i], (size_t) 2 * S * E * 4)) return 1;
    }
    c.gen_cap = n_ctx + 8;
    if (dev_alloc(bc->allocs, (void **) &c.keys, std::max<size_t>((size_t) S, BAMD_LOGIT_ROWS) * 8) || dev_alloc(bc->allocs, (void **) &c.step, 4) || dev_alloc(bc->allocs, (void **) &c.gen_out, (size_t) S * c.gen_cap * 4)) return 1;
    Ctx::Layout & y = c.lay;
    const int max_e = S;
    y.tiles = (int) R / 16 + max_e; y.kblks = c.max_pages + S; y.segs = (int) R / SEG_MIN + max_e;
    size_t at = 0;
    auto put = [&](size_t bytes) { const size_t p = at; at = (at + bytes + 63) / 64 * 64; return p; };
    y.ent = put(sizeof(bamd_entry) * (size_t) max_e); y.row = put(R * 4); y.tok = put(R * 4); y.want = put(R * 4); y.tile = put(sizeof(bamd_qtile) * (size_t) y.tiles); y.kblk = put((size_t) y.kblks * 4); y.seg = put(sizeof(bamd_segment) * (size_t) y.segs);
    y.total = at;
    if (dev_alloc(bc->allocs, (void **) &c.dev, y.total) || dev_alloc(bc->allocs, (void **) &c.pages, (size_t) S * c.max_pages * 4)) return 1;
    for (int i = 0; i < Ctx::RING; ++i) {
        HIPC(hipHostMalloc((void **) &c.host[i], y.total)); HIPC(hipHostMalloc((void **) &c.pages_host[i], (size_t) S * c.max_pages * 4));
        HIPC(hipEventCreateWithFlags(&c.ev[i], hipEventDisableTiming));
    }
    return 0;
}
void Stack::context_free(bamd_context * bc) {
    Ctx * c = (Ctx *) bc->arch_state;
    if (!c) return;
    for (auto & g : c->graphs) hipGraphExecDestroy(g.second);
    for (int i = 0; i < Ctx::RING; ++i) { if (c->host[i]) hipHostFree(c->host[i]); if (c->pages_host[i]) hipHostFree(c->pages_host[i]); if (c->ev[i]) hipEventDestroy(c->ev[i]); }
    for (void * p : { c->kc, c->kk, c->kv, (void *) c->filtered, (void *) c->steps, (void *) c->alpha, (void *) c->seg_state, (void *) c->seg_decay }) if (p) hipFree(p);
    delete c;
    bc->arch_state = nullptr;
}
void Stack::clear(bamd_context * bc) { for (int i = 0; i < bc->n_seq; ++i) seq_free(bc, i); }
int Stack::seq_len(bamd_context * bc, int seq) { Ctx & c = ctx_of(bc); return seq < 0 || seq >= bc->n_seq ? -1 : c.seqs[(size_t) seq].len; }
int Stack::seq_free(bamd_context * bc, int seq) {
    Ctx & c = ctx_of(bc);
    if (seq < 0 || seq >= bc->n_seq) return fail("sequence out of range");
    Seq & q = c.seqs[(size_t) seq];
    // later passes are enqueued behind whatever still reads these pages; states are taken as zero by a sequence's first token
    while (!q.pages.empty()) { c.free_pages.push_back(q.pages.back()); q.pages.pop_back(); }
    q.len = 0; q.par = 0;
    return 0;
}
int reserve(Ctx & c, int seq, int len) {
    Seq & q = c.seqs[(size_t) seq];
    const int need = (len + BAMD_PAGE - 1) / BAMD_PAGE;
    if (need > c.max_pages || need - (int) q.pages.size() > (int) c.free_pages.size()) return fail("context overflow: no free pages");
    while ((int) q.pages.size() < need) { q.pages.push_back(c.free_pages.back()); c.free_pages.pop_back(); c.pages_dirty = true; }
    return 0;
}

// ---- passes -------------------------------------------------------------------------------------------------------------------------------------------
int grow(Ctx & c, void ** p, size_t * have, size_t need, hipStream_t s) {
    if (need <= *have) return 0;
    HIPC(hipStreamSynchronize(s));
    if (*p) HIPC(hipFree(*p));
    *p = nullptr; *have = 0;
    HIPC(hipMalloc(p, need + 4096)); *have = need;
    return 0;
}
int Mamba2::run(Pass & p, MixState & st, Operand & o) {
    bamd_ssm_args a; memset(&a, 0, sizeof a);
    a.in = p.c.y; a.ld = ld_of(in); a.conv = conv; a.conv_b = conv_b; a.dt_bias = dt_bias; a.A_log = A_log; a.D = D; a.hist = st.a; a.state = st.b; a.out = p.c.y3; a.ldo = inner;
    a.heads = H; a.P = P; a.N = N; a.groups = G; a.taps = taps;
    p.begin(1, p.tm ? step_bytes(0) : 0);
    if (p.max_n > 1 && (grow(p.c, (void **) &p.c.filtered, &p.c.filtered_n, (size_t) p.b.rows * ch * 4, p.s) || grow(p.c, (void **) &p.c.steps, &p.c.steps_n, (size_t) p.b.rows * H * 8, p.s))) return 1;
    a.filtered = p.c.filtered; a.steps = p.c.steps;
    const int rc = bamd_launch_ssm(p.b, a, p.max_n, p.s);
    p.end();
    if (rc) return fail("state-space kernel: unsupported shape");
    o.pre = BAMD_PRE_GROUP;
    o.grp = { p.c.y3, inner, norm, ng, eps, p.c.h, inner, out.K };
    return 0;
}
int splits_for(const Ctx & c, int rows, int hgroups) { return std::max(1, std::min({ 512 / std::max(1, rows * hgroups), c.max_pages, 64 })); }
int LatentAttention::run(Pass & p, MixState & st, Operand & o) {
    Ctx & c = p.c;
    const int act = p.st.act;
    bamd_latent_args a; memset((void *) &a, 0, sizeof a);
    a.in = c.y; a.ld = ld_of(in); a.q_off = 0; a.c_off = H * D; a.g_off = g_off; a.c_norm = c_norm; a.eps = eps; a.scale = scale; a.sink = sink; a.gated = gated ? 1 : 0;
    a.heads = H; a.D = D; a.R = R; a.Rp = Rp; a.cache = st.cache; a.ukT = ukT; a.uk = uk; a.uv = uv; a.out = c.h; a.ldo = out.K;
    o.x = c.h; o.ldx = out.K;
    p.begin(1, p.tm ? step_bytes(c.seqs[0].len + 1) + (double) uk.bytes + (double) uv.bytes : 0);
    int rc = 0;
    if (p.decode) rc = bamd_launch_latent_decode(act, p.b, a, c.qp, c.part_o, c.part_ml, splits_for(c, p.b.rows, (H + 15) / 16), p.s);
    else {
        const size_t kr = (size_t) p.k_rows, el = p.st.el();
        if (grow(c, &c.kc, &c.kc_n, kr * Rp * el, p.s) || grow(c, &c.kk, &c.kk_n, kr * H * D * el, p.s) || grow(c, &c.kv, &c.kv_n, kr * H * D * el, p.s)) return 1;
        bamd_launch_latent_store(act, p.b, a, p.s);
        bamd_launch_latent_gather(act, p.b, a, (const int32_t *) (c.dev + c.lay.kblk), p.k_rows, c.kc, p.s);
        rc = bamd_launch_dense_gemm(act, uk, c.kc, Rp, p.k_rows, c.kk, H * D, BAMD_OUT_ACT, p.s) || bamd_launch_dense_gemm(act, uv, c.kc, Rp, p.k_rows, c.kv, p.k_rows, BAMD_OUT_ACT_T, p.s) ||
             bamd_launch_latent_prompt(act, p.b, a, (const bamd_qtile *) (c.dev + c.lay.tile), p.n_tiles, c.kk, c.kv, p.k_rows, p.s);
    }
    p.end();
    return rc ? fail("latent attention: unsupported shape") : 0;
}
bamd_kv_args KvAttention::args(Pass & p, MixState & st, int ld, int ldo) const {
    bamd_kv_args k = a;
    k.in = p.c.y; k.ld = ld; k.kc = st.cache; k.vc = st.cache2; k.out = p.c.h; k.ldo = ldo;
    return k;
}
int KvAttention::run(Pass & p, MixState & st, int ld, int ldo) {
    Ctx & c = p.c;
    const int act = p.st.act;
    const bamd_kv_args k = args(p, st, ld, ldo);
    int rc = 0;
    if (p.decode) rc = bamd_launch_kv_decode(act, p.b, k, c.part_o, c.part_ml, kv_splits(k, p.b.rows, c.max_pages), p.s);
    else {
        bamd_launch_kv_store(act, p.b, k, (const int32_t *) (c.dev + c.lay.kblk), p.k_rows, p.s);
        rc = bamd_launch_kv_prompt(act, p.b, k, (const bamd_qtile *) (c.dev + c.lay.tile), p.n_tiles, p.s);
    }
    return rc ? fail("attention over keys and values: unsupported shape") : 0;
}
bamd_gla_args GatedLinear::args(Pass & p, MixState & st, int ld, int ldo) const {
    bamd_gla_args g = a;
    g.in = p.c.y; g.ld = ld; g.state = st.b; g.y = p.c.y3; g.ldy = a.heads * a.Pp; g.out = p.c.h; g.ldo = ldo;
    return g;
}
int GatedLinear::run(Pass & p, MixState & st, int ld, int ldo) {
    Ctx & c = p.c;
    bamd_gla_args g = args(p, st, ld, ldo);
    if (p.max_n > 1) {
        const size_t ch = (size_t) a.heads * a.Np;
        if (grow(c, (void **) &c.alpha, &c.alpha_n, (size_t) p.b.rows * ch * 4, p.s)) return 1;
        if (p.n_segs > p.b.n_entries && (grow(c, (void **) &c.seg_state, &c.seg_state_n, p.n_segs * ch * a.Pp * 4, p.s) || grow(c, (void **) &c.seg_decay, &c.seg_decay_n, p.n_segs * ch * 4, p.s))) return 1;
        g.alpha = c.alpha; g.seg_state = c.seg_state; g.seg_decay = c.seg_decay;
    }
    if (bamd_launch_gla(p.b, g, p.max_n, (const bamd_segment *) (c.dev + c.lay.seg), p.n_segs, p.s)) return fail("gated linear attention: unsupported shape");
    bamd_launch_gla_norm(p.st.act, g, p.b.rows, p.s);
    return 0;
}
int Parallel::run(Pass & p, MixState & st, Operand & o) {
    o.x = p.c.h; o.ldx = out.K;
    p.begin(1, p.tm ? step_bytes(p.c.seqs[0].len + 1) : 0);
    auto * kv = dynamic_cast<KvAttention *>(br[0].get()); auto * gl = dynamic_cast<GatedLinear *>(br[1].get());
    if (p.decode && p.b.rows <= PAIR_ROWS && kv && gl) {           // few rows: the branches' blocks share their launches
        const bamd_kv_args k = kv->args(p, st.sub[0], ld_of(in), out.K);
        if (bamd_launch_kv_gla_decode(p.st.act, p.b, k, gl->args(p, st.sub[1], ld_of(in), out.K), p.c.part_o, p.c.part_ml, kv_splits(k, p.b.rows, p.c.max_pages), p.s)) return fail("attention beside gated linear attention: unsupported shape");
    } else for (size_t i = 0; i < br.size(); ++i) if (br[i]->run(p, st.sub[i], ld_of(in), out.K)) return 1;
    p.end();
    return 0;
}
int Pass::layers() {
    bamd_pre_args pa; memset((void *) &pa, 0, sizeof pa);
    for (size_t i = 0; i < st.layers.size(); ++i) {
        Layer & ly = st.layers[i];
        Mixer & mx = *ly.mix;
        pa.res = residual(ly.shift, c.prev[i], ly.pre1);
        if (product_pre(mx.in, BAMD_PRE_RESIDUAL, pa, c.y, ld_of(mx.in), 0)) return 1;
        Operand o;
        if (mx.run(*this, c.mix[i], o)) return 1;
        if (o.pre == BAMD_PRE_ROWS) { if (product(mx.out, o.x, o.ldx, c.y2, c.ldy2, 3)) return 1; }
        else { pa.grp = o.grp; if (product_pre(mx.out, o.pre, pa, c.y2, c.ldy2, 3)) return 1; }
        advanced(c.y2, c.ldy2, ly.norm1);
        if (!ly.mlp) continue;
        pa.res = residual(nullptr, nullptr, ly.pre2);
        const bool glu = st.d.mlp_act == STACK_ACT_CLAMPED_GLU;
        if (glu && b.rows > BAMD_MV_ROWS) {                        // the product's tiles write the down-projection's operand
            begin(2, 0); bamd_launch_residual_rows(st.act, b, pa.res, s); end();
            begin(4, (double) ly.up.bytes);
            const int rc = bamd_launch_dense_gemm(st.act, ly.up, c.h, pa.res.ldh, b.rows, c.y, ly.down.K, BAMD_OUT_GLU, s, ly.limit);
            end();
            if (rc) return fail("dense product: unsupported shape");
            if (product(ly.down, c.y, ly.down.K, c.y2, c.ldy2, 5)) return 1;
        } else {
            if (product_pre(ly.up, BAMD_PRE_RESIDUAL, pa, c.y, ld_of(ly.up), 4)) return 1;
            if (glu) pa.glu = { c.y, ld_of(ly.up), ly.limit, c.h, ly.down.K };
            else pa.poly = { c.y, ld_of(ly.up), ly.act, st.eps, c.h, ly.F, ly.down.K };
            if (product_pre(ly.down, glu ? BAMD_PRE_GLU : BAMD_PRE_POLY, pa, c.y2, c.ldy2, 5)) return 1;
        }
        advanced(c.y2, c.ldy2, ly.norm2);
    }
    return 0;
}
int Pass::head(const int32_t * want, int n, float * logits) {
    bamd_residual_args a = residual(nullptr, nullptr, nullptr);
    if (fused(st.head) && n == 1) {
        bamd_pre_args pa; memset((void *) &pa, 0, sizeof pa);
        pa.res = a; pa.gf = st.norm_f; pa.want = want;
        begin(6, (double) st.head.bytes);
        const int rc = bamd_launch_dense_mv(st.act, st.head, BAMD_PRE_FINAL, b, &pa, nullptr, 0, 1, logits, st.V, s);
        end();
        return rc ? fail("dense product: unsupported shape") : 0;
    }
    bamd_launch_final_rows(st.act, a, want, n, st.norm_f, s);
    begin(6, (double) st.head.bytes);
    const int rc = bamd_launch_dense_mv(st.act, st.head, BAMD_PRE_ROWS, b, nullptr, c.h, a.ldh, n, logits, st.V, s);
    end();
    return rc ? fail("dense product: unsupported shape") : 0;
}

// a piece of a batch entry in one pass
struct Piece { int seq, n; const int32_t * tokens; };

// fills the step descriptors of a pass and sends them; want: rows of the pass
int send(Pass & p, const std::vector<Piece> & pc, const std::vector<int32_t> & want) {
    Ctx & c = p.c;
    const int r = c.ring; c.ring = (c.ring + 1) % Ctx::RING;
    HIPC(hipEventSynchronize(c.ev[r]));                            // (never recorded yet: returns at once)
    unsigned char * h = c.host[r];
    bamd_entry * ent = (bamd_entry *) (h + c.lay.ent);
    int32_t * row = (int32_t *) (h + c.lay.row), * tok = (int32_t *) (h + c.lay.tok), * kblk = (int32_t *) (h + c.lay.kblk);
    bamd_qtile * tile = (bamd_qtile *) (h + c.lay.tile);
    int rows = 0, kb = 0, nt = 0, tq = 0;
    int scan = 0;
    for (const Layer & ly : p.st.layers) {
        if (const int q = ly.mix->prompt_rows(p.st.act)) tq = tq ? std::min(tq, q) : q;
        scan = std::max(scan, ly.mix->scan_blocks());
    }
    for (size_t e = 0; e < pc.size(); ++e) {
        Seq & q = c.seqs[(size_t) pc[e].seq];
        ent[e] = { pc[e].seq, rows, pc[e].n, q.len, q.par, kb * BAMD_PAGE };
        for (int i = 0; i < pc[e].n; ++i) { row[rows + i] = (int32_t) e; tok[rows + i] = pc[e].tokens ? pc[e].tokens[i] : 0; }
        if (!p.decode) {
            const int blocks = (q.len + pc[e].n + BAMD_PAGE - 1) / BAMD_PAGE;
            for (int i = 0; i < blocks; ++i) kblk[kb + i] = (int32_t) e;
            kb += blocks;
        }
        rows += pc[e].n; p.max_n = std::max(p.max_n, pc[e].n);
    }
    // longest key ranges first: the tail of the launch is short tiles
    if (!p.decode && tq) {
        for (size_t e = 0; e < pc.size(); ++e) for (int q0 = 0; q0 < pc[e].n; q0 += tq) tile[nt++] = { (int32_t) e, q0 };
        std::stable_sort(tile, tile + nt, [&](const bamd_qtile & a, const bamd_qtile & b) { return ent[a.entry].pos0 + a.q0 > ent[b.entry].pos0 + b.q0; });
    }
    // scan segments: as many as fill the chip, none short
    int ns = 0;
    if (!p.decode && scan) {
        const int shortest = std::max(SEG_MIN, (rows + (SEG_BLOCKS + scan - 1) / scan - 1) / ((SEG_BLOCKS + scan - 1) / scan));
        bamd_segment * seg = (bamd_segment *) (h + c.lay.seg);
        for (size_t e = 0; e < pc.size(); ++e) {
            const int n = pc[e].n, k = std::max(1, std::min(n / shortest, n / (2 * SEG_MIN))), len = up((n + k - 1) / k, 8), first = ns;
            for (int t = 0; t < n; t += len) seg[ns++] = { (int32_t) e, t, std::min(len, n - t), first, 0 };
            for (int i = first; i < ns; ++i) seg[i].last = ns - 1;
        }
    }
    memcpy(h + c.lay.want, want.data(), want.size() * 4);
    HIPC(hipMemcpyAsync(c.dev, h, c.lay.total, hipMemcpyHostToDevice, p.s));
    if (c.pages_dirty) {
        for (size_t i = 0; i < c.seqs.size(); ++i) std::copy(c.seqs[i].pages.begin(), c.seqs[i].pages.end(), c.pages_host[r] + i * c.max_pages);
        HIPC(hipMemcpyAsync(c.pages, c.pages_host[r], c.seqs.size() * (size_t) c.max_pages * 4, hipMemcpyHostToDevice, p.s));
        c.pages_dirty = false;
    }
    HIPC(hipEventRecord(c.ev[r], p.s));
    p.b = { (bamd_entry *) (c.dev + c.lay.ent), (int32_t *) (c.dev + c.lay.row), (int32_t *) (c.dev + c.lay.tok), (int) pc.size(), rows, c.c->n_seq, c.pages, c.max_pages };
    p.k_rows = kb * BAMD_PAGE; p.n_tiles = nt; p.n_segs = ns;
    p.x = c.xa; p.xo = c.xb; p.pend = nullptr; p.ldp = 0; p.pend_g = nullptr;
    return 0;
}
int embed(Pass & p) { bamd_launch_embed_rows(p.b, p.st.embd, p.st.pos, p.st.scale, p.st.E, p.st.V, p.x, p.s); return 0; }

// decoding rows -> logits of every row, as a graph (greedy: the loop's token hand-over in front, the arg-max behind)
int decode_rows(Pass & p, bool greedy) {
    Ctx & c = p.c;
    const int n = p.b.rows;
    auto enqueue = [&]() -> int {
        if (greedy) bamd_launch_advance((bamd_entry *) p.b.ent, (int32_t *) p.b.tokens, c.keys, n, c.gen_out, c.gen_cap, c.step, 1, p.st.V, p.s);
        if (embed(p) || p.layers() || p.head((const int32_t *) (c.dev + c.lay.want), n, c.c->logits)) return 1;
        if (greedy) bamd_launch_argmax_rows(c.c->logits, n, p.st.V, c.keys, false, p.s);
        return 0;
    };
    if (!g_graph) return enqueue();
    const int key = n * 2 + (greedy ? 1 : 0);
    auto it = c.graphs.find(key);
    if (it == c.graphs.end()) {
        hipGraph_t g = nullptr; hipGraphExec_t ex = nullptr;
        HIPC(hipStreamBeginCapture(p.s, hipStreamCaptureModeThreadLocal));
        const int rc = enqueue();
        const hipError_t e = hipStreamEndCapture(p.s, &g);
        if (rc || e != hipSuccess) { if (g) hipGraphDestroy(g); return rc ? rc : fail(std::string("hipStreamEndCapture: ") + hipGetErrorString(e)); }
        const hipError_t e2 = hipGraphInstantiate(&ex, g, nullptr, nullptr, 0);
        hipGraphDestroy(g);
        if (e2 != hipSuccess) return fail(std::string("hipGraphInstantiate: ") + hipGetErrorString(e2));
        it = c.graphs.emplace(key, ex).first;
    }
    HIPC(hipGraphLaunch(it->second, p.s));
    return 0;
}
void moved(Ctx & c, const std::vector<Piece> & pc) { for (const Piece & q : pc) { c.seqs[(size_t) q.seq].len += q.n; c.seqs[(size_t) q.seq].par ^= 1; } }

int Stack::decode_batch(bamd_context * bc, const bamd_batch_entry * e, int n, float * logits, bool wait) {
    Ctx & c = ctx_of(bc);
    if (!m->with_embd || !m->with_output) return fail("a batch needs a stage that owns embedding and output");
    HIPC(hipSetDevice(m->device));
    // checks and pages first: a batch either runs or leaves the sequences as they were
    std::vector<char> seen((size_t) bc->n_seq, 0);
    std::vector<size_t> first((size_t) n + 1, 0);
    size_t total = 0, n_want = 0;
    for (int i = 0; i < n; ++i) {
        if (e[i].seq < 0 || e[i].seq >= bc->n_seq || seen[(size_t) e[i].seq]) return fail("batch: sequence out of range, or twice");
        seen[(size_t) e[i].seq] = 1;
        if (e[i].n_tokens < 1 || !e[i].tokens || e[i].n_want < 0 || (e[i].n_want && !e[i].want)) return fail("batch: an entry without tokens");
        for (int k = 0; k < e[i].n_tokens; ++k) if (e[i].tokens[k] < 0 || e[i].tokens[k] >= V) return fail("batch: token id out of range");
        for (int k = 0; k < e[i].n_want; ++k) if (e[i].want[k] < 0 || e[i].want[k] >= e[i].n_tokens || (k && e[i].want[k] <= e[i].want[k - 1])) return fail("batch: wanted places must be ascending places of the entry's tokens");
        const int len = c.seqs[(size_t) e[i].seq].len + e[i].n_tokens;
        if (d.learned_positions && len > max_pos) return fail("context overflow: the model has " + std::to_string(max_pos) + " positions");
        if (len > bc->n_ctx) return fail("context overflow");
        total += (size_t) e[i].n_tokens; first[(size_t) i] = n_want; n_want += (size_t) e[i].n_want;
    }
    if (!total) return 0;
    {
        size_t need = 0;
        for (int i = 0; i < n; ++i) { const Seq & q = c.seqs[(size_t) e[i].seq]; need += (size_t) std::max(0, (q.len + e[i].n_tokens + BAMD_PAGE - 1) / BAMD_PAGE - (int) q.pages.size()); }
        if (need > c.free_pages.size()) return fail("context overflow: no free pages");
        for (int i = 0; i < n; ++i) if (reserve(c, e[i].seq, c.seqs[(size_t) e[i].seq].len + e[i].n_tokens)) return 1;
    }
    // decoding rows together, then the prompts' tokens in passes of at most rows_cap rows
    struct Plan { std::vector<Piece> pc; std::vector<int32_t> want; std::vector<size_t> dst; bool decode; int rows = 0; };
    std::vector<Plan> plans;
    auto add = [&](int i, int from, int cnt, bool dec) {
        if (plans.empty() || plans.back().decode != dec || plans.back().rows >= c.rows_cap) { plans.emplace_back(); plans.back().decode = dec; }
        Plan & pl = plans.back();
        for (int k = 0; k < e[i].n_want; ++k) if (e[i].want[k] >= from && e[i].want[k] < from + cnt) { pl.want.push_back(pl.rows + e[i].want[k] - from); pl.dst.push_back(first[(size_t) i] + (size_t) k); }
        pl.pc.push_back({ e[i].seq, cnt, e[i].tokens + from });
        pl.rows += cnt;
    };
    for (int i = 0; i < n; ++i) if (e[i].n_tokens == 1 && c.seqs[(size_t) e[i].seq].len > 0) add(i, 0, 1, true);
    for (int i = 0; i < n; ++i) if (!(e[i].n_tokens == 1 && c.seqs[(size_t) e[i].seq].len > 0))
        for (int from = 0; from < e[i].n_tokens; ) {
            const int room = plans.empty() || plans.back().decode || plans.back().rows >= c.rows_cap ? c.rows_cap : c.rows_cap - plans.back().rows;
            const int cnt = std::min(room, e[i].n_tokens - from);
            add(i, from, cnt, false);
            from += cnt;
        }
    for (Plan & pl : plans) {
        Pass p{ c, *this, bc->stream, {}, pl.decode };
        const bool graph = pl.decode && pl.rows <= BAMD_LOGIT_ROWS && !pl.want.empty();
        std::vector<int32_t> rows = pl.want;
        if (graph) { rows.resize((size_t) pl.rows); for (int i = 0; i < pl.rows; ++i) rows[(size_t) i] = i; }
        if (send(p, pl.pc, rows)) return 1;
        if (graph) { if (decode_rows(p, false)) return 1; }
        else if (embed(p) || p.layers()) return 1;
        moved(c, pl.pc);
        for (size_t w = 0; w < pl.want.size(); w += BAMD_LOGIT_ROWS) {
            const int k = (int) std::min<size_t>(BAMD_LOGIT_ROWS, pl.want.size() - w);
            if (!graph && p.head((const int32_t *) (c.dev + c.lay.want) + w, k, bc->logits)) return 1;
            if (!logits) continue;                                  // the last rows stay in c->logits
            const int back = graph ? pl.rows : k;
            HIPC(hipMemcpyAsync(bc->logits_host, bc->logits, (size_t) back * V * 4, hipMemcpyDeviceToHost, bc->stream));
            HIPC(hipStreamSynchronize(bc->stream));
            for (int i = 0; i < k; ++i) memcpy(logits + pl.dst[w + (size_t) i] * V, bc->logits_host + (size_t) (graph ? pl.want[w + (size_t) i] : i) * V, (size_t) V * 4);
        }
        HIPC(hipGetLastError());
    }
    if (wait) HIPC(hipStreamSynchronize(bc->stream));
    return 0;
}

int Stack::generate(bamd_context * bc, const int32_t * seqs, int n, int n_steps, const int32_t * first, int32_t * out, float * ms) {
    Ctx & c = ctx_of(bc);
    if (!m->with_embd || !m->with_output) return fail("generation needs a stage that owns embedding and output");
    if (n < 1 || n > BAMD_LOGIT_ROWS || n_steps < 1 || n_steps + 1 > c.gen_cap || (!first && n != 1)) return fail("bad number of sequences or steps");
    HIPC(hipSetDevice(m->device));
    hipStream_t s = bc->stream;
    std::vector<Piece> pc; std::vector<int32_t> want; std::vector<char> seen((size_t) bc->n_seq, 0);
    size_t need = 0;
    for (int i = 0; i < n; ++i) {
        if (seqs[i] < 0 || seqs[i] >= bc->n_seq || seen[(size_t) seqs[i]]) return fail("sequence out of range, or twice");
        seen[(size_t) seqs[i]] = 1;
        const Seq & q = c.seqs[(size_t) seqs[i]];
        if (q.len < 1) return fail("generation behind an empty sequence");
        if (q.len + n_steps > bc->n_ctx || (d.learned_positions && q.len + n_steps > max_pos)) return fail("context overflow");
        need += (size_t) std::max(0, (q.len + n_steps + BAMD_PAGE - 1) / BAMD_PAGE - (int) q.pages.size());
        pc.push_back({ seqs[i], 1, nullptr }); want.push_back(i);
    }
    if (need > c.free_pages.size()) return fail("context overflow: no free pages");
    for (int i = 0; i < n; ++i) if (reserve(c, seqs[i], c.seqs[(size_t) seqs[i]].len + n_steps)) return 1;
    if (first) {
        std::vector<unsigned long long> k((size_t) n);
        for (int i = 0; i < n; ++i) { if (first[i] < 0 || first[i] >= V) return fail("token id out of range"); k[(size_t) i] = 0xffffffffu - (uint32_t) first[i]; }
        HIPC(hipMemcpyAsync(c.keys, k.data(), k.size() * 8, hipMemcpyHostToDevice, s)); HIPC(hipStreamSynchronize(s));
    } else bamd_launch_argmax_rows(bc->logits, 1, V, c.keys, true, s);
    const int32_t zero = 0;
    HIPC(hipMemcpyAsync(c.step, &zero, 4, hipMemcpyHostToDevice, s));
    Pass p{ c, *this, s, {}, true };
    if (send(p, pc, want)) return 1;
    hipEvent_t a = nullptr, b = nullptr;
    HIPC(hipEventCreate(&a));
    if (hipEventCreate(&b) != hipSuccess) { hipEventDestroy(a); return fail("hipEventCreate"); }
    int rc = 0;
    hipEventRecord(a, s);
    for (int t = 0; t < n_steps && !rc; ++t) rc = decode_rows(p, true);
    hipEventRecord(b, s);
    if (!rc) {
        for (const Piece & q : pc) { c.seqs[(size_t) q.seq].len += n_steps; c.seqs[(size_t) q.seq].par ^= n_steps & 1; }
        bamd_launch_advance(nullptr, nullptr, c.keys, n, c.gen_out, c.gen_cap, c.step, 0, V, s);
        if (hipMemcpy2DAsync(out, (size_t) (n_steps + 1) * 4, c.gen_out, (size_t) c.gen_cap * 4, (size_t) (n_steps + 1) * 4, (size_t) n, hipMemcpyDeviceToHost, s) != hipSuccess ||
            hipMemcpyAsync(bc->logits_host, bc->logits, (size_t) n * V * 4, hipMemcpyDeviceToHost, s) != hipSuccess || hipStreamSynchronize(s) != hipSuccess || hipGetLastError() != hipSuccess)
            rc = fail("generation failed on the device");
    }
    if (!rc && ms) hipEventElapsedTime(ms, a, b);
    hipEventDestroy(a); hipEventDestroy(b);
    return rc;
}

int Stack::stage(bamd_context * bc, const int32_t * tokens, const void * token_dev, int n, int n_past, const void * hin, void * hout, bool want_logits, hipStream_t s) {
    Ctx & c = ctx_of(bc);
    HIPC(hipSetDevice(m->device));
    if (n < 1 || n > c.rows_cap) return fail("n_tokens out of range");
    if (n_past == 0) seq_free(bc, 0);
    if (n_past != c.seqs[0].len) return fail("positions cannot be taken back: the sequence holds " + std::to_string(c.seqs[0].len) + " tokens");
    if (n_past + n > bc->n_ctx || (d.learned_positions && n_past + n > max_pos)) return fail("context overflow");
    if ((m->with_embd && !tokens && !token_dev) || (!m->with_embd && !hin) || (!m->with_output && !hout)) return fail("stage: tokens or hidden state missing");
    if (tokens && m->with_embd) for (int i = 0; i < n; ++i) if (tokens[i] < 0 || tokens[i] >= V) return fail("token id out of range");
    if (reserve(c, 0, n_past + n)) return 1;
    Pass p{ c, *this, s, {}, n == 1 && n_past > 0 };
    const std::vector<Piece> pc{ { 0, n, m->with_embd ? tokens : nullptr } };
    if (send(p, pc, { n - 1 })) return 1;
    if (token_dev && m->with_embd) HIPC(hipMemcpyAsync(c.dev + c.lay.tok, token_dev, 4, hipMemcpyDeviceToDevice, s));
    if (m->with_embd) embed(p);
    else HIPC(hipMemcpyAsync(p.x, hin, (size_t) n * E * 4, hipMemcpyDeviceToDevice, s));
    if (p.layers()) return 1;
    moved(c, pc);
    if (!m->with_output) {
        bamd_residual_args a = p.residual(nullptr, nullptr, nullptr);
        a.xo = (float *) hout; a.h = nullptr;
        bamd_launch_residual_rows(act, p.b, a, s);
    } else if (want_logits) {
        if (p.head((const int32_t *) (c.dev + c.lay.want), 1, bc->logits)) return 1;
        bc->logits_host_valid = false;
    }
    HIPC(hipGetLastError());
    return 0;
}
int Stack::argmax_to(bamd_context * bc, int32_t * token_dev, hipStream_t s) {
    Ctx & c = ctx_of(bc);
    HIPC(hipSetDevice(m->device));
    bamd_launch_argmax_rows(bc->logits, 1, V, c.keys, true, s);
    bamd_launch_advance(nullptr, token_dev, c.keys, 1, nullptr, 0, nullptr, 0, V, s);
    HIPC(hipGetLastError());
    return 0;
}
int Stack::profile_kinds(bamd_context * bc, int pos, int * launches, double * ms, double * bytes) {
    Ctx & c = ctx_of(bc);
    HIPC(hipSetDevice(m->device));
    if (pos != c.seqs[0].len || pos < 1) return fail("the profiled step continues sequence 0: pos must be its length");
    if (reserve(c, 0, pos + 1)) return 1;
    Timer tm;
    Pass p{ c, *this, bc->stream, {}, true };
    p.tm = &tm;
    const int32_t tok = 1;
    const std::vector<Piece> pc{ { 0, 1, &tok } };
    if (send(p, pc, { 0 })) return 1;
    p.begin(2, 0); embed(p); p.end();
    if (p.layers() || p.head((const int32_t *) (c.dev + c.lay.want), 1, bc->logits)) return 1;
    for (int i = 0; i < 9; ++i) { p.begin(7, 0); p.end(); }
    moved(c, pc);
    HIPC(hipStreamSynchronize(bc->stream));
    for (int i = 0; i < 8; ++i) { launches[i] = 0; ms[i] = 0; bytes[i] = 0; }
    std::vector<float> empty;
    for (size_t i = 0; i < tm.kind.size(); ++i) {
        float t = 0.f; hipEventElapsedTime(&t, tm.ev[2 * i], tm.ev[2 * i + 1]);
        if (tm.kind[i] == 7) { empty.push_back(t); continue; }
        launches[tm.kind[i]] += 1; ms[tm.kind[i]] += t; bytes[tm.kind[i]] += tm.bytes[i];
    }
    std::sort(empty.begin(), empty.end());
    launches[7] = 1; ms[7] = empty[empty.size() / 2];
    return 0;
}
}  // namespace

int bamd_stack_load(bamd_model * m, const bamd_load_args & a, const bamd_arch & self) {
    Stack * st = new Stack();
    m->rt.reset(st);
    return st->load(m, a, *(const bamd_stack_design *) self.design);
}

// ---- op-level entry points (tests call the kernels through these; host pointers in, host out; activation rows cross as f32) -------------------------------
namespace {
struct OpScratch {                                 // device copies of one call
    bamd_model m; Loader l; std::vector<void *> & keep = m.allocs;
    ~OpScratch() { hipDeviceSynchronize(); for (void * p : keep) hipFree(p); }
    int init(int act) {
        if (act != BAMD_ACT_BF16 && act != BAMD_ACT_F32) return fail("act: 0 bfloat16, 1 float");
        if (bamd_device_count() <= 0) return fail("no HIP device available: libbooster_amd has no CPU fallback");
        l.m = &m; l.act = act;
        HIPC(hipStreamCreate(&l.s));
        return 0;
    }
    int alloc(void ** p, size_t bytes) { if (dev_alloc(keep, p, std::max<size_t>(bytes, 16))) return 1; HIPC(hipMemset(*p, 0, std::max<size_t>(bytes, 16))); return 0; }
    template <typename U> int up_(const U * h, size_t n, U ** d) { if (alloc((void **) d, n * sizeof(U))) return 1; if (n) HIPC(hipMemcpy(*d, h, n * sizeof(U), hipMemcpyHostToDevice)); return 0; }
    // f32 host rows [rows][n] -> activation rows [rows][ld]
    int act_rows(const float * h, int rows, int n, int ld, void ** d) {
        const bool f = l.act == BAMD_ACT_F32;
        std::vector<unsigned char> b((size_t) rows * ld * (f ? 4 : 2), 0);
        for (int r = 0; r < rows; ++r) for (int i = 0; i < n; ++i) {
            const float v = h[(size_t) r * n + i];
            if (f) memcpy(&b[((size_t) r * ld + i) * 4], &v, 4);
            else { uint32_t u; memcpy(&u, &v, 4); u += 0x7fff + ((u >> 16) & 1); const uint16_t o = (uint16_t) (u >> 16); memcpy(&b[((size_t) r * ld + i) * 2], &o, 2); }
        }
        if (alloc(d, b.size())) return 1;
        HIPC(hipMemcpy(*d, b.data(), b.size(), hipMemcpyHostToDevice));
        return 0;
    }
    int rows_back(const void * d, int rows, int n, int ld, float * h, bool f) {
        std::vector<unsigned char> b((size_t) rows * ld * (f ? 4 : 2));
        HIPC(hipStreamSynchronize(l.s));
        HIPC(hipMemcpy(b.data(), d, b.size(), hipMemcpyDeviceToHost));
        for (int r = 0; r < rows; ++r) for (int i = 0; i < n; ++i) {
            if (f) memcpy(&h[(size_t) r * n + i], &b[((size_t) r * ld + i) * 4], 4);
            else { uint16_t o; memcpy(&o, &b[((size_t) r * ld + i) * 2], 2); const uint32_t u = (uint32_t) o << 16; memcpy(&h[(size_t) r * n + i], &u, 4); }
        }
        return 0;
    }
    int one_entry(int rows, int pos0, bamd_batch_dev & b) {
        const bamd_entry e = { 0, 0, rows, pos0, 0, 0 };
        bamd_entry * de; int32_t * re, * tk, * pg;
        std::vector<int32_t> z((size_t) rows, 0), pages;
        const int n_pg = (pos0 + rows + BAMD_PAGE - 1) / BAMD_PAGE;
        for (int i = 0; i < n_pg; ++i) pages.push_back(n_pg - 1 - i);            // backwards: the order of pages must not matter
        if (up_(&e, 1, &de) || up_(z.data(), z.size(), &re) || up_(z.data(), z.size(), &tk) || up_(pages.data(), pages.size(), &pg)) return 1;
        b = { de, re, tk, 1, rows, 1, pg, n_pg };
        return 0;
    }
};
SafeTensor bf16_tensor(const uint16_t * p, std::vector<int64_t> shape) { SafeTensor t; t.dtype = "BF16"; t.shape = shape; t.data = (const uint8_t *) p; t.nbytes = (size_t) t.count() * 2; return t; }
}  // namespace
#define BAMD_OP extern "C" __attribute__((visibility("default"))) int

BAMD_OP bamd_op_dense(int act, const uint16_t * w, int nrows, int k, const float * x, int rows, int impl, float * y) {
    OpScratch s; bamd_dense d; void * dx; float * dy = nullptr;
    if (!w || !x || !y || nrows < 1 || k < 1 || rows < 1 || s.init(act)) return fail("bamd_op_dense: bad arguments");
    const SafeTensor t = bf16_tensor(w, { nrows, k });
    if (s.l.alloc(d, nrows, k) || s.l.pack(&t, Loader::steps(nrows, k), Loader::steps(k, 1), const_cast<uint16_t *>(d.w)) || s.act_rows(x, rows, k, d.K, &dx)) return 1;
    const int ldo = impl == 3 ? up(rows, 64) : ld_of(d);
    if (s.alloc((void **) &dy, (size_t) (impl == 3 ? ld_of(d) : rows) * ldo * 4)) return 1;
    bamd_batch_dev b; memset((void *) &b, 0, sizeof b);
    int rc;
    if (impl == 1) rc = bamd_launch_dense_mv(act, d, BAMD_PRE_ROWS, b, nullptr, dx, d.K, rows, dy, ldo, s.l.s);
    else rc = bamd_launch_dense_gemm(act, d, dx, d.K, rows, dy, ldo, impl == 0 ? BAMD_OUT_F32 : impl == 2 ? BAMD_OUT_ACT : BAMD_OUT_ACT_T, s.l.s);
    if (rc) return fail("bamd_op_dense: unsupported shape");
    HIPC(hipGetLastError());
    if (impl != 3) return s.rows_back(dy, rows, nrows, ldo, y, impl != 2 || act == BAMD_ACT_F32);
    std::vector<float> tr((size_t) nrows * rows);
    if (s.rows_back(dy, nrows, rows, ldo, tr.data(), act == BAMD_ACT_F32)) return 1;
    for (int n = 0; n < nrows; ++n) for (int r = 0; r < rows; ++r) y[(size_t) r * nrows + n] = tr[(size_t) n * rows + r];
    return 0;
}
BAMD_OP bamd_op_residual_rows(int act, const float * x, const float * y, float g, float eps, const float * mu, float * prev, int pos0, int rows, int E, float * xo, float * h) {
    OpScratch s; bamd_batch_dev b; bamd_residual_args a; memset((void *) &a, 0, sizeof a);
    if (!x || !xo || !h || rows < 1 || E < 1 || (mu && !prev) || s.init(act) || s.one_entry(rows, pos0, b)) return fail("bamd_op_residual_rows: bad arguments");
    const size_t n = (size_t) rows * E;
    float * dx, * dy = nullptr, * dg, * dmu = nullptr, * dp = nullptr, * dxo; void * dh;
    if (s.up_(x, n, &dx) || (y && s.up_(y, n, &dy)) || s.up_(&g, 1, &dg) || (mu && (s.up_(mu, (size_t) E, &dmu) || s.alloc((void **) &dp, (size_t) 8 * E))) || s.alloc((void **) &dxo, n * 4) || s.alloc(&dh, (size_t) rows * up(E, 32) * 4)) return 1;
    if (mu) HIPC(hipMemcpy(dp, prev, (size_t) E * 4, hipMemcpyHostToDevice));
    a.x = dx; a.y = dy; a.ldy = E; a.g = dg; a.eps = eps; a.mu = dmu; a.prev = dp; a.xo = dxo; a.h = dh; a.E = E; a.ldh = up(E, 32);
    bamd_launch_residual_rows(act, b, a, s.l.s);
    HIPC(hipGetLastError());
    if (s.rows_back(dxo, rows, E, E, xo, true) || s.rows_back(dh, rows, E, a.ldh, h, act == BAMD_ACT_F32)) return 1;
    if (mu) HIPC(hipMemcpy(prev, dp + E, (size_t) E * 4, hipMemcpyDeviceToHost));
    return 0;
}
BAMD_OP bamd_op_poly_norm(int act, const float * z, const float * coef, float eps, int rows, int F, float * out) {
    OpScratch s; float * dz, * dc; void * dh;
    if (!z || !coef || !out || rows < 1 || F < 1 || s.init(act) || s.up_(z, (size_t) rows * F, &dz) || s.up_(coef, 4, &dc) || s.alloc(&dh, (size_t) rows * up(F, 32) * 4)) return fail("bamd_op_poly_norm: bad arguments");
    bamd_launch_poly_rows(act, rows, { dz, F, dc, eps, dh, F, up(F, 32) }, s.l.s);
    HIPC(hipGetLastError());
    return s.rows_back(dh, rows, F, up(F, 32), out, act == BAMD_ACT_F32);
}
BAMD_OP bamd_op_group_norm(int act, const float * y, const float * w, int groups, float eps, int rows, int n, float * out) {
    OpScratch s; float * dy, * dw; void * dh;
    if (!y || !w || !out || rows < 1 || n < 1 || groups < 1 || groups > BAMD_MAX_NORM_GROUPS || n % groups || s.init(act) || s.up_(y, (size_t) rows * n, &dy) || s.up_(w, (size_t) n, &dw) || s.alloc(&dh, (size_t) rows * up(n, 32) * 4)) return fail("bamd_op_group_norm: bad arguments");
    bamd_launch_group_norm_rows(act, rows, { dy, n, dw, groups, eps, dh, n, up(n, 32) }, s.l.s);
    HIPC(hipGetLastError());
    return s.rows_back(dh, rows, n, up(n, 32), out, act == BAMD_ACT_F32);
}
BAMD_OP bamd_op_ssm(const float * in, int rows, int pos0, int heads, int P, int N, int groups, int taps, const float * conv, const float * conv_b, const float * dt_bias, const float * A_log, const float * D,
                    float * hist, float * state, float * out) {
    OpScratch s; bamd_batch_dev b; bamd_ssm_args a; memset((void *) &a, 0, sizeof a);
    if (!in || !out || rows < 1 || heads < 1 || P < 1 || N < 1 || groups < 1 || heads % groups || taps < 1 || s.init(BAMD_ACT_F32) || s.one_entry(rows, pos0, b)) return fail("bamd_op_ssm: bad arguments");
    const int inner = heads * P, ch = inner + 2 * groups * N, ld = inner + ch + heads;
    const size_t hn = (size_t) (taps - 1) * ch, sn = (size_t) heads * N * P;
    float * din, * dc, * dcb, * ddt, * dA, * dD, * dh, * ds, * dout;
    if (s.up_(in, (size_t) rows * ld, &din) || s.up_(conv, (size_t) ch * taps, &dc) || s.up_(conv_b, (size_t) ch, &dcb) || s.up_(dt_bias, (size_t) heads, &ddt) || s.up_(A_log, (size_t) heads, &dA) || s.up_(D, (size_t) heads, &dD) ||
        s.alloc((void **) &dh, hn * 8) || s.up_(state, sn, &ds) || s.alloc((void **) &dout, (size_t) rows * inner * 4)) return 1;
    HIPC(hipMemcpy(dh, hist, hn * 4, hipMemcpyHostToDevice));
    a.in = din; a.ld = ld; a.conv = dc; a.conv_b = dcb; a.dt_bias = ddt; a.A_log = dA; a.D = dD; a.hist = dh; a.state = ds; a.out = dout; a.ldo = inner; a.heads = heads; a.P = P; a.N = N; a.groups = groups; a.taps = taps;
    if (s.alloc((void **) &a.filtered, (size_t) rows * ch * 4) || s.alloc((void **) &a.steps, (size_t) rows * heads * 8)) return 1;
    if (bamd_launch_ssm(b, a, rows, s.l.s)) return fail("bamd_op_ssm: unsupported shape");
    HIPC(hipGetLastError());
    if (s.rows_back(dout, rows, inner, inner, out, true)) return 1;
    HIPC(hipMemcpy(hist, dh + hn, hn * 4, hipMemcpyDeviceToHost)); HIPC(hipMemcpy(state, ds, sn * 4, hipMemcpyDeviceToHost));
    return 0;
}
BAMD_OP bamd_op_latent_attention(int act, const float * q, const float * c, const float * gate, int rows, const float * past, int pos0, int heads, int dim, int vdim, int rank, float scale, float eps,
                                 const float * c_norm, const uint16_t * uk, const uint16_t * uv, const float * sink, int decode, float * out) {
    OpScratch s; bamd_batch_dev b; bamd_latent_args a; memset((void *) &a, 0, sizeof a);
    if (!q || !c || !c_norm || !uk || !uv || !out || rows < 1 || pos0 < 0 || (pos0 && !past) || heads < 1 || dim < 1 || dim > 256 || vdim < 1 || vdim > 256 || rank < 1 || rank > 1024 || (decode && rows != 1) || s.init(act) || s.one_entry(rows, pos0, b))
        return fail("bamd_op_latent_attention: bad arguments");
    int D = 32; while (D < std::max(dim, vdim)) D *= 2;
    const int Rp = up(rank, 32), HD = heads * D, g_off = HD + up(rank, 16), ld = up(g_off + heads, 16), len = pos0 + rows, kr = up(len, BAMD_PAGE), hp = up(heads, 16);
    std::vector<float> in((size_t) rows * ld, 0.f);
    for (int r = 0; r < rows; ++r) {
        for (int h = 0; h < heads; ++h) for (int i = 0; i < dim; ++i) in[(size_t) r * ld + h * D + i] = q[((size_t) r * heads + h) * dim + i];
        for (int i = 0; i < rank; ++i) in[(size_t) r * ld + HD + i] = c[(size_t) r * rank + i];
        for (int h = 0; h < heads && gate; ++h) in[(size_t) r * ld + g_off + h] = gate[(size_t) r * heads + h];
    }
    const SafeTensor tk = bf16_tensor(uk, { heads * dim, rank }), tv = bf16_tensor(uv, { heads * vdim, rank });
    float * din, * dn, * dsink = nullptr, * po, * pm; void * cache, * qp, * o, * kc, * kk, * kv; uint16_t * ukT; bamd_qtile * tiles; int32_t * kblk;
    const int n_pg = kr / BAMD_PAGE, splits = std::min(n_pg, 3), tq = bamd_latent_prompt_rows(act, D);
    if (s.up_(in.data(), in.size(), &din) || s.up_(c_norm, (size_t) rank, &dn) || (sink && s.up_(sink, (size_t) heads, &dsink)) || s.alloc(&o, (size_t) rows * HD * 4) || s.alloc(&qp, (size_t) hp * Rp * 4) ||
        s.alloc((void **) &po, (size_t) hp * splits * Rp * 4) || s.alloc((void **) &pm, (size_t) hp * splits * 8) || s.alloc(&kc, (size_t) kr * Rp * 4) || s.alloc(&kk, (size_t) kr * HD * 4) || s.alloc(&kv, (size_t) kr * HD * 4)) return 1;
    // the cache in front: page i of the sequence lies at place n_pg - 1 - i
    std::vector<float> flat((size_t) n_pg * BAMD_PAGE * rank, 0.f);
    for (int p = 0; p < pos0; ++p) memcpy(&flat[((size_t) (n_pg - 1 - p / BAMD_PAGE) * BAMD_PAGE + p % BAMD_PAGE) * rank], past + (size_t) p * rank, (size_t) rank * 4);
    if (s.act_rows(flat.data(), n_pg * BAMD_PAGE, rank, Rp, &cache)) return 1;
    if (s.l.alloc(a.uk, HD, rank) || s.l.pack(&tk, Loader::grouped(heads, dim, D, rank), Loader::steps(rank, 1), const_cast<uint16_t *>(a.uk.w)) ||
        s.l.alloc(a.uv, HD, rank) || s.l.pack(&tv, Loader::grouped(heads, vdim, D, rank), Loader::steps(rank, 1), const_cast<uint16_t *>(a.uv.w)) || s.alloc((void **) &ukT, (size_t) heads * Rp * D * 2)) return 1;
    std::vector<int32_t> rr = Loader::steps(rank, 1); rr.resize((size_t) Rp, -1);
    for (int h = 0; h < heads; ++h) {
        std::vector<int32_t> cc((size_t) D, -1);
        for (int i = 0; i < dim; ++i) cc[(size_t) i] = (h * dim + i) * rank;
        if (s.l.pack(&tk, rr, cc, ukT + (size_t) h * Rp * D)) return 1;
    }
    std::vector<bamd_qtile> t; for (int q0 = 0; q0 < rows; q0 += tq) t.push_back({ 0, q0 });
    std::vector<int32_t> kb((size_t) n_pg, 0);
    if (s.up_(t.data(), t.size(), &tiles) || s.up_(kb.data(), kb.size(), &kblk)) return 1;
    a.in = din; a.ld = ld; a.c_off = HD; a.g_off = g_off; a.c_norm = dn; a.eps = eps; a.scale = scale; a.sink = dsink; a.gated = gate ? 1 : 0; a.heads = heads; a.D = D; a.R = rank; a.Rp = Rp; a.cache = cache; a.ukT = ukT; a.out = o; a.ldo = HD;
    int rc;
    if (decode) rc = bamd_launch_latent_decode(act, b, a, qp, po, pm, splits, s.l.s);
    else {
        bamd_launch_latent_store(act, b, a, s.l.s);
        bamd_launch_latent_gather(act, b, a, kblk, kr, kc, s.l.s);
        rc = bamd_launch_dense_gemm(act, a.uk, kc, Rp, kr, kk, HD, BAMD_OUT_ACT, s.l.s) || bamd_launch_dense_gemm(act, a.uv, kc, Rp, kr, kv, kr, BAMD_OUT_ACT_T, s.l.s) ||
             bamd_launch_latent_prompt(act, b, a, tiles, (int) t.size(), kk, kv, kr, s.l.s);
    }
    if (rc) return fail("bamd_op_latent_attention: unsupported shape");
    HIPC(hipGetLastError());
    std::vector<float> wide((size_t) rows * HD);
    if (s.rows_back(o, rows, HD, HD, wide.data(), act == BAMD_ACT_F32)) return 1;
    for (int r = 0; r < rows; ++r) for (int h = 0; h < heads; ++h) memcpy(out + ((size_t) r * heads + h) * vdim, &wide[(size_t) r * HD + h * D], (size_t) vdim * 4);
    return 0;
}
BAMD_OP bamd_op_layer_rows(int act, const float * x, const float * y, const float * g, const float * gi, float eps, int rows, int E, float * xo, float * h) {
    OpScratch s; bamd_batch_dev b; bamd_residual_args a; memset(&a, 0, sizeof a);
    if (!x || !xo || !h || (y && !g) || rows < 1 || E < 1 || s.init(act) || s.one_entry(rows, 0, b)) return fail("bamd_op_layer_rows: bad arguments");
    const size_t n = (size_t) rows * E;
    float * dx, * dy = nullptr, * dg = nullptr, * di = nullptr, * dxo; void * dh;
    if (s.up_(x, n, &dx) || (y && (s.up_(y, n, &dy) || s.up_(g, (size_t) E, &dg))) || (gi && s.up_(gi, (size_t) E, &di)) || s.alloc((void **) &dxo, n * 4) || s.alloc(&dh, (size_t) rows * up(E, 32) * 4)) return 1;
    a.norm = BAMD_NORM_LAYER; a.x = dx; a.y = dy; a.ldy = E; a.g = dg; a.gi = di; a.eps = eps; a.xo = dxo; a.h = dh; a.E = E; a.ldh = up(E, 32);
    bamd_launch_residual_rows(act, b, a, s.l.s);
    HIPC(hipGetLastError());
    return s.rows_back(dxo, rows, E, E, xo, true) || s.rows_back(dh, rows, E, a.ldh, h, act == BAMD_ACT_F32);
}
BAMD_OP bamd_op_clamped_glu(int act, const float * gate, const float * upv, float limit, int rows, int F, float * out) {
    OpScratch s; float * dz; void * dh;
    if (!gate || !upv || !out || rows < 1 || F < 1 || s.init(act)) return fail("bamd_op_clamped_glu: bad arguments");
    const int ldh = up(F, 32);
    std::vector<float> z((size_t) rows * 2 * ldh, 0.f);
    for (int r = 0; r < rows; ++r) for (int i = 0; i < F; ++i) { float * p = &z[(size_t) r * 2 * ldh + (i / 16) * 32 + i % 16]; p[0] = gate[(size_t) r * F + i]; p[16] = upv[(size_t) r * F + i]; }
    if (s.up_(z.data(), z.size(), &dz) || s.alloc(&dh, (size_t) rows * ldh * 4)) return 1;
    bamd_launch_glu_rows(act, rows, { dz, 2 * ldh, limit, dh, ldh }, s.l.s);
    HIPC(hipGetLastError());
    return s.rows_back(dh, rows, F, ldh, out, act == BAMD_ACT_F32);
}
// past_k, past_v: what the cache holds in front of the rows (keys as they are cached), [pos0][kv_heads][dim / vdim]; rel: [rel_rows][heads] or null; splits: shares of a decoded row
BAMD_OP bamd_op_kv_attention(int act, const float * q, const float * k, const float * v, const float * gate, int rows, const float * past_k, const float * past_v, int pos0, int heads, int kv_heads, int dim, int vdim,
                             float scale, float cap, float eps, int unit, const float * rel, int rel_rows, int bias_max, int window, int keep, float out_scale, int splits, float * out) {
    OpScratch s; bamd_batch_dev b; bamd_kv_args a; memset((void *) &a, 0, sizeof a);
    if (!q || !k || !v || !out || rows < 1 || pos0 < 0 || (pos0 && (!past_k || !past_v)) || heads < 1 || kv_heads < 1 || heads % kv_heads || dim < 1 || dim > 256 || vdim < 1 || vdim > 256 || window < 1 || keep < 0 || splits > 64 ||
        (splits && rows != 1) || (rel && (rel_rows < 2 || bias_max <= rel_rows / 2)) || s.init(act) || s.one_entry(rows, pos0, b)) return fail("bamd_op_kv_attention: bad arguments");
    int D = 32; while (D < std::max(dim, vdim)) D *= 2;
    const int H = heads, G = kv_heads, ld = up((H + 2 * G) * D + H, 16), kr = up(pos0 + rows, BAMD_PAGE), n_pg = kr / BAMD_PAGE, tq = bamd_kv_prompt_rows(act, D);
    a.ld = ld; a.q_off = 0; a.k_off = H * D; a.v_off = (H + G) * D; a.g_off = (H + 2 * G) * D; a.heads = H; a.kv_heads = G; a.D = D; a.dim = dim; a.eps = eps; a.scale = scale; a.cap = cap; a.unit = unit; a.gated = gate ? 1 : 0;
    a.window = window; a.keep = keep; a.out_scale = out_scale; a.ldo = H * D;
    std::vector<float> in((size_t) rows * ld, 0.f), fk((size_t) kr * G * D, 0.f), fv((size_t) kr * G * D, 3.f);      // (whatever lies behind the past must not matter)
    for (int r = 0; r < rows; ++r) {
        float * p = &in[(size_t) r * ld];
        for (int h = 0; h < H; ++h) { memcpy(p + h * D, q + ((size_t) r * H + h) * dim, (size_t) dim * 4); if (gate) p[a.g_off + h] = gate[(size_t) r * H + h]; }
        for (int g = 0; g < G; ++g) { memcpy(p + a.k_off + g * D, k + ((size_t) r * G + g) * dim, (size_t) dim * 4); memcpy(p + a.v_off + g * D, v + ((size_t) r * G + g) * vdim, (size_t) vdim * 4); }
    }
    // page i of the sequence lies at place n_pg - 1 - i
    for (int p = 0; p < pos0; ++p) for (int g = 0; g < G; ++g) {
        const size_t at = ((size_t) (n_pg - 1 - p / BAMD_PAGE) * G + g) * BAMD_PAGE * D;
        for (int i = 0; i < dim; ++i) fk[at + (size_t) (p % BAMD_PAGE) * D + i] = past_k[((size_t) p * G + g) * dim + i];
        for (int i = 0; i < D; ++i) fv[at + (size_t) i * BAMD_PAGE + p % BAMD_PAGE] = i < vdim ? past_v[((size_t) p * G + g) * vdim + i] : 0.f;
    }
    float * din, * po, * pm, * db = nullptr; bamd_qtile * tiles; int32_t * kblk; void * o;
    std::vector<bamd_qtile> t; for (int q0 = 0; q0 < rows; q0 += tq) t.push_back({ 0, q0 });
    std::vector<int32_t> kb((size_t) n_pg, 0);
    if (rel) { a.bias_top = bias_max; const std::vector<float> e = expand_bias(std::vector<float>(rel, rel + (size_t) rel_rows * H), rel_rows, H, bias_max); if (s.up_(e.data(), e.size(), &db)) return 1; }
    const size_t cells = (size_t) bamd_kv_groups(a) * std::max(splits, 1);
    if (s.up_(in.data(), in.size(), &din) || s.act_rows(fk.data(), kr, G * D, G * D, &a.kc) || s.act_rows(fv.data(), kr, G * D, G * D, &a.vc) || s.up_(t.data(), t.size(), &tiles) || s.up_(kb.data(), kb.size(), &kblk) ||
        s.alloc(&o, (size_t) rows * H * D * 4) || s.alloc((void **) &po, cells * 16 * D * 4) || s.alloc((void **) &pm, cells * 128)) return 1;
    a.in = din; a.bias = db; a.out = o;
    int rc;
    if (splits) rc = bamd_launch_kv_decode(act, b, a, po, pm, splits, s.l.s);
    else { bamd_launch_kv_store(act, b, a, kblk, kr, s.l.s); rc = bamd_launch_kv_prompt(act, b, a, tiles, (int) t.size(), s.l.s); }
    if (rc) return fail("bamd_op_kv_attention: unsupported shape");
    HIPC(hipGetLastError());
    std::vector<float> wide((size_t) rows * H * D);
    if (s.rows_back(o, rows, H * D, H * D, wide.data(), act == BAMD_ACT_F32)) return 1;
    for (int r = 0; r < rows; ++r) for (int h = 0; h < H; ++h) memcpy(out + ((size_t) r * H + h) * vdim, &wide[((size_t) r * H + h) * D], (size_t) vdim * 4);
    return 0;
}
// q, k [rows][heads][dim], v, gate [rows][heads][vdim], low [rows][rank], a2 bfloat16 [heads * dim][rank]; state [heads][dim][vdim]; segment: tokens per scan segment (0: one).
// y: outputs of the recurrence, out: normed and gated
BAMD_OP bamd_op_gated_linear(int act, const float * q, const float * k, const float * v, const float * gate, const float * low, const uint16_t * a2, const float * a2b, const float * norm, int rows, int pos0, int heads, int dim,
                             int vdim, int rank, float tau, float q_scale, float eps, float out_scale, int segment, float * state, float * y, float * out) {
    OpScratch s; bamd_batch_dev b; bamd_gla_args a; memset((void *) &a, 0, sizeof a);
    if (!q || !k || !v || !low || !a2 || !a2b || !norm || !state || !y || !out || rows < 1 || heads < 1 || dim < 1 || dim > 256 || vdim < 1 || rank < 1 || rank > 1024 || segment < 0 || s.init(act) || s.one_entry(rows, pos0, b))
        return fail("bamd_op_gated_linear: bad arguments");
    const int H = heads, Np = up(dim, 4), Pp = up(vdim, 4), ch = H * Np;
    a.q_off = 0; a.k_off = ch; a.v_off = 2 * ch; a.g_off = a.v_off + H * Pp; a.t_off = a.g_off + H * Pp; a.ld = up(a.t_off + rank, 16); a.rank = rank; a.inv_tau = 1.f / tau; a.q_scale = q_scale; a.ldy = H * Pp;
    a.heads = H; a.Np = Np; a.Pp = Pp; a.P = vdim; a.eps = eps; a.out_cols = up(H * Pp, 32); a.ldo = a.out_cols;
    std::vector<float> in((size_t) rows * a.ld, 0.f), st((size_t) ch * Pp, 0.f), bias((size_t) ch, 0.f), nm((size_t) Pp, 0.f);
    std::vector<uint16_t> w((size_t) rank * ch, 0);
    for (int r = 0; r < rows; ++r) {
        float * p = &in[(size_t) r * a.ld];
        for (int h = 0; h < H; ++h) {
            memcpy(p + h * Np, q + ((size_t) r * H + h) * dim, (size_t) dim * 4); memcpy(p + a.k_off + h * Np, k + ((size_t) r * H + h) * dim, (size_t) dim * 4); memcpy(p + a.v_off + h * Pp, v + ((size_t) r * H + h) * vdim, (size_t) vdim * 4);
            if (gate) memcpy(p + a.g_off + h * Pp, gate + ((size_t) r * H + h) * vdim, (size_t) vdim * 4);
        }
        memcpy(p + a.t_off, low + (size_t) r * rank, (size_t) rank * 4);
    }
    if (!gate) a.g_off = -1;
    for (int h = 0; h < H; ++h) for (int i = 0; i < dim; ++i) {
        bias[(size_t) h * Np + i] = a2b[h * dim + i];
        for (int r = 0; r < rank; ++r) w[(size_t) r * ch + h * Np + i] = a2[((size_t) h * dim + i) * rank + r];
        memcpy(&st[((size_t) h * Np + i) * Pp], state + ((size_t) h * dim + i) * vdim, (size_t) vdim * 4);
    }
    for (int i = 0; i < vdim; ++i) nm[(size_t) i] = norm[i] * out_scale;
    std::vector<bamd_segment> seg;
    const int len = segment ? segment : rows;
    for (int t = 0; t < rows; t += len) seg.push_back({ 0, t, std::min(len, rows - t), 0, 0 });
    for (bamd_segment & g : seg) g.last = (int) seg.size() - 1;
    float * din, * ds, * db, * dn, * dy; uint16_t * dw; bamd_segment * dseg; void * o;
    if (s.up_(in.data(), in.size(), &din) || s.up_(st.data(), st.size(), &ds) || s.up_(bias.data(), bias.size(), &db) || s.up_(nm.data(), nm.size(), &dn) || s.up_(w.data(), w.size(), &dw) || s.up_(seg.data(), seg.size(), &dseg) ||
        s.alloc((void **) &dy, (size_t) rows * H * Pp * 4) || s.alloc(&o, (size_t) rows * a.ldo * 4) || s.alloc((void **) &a.alpha, (size_t) rows * ch * 4) || s.alloc((void **) &a.seg_state, seg.size() * ch * Pp * 4) ||
        s.alloc((void **) &a.seg_decay, seg.size() * ch * 4)) return 1;
    a.in = din; a.a2 = dw; a.a2b = db; a.norm = dn; a.state = ds; a.y = dy; a.out = o;
    if (bamd_launch_gla(b, a, rows, dseg, (int) seg.size(), s.l.s)) return fail("bamd_op_gated_linear: unsupported shape");
    bamd_launch_gla_norm(act, a, rows, s.l.s);
    HIPC(hipGetLastError());
    std::vector<float> wy((size_t) rows * H * Pp), wo(wy.size());
    if (s.rows_back(dy, rows, H * Pp, H * Pp, wy.data(), true) || s.rows_back(o, rows, H * Pp, a.ldo, wo.data(), act == BAMD_ACT_F32)) return 1;
    HIPC(hipMemcpy(st.data(), ds, st.size() * 4, hipMemcpyDeviceToHost));
    for (int r = 0; r < rows; ++r) for (int h = 0; h < H; ++h) {
        memcpy(y + ((size_t) r * H + h) * vdim, &wy[((size_t) r * H + h) * Pp], (size_t) vdim * 4);
        memcpy(out + ((size_t) r * H + h) * vdim, &wo[((size_t) r * H + h) * Pp], (size_t) vdim * 4);
    }
    for (int h = 0; h < H; ++h) for (int i = 0; i < dim; ++i) memcpy(state + ((size_t) h * dim + i) * vdim, &st[((size_t) h * Np + i) * Pp], (size_t) vdim * 4);
    return 0;
}
