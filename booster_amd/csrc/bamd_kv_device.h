// bamd_kv_device.h — decoding side of the attention over cached keys and values (bamd_kv.hip) as device functions: one block's share of the keys, and the sum over the shares
#pragma once
#include "bamd_dense_device.h"

#define KV_LOG2E 1.4426950408889634f

// a score in front of the softmax, times log2(e): capped, then biased
struct KvCap { float pre, cap2; bool on; };
__device__ __forceinline__ KvCap kv_cap(const bamd_kv_args & a) { return a.cap > 0.f ? KvCap{ a.scale / a.cap, a.cap * KV_LOG2E, true } : KvCap{ a.scale * KV_LOG2E, 0.f, false }; }
template <typename T> __device__ __forceinline__ float kv_score(float s, const KvCap & c, float bias2) {
    const float x = s * c.pre;
    if (!c.on) return x + bias2;
    if constexpr (sizeof(T) == 4) return c.cap2 * tanhf(x) + bias2;
    // cap tanh(x) = cap - 2 cap / (1 + exp(2 x))
    return fmaf(-2.0f * c.cap2, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(2.0f * KV_LOG2E * x)), c.cap2 + bias2);
}
__device__ __forceinline__ float kv_bias(const bamd_kv_args & a, int h, int dist) { return a.bias ? a.bias[(size_t) h * (a.bias_top + 1) + min(dist, a.bias_top)] * KV_LOG2E : 0.f; }
// pages a range of queries reads: the kept ones first, then those of the window.  wlo: first position of the window of the lowest query
struct KvPages {
    int kept, first, count;
    __device__ __forceinline__ KvPages(const bamd_kv_args & a, int wlo, int n_pages) {
        kept = min((a.keep + BAMD_PAGE - 1) / BAMD_PAGE, n_pages);
        first = max(max(wlo, 0) / BAMD_PAGE, kept);
        count = kept + max(0, n_pages - first);
    }
    __device__ __forceinline__ int page(int i) const { return i < kept ? i : first + (i - kept); }
};
// eight consecutive values of a row of the projection, as an operand piece; ss: sum of their squares
template <typename T> struct KvRow8 {
    bamd_v4 x, y;
    __device__ __forceinline__ void load(const float * p) { x = *(const bamd_v4 *) p; y = *(const bamd_v4 *) (p + 4); }
    __device__ __forceinline__ float squares() const { float t = 0.f; for (int j = 0; j < 4; ++j) t += x[j] * x[j] + y[j] * y[j]; return t; }
    __device__ __forceinline__ void put(Frag<T> & f, float r) const {
#pragma unroll
        for (int j = 0; j < 4; ++j) { f.set(j, x[j] * r); f.set(4 + j, y[j] * r); }
    }
};
// a head's row as operand pieces (lane / 16 takes columns lq * 8 .. + 8 of every 32), divided by its root mean square
template <typename T, int ND> __device__ __forceinline__ void kv_head_load(const float * src, int lq, KvRow8<T> (&r)[ND]) {
#pragma unroll
    for (int k = 0; k < ND; ++k) r[k].load(src + k * 32 + lq * 8);
}
template <typename T, int ND> __device__ __forceinline__ void kv_head_norm(const bamd_kv_args & a, const KvRow8<T> (&r)[ND], Frag<T> (&f)[ND]) {
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < ND; ++k) ss += r[k].squares();
    ss += __shfl_xor(ss, 16); ss += __shfl_xor(ss, 32);
    const float n = a.unit ? 1.0f / sqrtf(ss / (float) a.dim + a.eps) : 1.0f;
#pragma unroll
    for (int k = 0; k < ND; ++k) r[k].put(f[k], n);
}
template <typename T, int ND> __device__ __forceinline__ void kv_head(const bamd_kv_args & a, const float * src, int lq, Frag<T> (&f)[ND]) {
    KvRow8<T> r[ND];
    kv_head_load<T, ND>(src, lq, r);
    kv_head_norm<T, ND>(a, r, f);
}

// LDS of a decoding block: the waves' weights, then their sums
template <typename T, int ND> struct KvDecodeLds {
    static constexpr int D = ND * 32, NP = sizeof(T) == 2 ? 2 : 1, PS = 32 + 16 / sizeof(T);
    static constexpr size_t weights = (size_t) 4 * NP * 16 * PS * sizeof(T), sums = ((size_t) 4 * 16 * D + 4 * 16 * 2) * 4, bytes = weights > sums ? weights : sums;
};
// one of `splits` shares of a row's keys for (kv head, group of 16 heads) = y; four waves take half pages in turn; the last wave of the last share brings the row's own key and value
// and stores them in the cache
template <typename T, int ND>
__device__ __forceinline__ void kv_decode_block(const bamd_batch_dev & b, const bamd_kv_args & a, int sp, int splits, int y, int row, float * part_o, float * part_ml, unsigned char * lds) {
    typedef KvDecodeLds<T, ND> L;
    constexpr int D = L::D, NV = ND * 2, NP = L::NP, PS = L::PS;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lq = lane >> 4;
    const int rep = a.heads / a.kv_heads, hgs = (rep + 15) / 16, g = y / hgs, hg = y % hgs, h0 = g * rep + hg * 16, nh = min(16, rep - hg * 16);
    const bamd_entry e = b.ent[row];
    const int pos = e.pos0, wi = sp * 4 + wave, nw = splits * 4;
    const KvPages pg(a, pos - a.window + 1, (pos + BAMD_PAGE - 1) / BAMD_PAGE);
    const int per = (2 * pg.count + nw - 1) / nw, t0 = wi * per, t1 = min(2 * pg.count, t0 + per);
    const bool own = wi == nw - 1;
    const size_t base = ((size_t) row * a.kv_heads * hgs + y) * splits + sp;
    if (sp * 4 * per >= 2 * pg.count && sp != splits - 1) {        // a share without keys
        for (int i = tid; i < nh * D; i += 256) part_o[base * 16 * D + i] = 0.f;
        if (tid < nh) { part_ml[(base * 16 + tid) * 2] = -INFINITY; part_ml[(base * 16 + tid) * 2 + 1] = 0.f; }
        return;
    }
    const int32_t * pages = b.pages + (size_t) e.seq * b.max_pages;
    const float * in = a.in + (size_t) row * a.ld;
    const KvCap cap = kv_cap(a);
    T * P = (T *) lds + (size_t) wave * NP * 16 * PS;
    // everything the first 32 keys need is on its way before the queries are normed (heads too wide for the registers read them as they go)
    constexpr bool AHEAD = ND * sizeof(T) <= 8;
    Frag<T> kf[AHEAD ? 2 : 1][ND], vf[NV];
    float bias[2][4];
    const T * K = nullptr, * V = nullptr;
    int k0 = 0;
    auto request = [&](int i) {
        const int p = pg.page(i >> 1), half = (i & 1) * 32;
        const size_t at = ((size_t) pages[p] * a.kv_heads + g) * BAMD_PAGE * D;
        K = (const T *) a.kc + at + (size_t) half * D; V = (const T *) a.vc + at + half; k0 = p * BAMD_PAGE + half;
        if constexpr (AHEAD) {
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int k = 0; k < ND; ++k) kf[t][k].load(K + (t * 16 + lr) * D + k * 32 + lq * 8);
#pragma unroll
            for (int j = 0; j < NV; ++j) vf[j].load(V + (j * 16 + lr) * BAMD_PAGE + lq * 8);
        }
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) bias[t][r] = kv_bias(a, h0 + min(lq * 4 + r, nh - 1), max(pos - (k0 + t * 16 + lr), 0));
    };
    KvRow8<T> qr[ND], kr[ND];
    float vr[NV];
    kv_head_load<T, ND>(in + a.q_off + (h0 + min(lr, nh - 1)) * D, lq, qr);
    if (t0 < t1) request(t0);
    if (own) {
        kv_head_load<T, ND>(in + a.k_off + g * D, lq, kr);         // the same in every column
#pragma unroll
        for (int j = 0; j < NV; ++j) vr[j] = in[a.v_off + g * D + j * 16 + lr];
    }
    Frag<T> q[ND];
    kv_head_norm<T, ND>(a, qr, q);
    bamd_v4 o[NV]; float m[4], l[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) { m[r] = -INFINITY; l[r] = 0.f; }
#pragma unroll
    for (int j = 0; j < NV; ++j) o[j] = bamd_v4{ 0, 0, 0, 0 };
    // scores -> weights in LDS, running maximum and sum
    auto weigh = [&](bamd_v4 (&sc)[2]) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float mx = fmaxf(m[r], row_max16(fmaxf(sc[0][r], sc[1][r])));
            const float al = mx == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m[r] - mx), ref = mx == -INFINITY ? 0.f : mx;
            float sum = 0.f;
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                const float pe = __builtin_amdgcn_exp2f(sc[t][r] - ref);
                sum += pe;
                T * d = P + (lq * 4 + r) * PS + t * 16 + lr;
                const T hi = to_act<T>(pe);
                *d = hi;
                if constexpr (NP == 2) d[16 * PS] = to_act<T>(pe - (float) hi);
            }
            l[r] = l[r] * al + sum; m[r] = mx;                    // (sums of this lane's columns; added up at the end)
#pragma unroll
            for (int j = 0; j < NV; ++j) o[j][r] *= al;
        }
        wave_lds_fence();
    };
    for (int i = t0; i < t1; ++i) {
        bamd_v4 sc[2];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            sc[t] = bamd_v4{ 0, 0, 0, 0 };
#pragma unroll
            for (int k = 0; k < ND; ++k) {
                if constexpr (!AHEAD) kf[0][k].load(K + (t * 16 + lr) * D + k * 32 + lq * 8);
                sc[t] = mma(q[k], kf[AHEAD ? t : 0][k], sc[t]);
            }
        }
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            const int j = k0 + t * 16 + lr;
            const bool seen = j < pos && (pos - j < a.window || j < a.keep);
#pragma unroll
            for (int r = 0; r < 4; ++r) sc[t][r] = seen ? kv_score<T>(sc[t][r], cap, bias[t][r]) : -INFINITY;
        }
        weigh(sc);
        Frag<T> pf[NP];
#pragma unroll
        for (int n = 0; n < NP; ++n) pf[n].load(P + (n * 16 + lr) * PS + lq * 8);
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            if constexpr (!AHEAD) vf[j].load(V + (j * 16 + lr) * BAMD_PAGE + lq * 8);
#pragma unroll
            for (int n = 0; n < NP; ++n) o[j] = mma(pf[n], vf[j], o[j]);
        }
        wave_lds_fence();
        if (i + 1 < t1) request(i + 1);
    }
    if (own) {
        Frag<T> kn[ND];
        kv_head_norm<T, ND>(a, kr, kn);
        bamd_v4 sc[2];
        sc[0] = bamd_v4{ 0, 0, 0, 0 };
#pragma unroll
        for (int k = 0; k < ND; ++k) sc[0] = mma(q[k], kn[k], sc[0]);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            sc[0][r] = lr == 0 ? kv_score<T>(sc[0][r], cap, kv_bias(a, h0 + min(lq * 4 + r, nh - 1), 0)) : -INFINITY;
            sc[1][r] = -INFINITY;
        }
        weigh(sc);
        Frag<T> pf[NP];
#pragma unroll
        for (int n = 0; n < NP; ++n) pf[n].load(P + (n * 16 + lr) * PS + lq * 8);
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            Frag<T> vn; vn.zero();
            if (lq == 0) vn.set(0, vr[j]);
#pragma unroll
            for (int n = 0; n < NP; ++n) o[j] = mma(pf[n], vn, o[j]);
        }
        if (hg == 0) {                                             // into the cache; a page's first position also clears the places behind it
            const int off = pos % BAMD_PAGE;
            const size_t at = ((size_t) pages[pos / BAMD_PAGE] * a.kv_heads + g) * BAMD_PAGE * D;
            if (lr == 0)
#pragma unroll
                for (int k = 0; k < ND; ++k) kn[k].store((T *) a.kc + at + (size_t) off * D + k * 32 + lq * 8);
            T * vd = (T *) a.vc + at;
            if (off == 0) for (int c = lane; c < D * BAMD_PAGE * (int) sizeof(T) / 16; c += 64) if (c % (BAMD_PAGE * (int) sizeof(T) / 16)) ((bamd_u4 *) vd)[c] = bamd_u4{ 0, 0, 0, 0 };
            if (lq == 0)
#pragma unroll
                for (int j = 0; j < NV; ++j) {
                    T * row = vd + (size_t) (j * 16 + lr) * BAMD_PAGE;
                    if (off == 0) { Frag<T> f; f.zero(); f.set(0, vr[j]); f.store(row); }       // (the first eight places)
                    else row[off] = to_act<T>(vr[j]);
                }
        }
    }
    // the four waves' sums
    __syncthreads();
    float * so = (float *) lds, * sml = so + 4 * 16 * D;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int hd = lq * 4 + r;
        const float sum = row_sum16(l[r]);
        if (lr == 0) { sml[(wave * 16 + hd) * 2] = m[r]; sml[(wave * 16 + hd) * 2 + 1] = sum; }
#pragma unroll
        for (int j = 0; j < NV; ++j) so[((size_t) wave * 16 + hd) * D + j * 16 + lr] = o[j][r];
    }
    __syncthreads();
    for (int i = tid; i < nh * D; i += 256) {
        const int hd = i / D, d = i % D;
        float mx = -INFINITY, s = 0.f, t = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) mx = fmaxf(mx, sml[(w * 16 + hd) * 2]);
        if (mx != -INFINITY)
#pragma unroll
            for (int w = 0; w < 4; ++w) { const float f = __builtin_amdgcn_exp2f(sml[(w * 16 + hd) * 2] - mx); s += f * sml[(w * 16 + hd) * 2 + 1]; t += f * so[((size_t) w * 16 + hd) * D + d]; }
        part_o[(base * 16 + hd) * D + d] = t;
        if (d == 0) { part_ml[(base * 16 + hd) * 2] = mx; part_ml[(base * 16 + hd) * 2 + 1] = s; }
    }
}
// the shares of head h of a row summed, gated and written as operand; a whole block
template <typename T>
__device__ __forceinline__ void kv_combine_block(const bamd_kv_args & a, int h, int row, const float * part_o, const float * part_ml, int splits) {
    const int rep = a.heads / a.kv_heads, hgs = (rep + 15) / 16, g = h / rep, hh = h % rep, y = g * hgs + hh / 16;
    const size_t base = ((size_t) row * a.kv_heads * hgs + y) * splits;
    const int lane = threadIdx.x & 63;
    __shared__ float wt[64];
    // every wave finds the weights of the shares by itself
    const float ms = lane < splits ? part_ml[((base + lane) * 16 + hh % 16) * 2] : -INFINITY, ls = lane < splits ? part_ml[((base + lane) * 16 + hh % 16) * 2 + 1] : 0.f;
    float mx = row_max16(ms);
    mx = fmaxf(mx, __shfl_xor(mx, 16)); mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float w = ms == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(ms - mx);
    const float sum = wave_sum(w * ls);
    if (threadIdx.x < 64) wt[lane] = w;
    __syncthreads();
    const float f = (a.gated ? sigmoid_f(a.in[(size_t) row * a.ld + a.g_off + h]) : 1.f) * a.out_scale / sum;
    for (int d = threadIdx.x; d < a.D; d += blockDim.x) {
        const float * src = part_o + (base * 16 + hh % 16) * a.D + d;
        float t = 0.f;
        for (int s = 0; s < splits; ++s) t += wt[s] * src[(size_t) s * 16 * a.D];
        ((T *) a.out)[(size_t) row * a.ldo + a.out_off + h * a.D + d] = to_act<T>(t * f);
    }
}
