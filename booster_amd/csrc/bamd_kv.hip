// bamd_kv.hip — attention over cached keys and values: grouped heads, 64-position pages, a sliding window beside a number of first tokens that stay visible; optional unit-RMS
// queries and keys, capped scores, a bias per distance and head, a gate per head.
//   The cache holds keys as rows and values transposed, per page and kv head contiguous, so that prompts and decoding read both straight as matrix operands.  Places of a page
//   behind the sequence's last position are zero in the values (whoever writes a page's first place clears it).
//   prompts: the new keys and values go to the cache, then a flash kernel runs per head over the pages its queries see — 64 keys per pass, scores and sums in 32-bit, the
//     weights as two bfloat16 terms (value + remainder) in front of the matrix cores.  The bias of a pass is one value per distance, staged in LDS;
//   decoding: up to sixteen heads of a kv head share one pass over the visible pages in `splits` parts; the row's own key enters from the projection.
// Scores are kept times log2(e).
#include "bamd_kv_device.h"
#include <math.h>

// block (64 positions of an entry, kv head)
template <typename T> __global__ void __launch_bounds__(256) kv_store_kernel(bamd_batch_dev b, bamd_kv_args a, const int32_t * k_entry) {
    extern __shared__ __align__(16) unsigned char lds[];
    T * vs = (T *) lds;                                            // [64][D + 2]
    const bamd_entry e = b.ent[k_entry[blockIdx.x]];
    const int pg = blockIdx.x - e.kbase / BAMD_PAGE, g = blockIdx.y, D = a.D, S = D + 2, p0 = pg * BAMD_PAGE;
    const int lo = max(p0, e.pos0) - p0, hi = min(p0 + BAMD_PAGE, e.pos0 + e.n) - p0;      // places of the page that this step brings
    if (lo >= hi) return;
    const size_t at = ((size_t) b.pages[(size_t) e.seq * b.max_pages + pg] * a.kv_heads + g) * BAMD_PAGE * D;
    // sixteen lanes per row, RU rows of a lane on their way at once
    constexpr int RU = 2;
    const int l = (threadIdx.x & 15) * 4, nc = (D + 63) / 64;
    for (int c0 = lo + (threadIdx.x >> 4); c0 < hi; c0 += 16 * RU) {
        bamd_v4 kv[RU][4], vv[RU][4];
#pragma unroll
        for (int u = 0; u < RU; ++u) {
            const int c = min(c0 + 16 * u, hi - 1);
            const float * in = a.in + (size_t) (e.row0 + p0 + c - e.pos0) * a.ld, * k = in + a.k_off + g * D, * v = in + a.v_off + g * D;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const bool live = i < nc && l + i * 64 < D;
                kv[u][i] = live ? *(const bamd_v4 *) (k + l + i * 64) : bamd_v4{ 0, 0, 0, 0 }; vv[u][i] = live ? *(const bamd_v4 *) (v + l + i * 64) : bamd_v4{ 0, 0, 0, 0 };
            }
        }
#pragma unroll
        for (int u = 0; u < RU; ++u) {
            const int c = c0 + 16 * u;
            float ss = 0.f;
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) ss += kv[u][i][j] * kv[u][i][j];
            ss = row_sum16(ss);
            if (c >= hi) continue;
            const float r = a.unit ? 1.0f / sqrtf(ss / (float) a.dim + a.eps) : 1.0f;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (i >= nc || l + i * 64 >= D) continue;
                store4<T>((T *) a.kc + at + (size_t) c * D + l + i * 64, kv[u][i] * r);
#pragma unroll
                for (int j = 0; j < 4; ++j) vs[c * S + l + i * 64 + j] = to_act<T>(vv[u][i][j]);
            }
        }
    }
    __syncthreads();
    for (int i = threadIdx.x * 4; i < D * BAMD_PAGE; i += 1024) {
        const int d = i / BAMD_PAGE, c = i % BAMD_PAGE;
        bamd_v4 t;
#pragma unroll
        for (int j = 0; j < 4; ++j) t[j] = c + j >= lo && c + j < hi ? (float) vs[(c + j) * S + d] : 0.f;
        if (c >= lo) store4<T>((T *) a.vc + at + i, t);
        else for (int j = 0; j < 4; ++j) if (c + j >= lo) ((T *) a.vc)[at + i + j] = to_act<T>(t[j]);
    }
}

// ND: head size in 32s; RT: 16-row query tiles per wave; four waves
template <typename T, int ND, int RT>
__global__ void __launch_bounds__(256) kv_prompt_kernel(bamd_batch_dev b, bamd_kv_args a, const bamd_qtile * tiles) {
    constexpr int D = ND * 32, NV = ND * 2, KS = D + 16 / sizeof(T), VS = 64 + 16 / sizeof(T), NP = sizeof(T) == 2 ? 2 : 1;     // NP: terms of a weight
    constexpr int PIECES = 64 * D * (int) sizeof(T) / 16, PER = PIECES / 256 > 0 ? PIECES / 256 : 1, NB = 64 * RT + 63;         // NB: distances of a pass
    extern __shared__ __align__(16) unsigned char lds[];
    T * Ks = (T *) lds, * Vs = Ks + 64 * KS, * Ps = Vs + D * VS;                 // Ps: per wave [NP][16 RT][VS]
    __shared__ float bs[NB + 1];
    // blocks of one kv head stay on one XCD (every eighth block) as far as the head counts allow
    const int rep = a.heads / a.kv_heads, hb = blockIdx.x % a.heads, g = hb % a.kv_heads, h = g * rep + hb / a.kv_heads;
    const bamd_qtile qt = tiles[blockIdx.x / a.heads];
    const bamd_entry e = b.ent[qt.entry];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lq = lane >> 4;
    T * P = Ps + (size_t) wave * NP * 16 * RT * VS;
    const int r0 = qt.q0 + wave * 16 * RT;                         // first query of this wave, counted in the entry
    Frag<T> q[RT][ND];
#pragma unroll
    for (int i = 0; i < RT; ++i) {
        int r = r0 + i * 16 + lr; r = r < e.n ? r : e.n - 1;
        kv_head<T, ND>(a, a.in + (size_t) (e.row0 + r) * a.ld + a.q_off + h * D, lq, q[i]);
    }
    bamd_v4 o[RT][NV]; float m[RT][4], l[RT][4];
#pragma unroll
    for (int i = 0; i < RT; ++i) {
#pragma unroll
        for (int k = 0; k < 4; ++k) { m[i][k] = -INFINITY; l[i][k] = 0.f; }
#pragma unroll
        for (int j = 0; j < NV; ++j) o[i][j] = bamd_v4{ 0, 0, 0, 0 };
    }
    const KvCap cap = kv_cap(a);
    const int lo = e.pos0 + qt.q0, hi = e.pos0 + min(qt.q0 + 64 * RT, e.n) - 1;      // positions of this block's queries
    const int w_lo = e.pos0 + r0, w_hi = e.pos0 + min(r0 + 16 * RT, e.n) - 1;        // of this wave's
    const KvPages pg(a, lo - a.window + 1, hi / BAMD_PAGE + 1);
    const int32_t * pages = b.pages + (size_t) e.seq * b.max_pages;
    bamd_u4 kr[PER], vr[PER];
    float br = 0.f;
    int phys = pages[pg.page(0)];
    auto fetch = [&](int i) {
        const size_t at = ((size_t) phys * a.kv_heads + g) * BAMD_PAGE * D;
        const bamd_u4 * kp = (const bamd_u4 *) ((const T *) a.kc + at), * vp = (const bamd_u4 *) ((const T *) a.vc + at);
#pragma unroll
        for (int c = 0; c < PER; ++c) if (PIECES >= 256 || tid < PIECES) { kr[c] = kp[tid + 256 * c]; vr[c] = vp[tid + 256 * c]; }
        if (tid < NB) br = kv_bias(a, h, max(lo - pg.page(i) * BAMD_PAGE + tid - 63, 0));
        if (i + 1 < pg.count) phys = pages[pg.page(i + 1)];
    };
    fetch(0);
    for (int i0 = 0; i0 < pg.count; ++i0) {
        const int k0 = pg.page(i0) * BAMD_PAGE;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int c = tid + 256 * i;
            if (PIECES >= 256 || c < PIECES) {
                constexpr int pk = D * (int) sizeof(T) / 16, pv = 64 * (int) sizeof(T) / 16;
                *(bamd_u4 *) ((unsigned char *) (Ks + (c / pk) * KS) + (c % pk) * 16) = kr[i];
                *(bamd_u4 *) ((unsigned char *) (Vs + (c / pv) * VS) + (c % pv) * 16) = vr[i];
            }
        }
        if (tid < NB) bs[tid] = br;
        __syncthreads();
        if (i0 + 1 < pg.count) fetch(i0 + 1);
        if (k0 > w_hi || r0 >= e.n || (k0 + 63 <= w_lo - a.window && k0 >= a.keep)) continue;      // nothing in this pass for this wave
        bamd_v4 sc[RT][4];
#pragma unroll
        for (int i = 0; i < RT; ++i)
#pragma unroll
            for (int t = 0; t < 4; ++t) sc[i][t] = bamd_v4{ 0, 0, 0, 0 };
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int k = 0; k < ND; ++k) {
                Frag<T> kf; kf.load(Ks + (t * 16 + lr) * KS + k * 32 + lq * 8);
#pragma unroll
                for (int i = 0; i < RT; ++i) sc[i][t] = mma(q[i][k], kf, sc[i][t]);
            }
        const bool all = k0 + 63 <= w_lo && (k0 + 63 < a.keep || w_hi - k0 < a.window);            // every key of the pass is seen by every row
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            const float * bw = bs + (wave * 16 * RT + i * 16 + lq * 4 + 63 - lr);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int pos = e.pos0 + r0 + i * 16 + lq * 4 + r;
                float mx = m[i][r];
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    float v = kv_score<T>(sc[i][t][r], cap, bw[r - t * 16]);
                    if (!all) { const int j = k0 + t * 16 + lr; if (j > pos || (pos - j >= a.window && j >= a.keep)) v = -INFINITY; }
                    sc[i][t][r] = v; mx = fmaxf(mx, v);
                }
                mx = row_max16(mx);
                const float al = mx == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m[i][r] - mx), ref = mx == -INFINITY ? 0.f : mx;
                float sum = 0.f;
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    const float pe = __builtin_amdgcn_exp2f(sc[i][t][r] - ref);
                    sum += pe;
                    T * d = P + (i * 16 + lq * 4 + r) * VS + t * 16 + lr;
                    const T hi16 = to_act<T>(pe);
                    *d = hi16;
                    if constexpr (NP == 2) d[16 * RT * VS] = to_act<T>(pe - (float) hi16);
                }
                l[i][r] = l[i][r] * al + sum; m[i][r] = mx;       // (sums of this lane's columns; added up at the end)
#pragma unroll
                for (int j = 0; j < NV; ++j) o[i][j][r] *= al;
            }
        }
        wave_lds_fence();
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            Frag<T> pf[RT][NP];
#pragma unroll
            for (int i = 0; i < RT; ++i)
#pragma unroll
                for (int n = 0; n < NP; ++n) pf[i][n].load(P + (n * 16 * RT + i * 16 + lr) * VS + k * 32 + lq * 8);
#pragma unroll
            for (int j = 0; j < NV; ++j) {
                Frag<T> vf; vf.load(Vs + (j * 16 + lr) * VS + k * 32 + lq * 8);
#pragma unroll
                for (int i = 0; i < RT; ++i)
#pragma unroll
                    for (int n = 0; n < NP; ++n) o[i][j] = mma(pf[i][n], vf, o[i][j]);
            }
        }
        wave_lds_fence();
    }
#pragma unroll
    for (int i = 0; i < RT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = r0 + i * 16 + lq * 4 + r;
            const float sum = row_sum16(l[i][r]);
            if (row >= e.n) continue;
            float f = a.out_scale / sum;
            if (a.gated) f *= sigmoid_f(a.in[(size_t) (e.row0 + row) * a.ld + a.g_off + h]);
            T * d = (T *) a.out + (size_t) (e.row0 + row) * a.ldo + a.out_off + h * D;
#pragma unroll
            for (int j = 0; j < NV; ++j) d[j * 16 + lr] = to_act<T>(o[i][j][r] * f);
        }
}

// block (kv head and head group, share, row): where only some shares hold keys, their blocks still spread over all XCDs
template <typename T, int ND>
__global__ void __launch_bounds__(256, ND <= 4 ? 2 : 1) kv_decode_kernel(bamd_batch_dev b, bamd_kv_args a, float * part_o, float * part_ml, int splits) {
    extern __shared__ __align__(16) unsigned char lds[];
    kv_decode_block<T, ND>(b, a, blockIdx.y, splits, blockIdx.x, blockIdx.z, part_o, part_ml, lds);
}
template <typename T> __global__ void __launch_bounds__(256) kv_combine_kernel(bamd_kv_args a, const float * part_o, const float * part_ml, int splits) {
    kv_combine_block<T>(a, blockIdx.x, blockIdx.y, part_o, part_ml, splits);
}

// ---- launches ---------------------------------------------------------------------------------------------------------------------------------------
void bamd_launch_kv_store(int act, const bamd_batch_dev & b, const bamd_kv_args & a, const int32_t * k_entry, int k_rows, hipStream_t s) {
    const dim3 grid(k_rows / BAMD_PAGE, a.kv_heads);
    if (act == BAMD_ACT_F32) hipLaunchKernelGGL(kv_store_kernel<float>, grid, dim3(256), (size_t) 64 * (a.D + 2) * 4, s, b, a, k_entry);
    else hipLaunchKernelGGL(kv_store_kernel<bamd_bf>, grid, dim3(256), (size_t) 64 * (a.D + 2) * 2, s, b, a, k_entry);
}
static int prompt_rt(int act, int D) { return act == BAMD_ACT_F32 ? 1 : D <= 128 ? 2 : 1; }
int bamd_kv_prompt_rows(int act, int D) { return 64 * prompt_rt(act, D); }
template <typename T, int ND, int RT>
static int prompt_go(const bamd_batch_dev & b, const bamd_kv_args & a, const bamd_qtile * tiles, int n, hipStream_t s) {
    constexpr int D = ND * 32, KS = D + 16 / sizeof(T), VS = 64 + 16 / sizeof(T), NP = sizeof(T) == 2 ? 2 : 1;
    const size_t lds = sizeof(T) * ((size_t) 64 * KS + (size_t) D * VS + (size_t) 4 * NP * 16 * RT * VS);
    hipLaunchKernelGGL((kv_prompt_kernel<T, ND, RT>), dim3(n * a.heads), dim3(256), lds, s, b, a, tiles);
    return 0;
}
bool bamd_kv_valid(const bamd_kv_args & a) {
    return a.heads >= 1 && a.kv_heads >= 1 && a.heads % a.kv_heads == 0 && a.window >= 1 && a.keep >= 0 && (!a.bias || a.bias_top >= 0) && !(a.ld & 3) && !(a.q_off & 3) && !(a.k_off & 3) && !(a.v_off & 3);
}
int bamd_launch_kv_prompt(int act, const bamd_batch_dev & b, const bamd_kv_args & a, const bamd_qtile * tiles, int n, hipStream_t s) {
    if (n < 1 || !bamd_kv_valid(a)) return 1;
    if (act == BAMD_ACT_F32) switch (a.D) {
        case 32: return prompt_go<float, 1, 1>(b, a, tiles, n, s);
        case 64: return prompt_go<float, 2, 1>(b, a, tiles, n, s);
        case 128: return prompt_go<float, 4, 1>(b, a, tiles, n, s);
        case 256: return prompt_go<float, 8, 1>(b, a, tiles, n, s);
    } else switch (a.D) {
        case 32: return prompt_go<bamd_bf, 1, 2>(b, a, tiles, n, s);
        case 64: return prompt_go<bamd_bf, 2, 2>(b, a, tiles, n, s);
        case 128: return prompt_go<bamd_bf, 4, 2>(b, a, tiles, n, s);
        case 256: return prompt_go<bamd_bf, 8, 1>(b, a, tiles, n, s);
    }
    return 1;
}
int bamd_kv_groups(const bamd_kv_args & a) { return a.kv_heads * ((a.heads / a.kv_heads + 15) / 16); }
int bamd_kv_span(const bamd_kv_args & a, int pages) {
    const long w = ((long) a.window + BAMD_PAGE - 1) / BAMD_PAGE + 1 + (a.keep + BAMD_PAGE - 1) / BAMD_PAGE;
    return w < pages ? (int) w : pages;
}
template <typename T, int ND>
static int decode_go(const bamd_batch_dev & b, const bamd_kv_args & a, float * po, float * pm, int splits, hipStream_t s) {
    constexpr size_t lds = KvDecodeLds<T, ND>::bytes;
    hipLaunchKernelGGL((kv_decode_kernel<T, ND>), dim3(bamd_kv_groups(a), splits, b.rows), dim3(256), lds, s, b, a, po, pm, splits);
    hipLaunchKernelGGL(kv_combine_kernel<T>, dim3(a.heads, b.rows), dim3(a.D < 64 ? 64 : a.D), 0, s, a, po, pm, splits);
    return 0;
}
int bamd_launch_kv_decode(int act, const bamd_batch_dev & b, const bamd_kv_args & a, float * po, float * pm, int splits, hipStream_t s) {
    if (splits < 1 || splits > 64 || !bamd_kv_valid(a)) return 1;
    if (act == BAMD_ACT_F32) switch (a.D) {
        case 32: return decode_go<float, 1>(b, a, po, pm, splits, s);
        case 64: return decode_go<float, 2>(b, a, po, pm, splits, s);
        case 128: return decode_go<float, 4>(b, a, po, pm, splits, s);
        case 256: return decode_go<float, 8>(b, a, po, pm, splits, s);
    } else switch (a.D) {
        case 32: return decode_go<bamd_bf, 1>(b, a, po, pm, splits, s);
        case 64: return decode_go<bamd_bf, 2>(b, a, po, pm, splits, s);
        case 128: return decode_go<bamd_bf, 4>(b, a, po, pm, splits, s);
        case 256: return decode_go<bamd_bf, 8>(b, a, po, pm, splits, s);
    }
    return 1;
}
