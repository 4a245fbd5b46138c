// bamd_latent.hip — latent attention: per position one vector c of kv_rank values is cached (64-position pages); keys and values are linear in it.
//   prompts: the latents of the sequence are unpacked once per step into keys and transposed values (two dense products) and a flash kernel runs per head — 64 keys per
//     pass, scores, running maximum and sums in 32-bit, the weights as two bfloat16 terms (value + remainder) in front of the matrix cores;
//   decoding: the query is carried into the latent space (q W_uk per head) and all heads of a sequence share the cached rows: one pass over the cache in `splits`
//     parts, partial sums combined, then the value up-projection per head.
// A sink enters as the first key's place in the running maximum and sum (weight exp(sink), no value); a gate multiplies each head by sigmoid of its own projection.
#include "bamd_dense_device.h"
#include <math.h>

// ---- the cache --------------------------------------------------------------------------------------------------------------------------------------
template <typename T> __device__ __forceinline__ void latent_store_row(const bamd_batch_dev & b, const bamd_latent_args & a, int row, float * red) {
    const bamd_entry e = b.ent[b.row_entry[row]];
    const int p = e.pos0 + (row - e.row0);
    const float * c = a.in + (size_t) row * a.ld + a.c_off;
    float v[1] = { 0.f };
    for (int i = threadIdx.x; i < a.R; i += blockDim.x) v[0] += c[i] * c[i];
    block_sum<1>(v, red);
    const float r = 1.0f / sqrtf(v[0] / (float) a.R + a.eps);
    T * d = (T *) a.cache + ((size_t) b.pages[(size_t) e.seq * b.max_pages + p / BAMD_PAGE] * BAMD_PAGE + p % BAMD_PAGE) * a.Rp;
    for (int i = threadIdx.x; i < a.Rp; i += blockDim.x) d[i] = to_act<T>(i < a.R ? c[i] * r * a.c_norm[i] : 0.f);
}
template <typename T> __global__ void __launch_bounds__(256) latent_store_kernel(bamd_batch_dev b, bamd_latent_args a) {
    __shared__ float red[16];
    latent_store_row<T>(b, a, blockIdx.x, red);
}
// one block per 64 rows of the destination = one page of a sequence
template <typename T> __global__ void __launch_bounds__(256) latent_gather_kernel(bamd_batch_dev b, bamd_latent_args a, const int32_t * k_entry, T * dst) {
    const bamd_entry e = b.ent[k_entry[blockIdx.x]];
    const int pg = blockIdx.x - e.kbase / BAMD_PAGE, len = e.pos0 + e.n, n = min(BAMD_PAGE, len - pg * BAMD_PAGE);
    const bamd_u4 * src = (const bamd_u4 *) ((const T *) a.cache + (size_t) b.pages[(size_t) e.seq * b.max_pages + pg] * BAMD_PAGE * a.Rp);
    bamd_u4 * d = (bamd_u4 *) (dst + (size_t) blockIdx.x * BAMD_PAGE * a.Rp);
    const int per = a.Rp * (int) sizeof(T) / 16;
    for (int i = threadIdx.x; i < BAMD_PAGE * per; i += 256) d[i] = i < n * per ? src[i] : bamd_u4{ 0, 0, 0, 0 };
}

// ---- prompts ----------------------------------------------------------------------------------------------------------------------------------------
// ND: head size in 32s (queries, keys and values); RT: 16-row query tiles per wave; four waves
template <typename T, int ND, int RT>
__global__ void __launch_bounds__(256) latent_prompt_kernel(bamd_batch_dev b, bamd_latent_args a, const bamd_qtile * tiles, int n_heads, const T * kmat, const T * vt, int ldv) {
    constexpr int D = ND * 32, NV = ND * 2, KS = D + 16 / sizeof(T), VS = 64 + 16 / sizeof(T), NP = sizeof(T) == 2 ? 2 : 1;     // NP: terms of a weight
    constexpr int PIECES = 64 * D * (int) sizeof(T) / 16;
    extern __shared__ __align__(16) unsigned char lds[];
    T * Ks = (T *) lds, * Vs = Ks + 64 * KS, * Ps = Vs + D * VS;                 // Ps: per wave [NP][16 RT][VS]
    const int h = blockIdx.x % n_heads;
    const bamd_qtile qt = tiles[blockIdx.x / n_heads];
    const bamd_entry e = b.ent[qt.entry];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lq = lane >> 4;
    T * P = Ps + (size_t) wave * NP * 16 * RT * VS;
    const int r0 = qt.q0 + wave * 16 * RT;                         // first query of this wave, counted in the entry
    Frag<T> q[RT][ND];
#pragma unroll
    for (int i = 0; i < RT; ++i) {
        int r = r0 + i * 16 + lr; r = r < e.n ? r : e.n - 1;
        const float * src = a.in + (size_t) (e.row0 + r) * a.ld + a.q_off + h * D;
#pragma unroll
        for (int k = 0; k < ND; ++k) {
            const bamd_v4 x = *(const bamd_v4 *) (src + k * 32 + lq * 8), y = *(const bamd_v4 *) (src + k * 32 + lq * 8 + 4);
#pragma unroll
            for (int j = 0; j < 4; ++j) { q[i][k].set(j, x[j]); q[i][k].set(4 + j, y[j]); }
        }
    }
    bamd_v4 o[RT][NV]; float m[RT][4], l[RT][4];
    const float snk = a.sink ? a.sink[h] : -INFINITY;
#pragma unroll
    for (int i = 0; i < RT; ++i) {
#pragma unroll
        for (int k = 0; k < 4; ++k) { m[i][k] = snk; l[i][k] = a.sink ? 1.f : 0.f; }
#pragma unroll
        for (int j = 0; j < NV; ++j) o[i][j] = bamd_v4{ 0, 0, 0, 0 };
    }
    const int q_hi = min(qt.q0 + 64 * RT, e.n) - 1, len = e.pos0 + q_hi + 1;    // keys 0 .. len - 1
    const int w_hi = e.pos0 + min(r0 + 16 * RT, e.n) - 1;                       // last key any row of this wave sees
    const int kstride = n_heads * D;
    const T * kb = kmat + (size_t) e.kbase * kstride + h * D;
    const T * vb = vt + (size_t) h * D * ldv + e.kbase;
    constexpr int PER = PIECES / 256 > 0 ? PIECES / 256 : 1;
    bamd_u4 kr[PER], vr[PER];
    auto fetch = [&](int k0) {                                     // scratch rows are padded to whole 64s
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int c = tid + 256 * i;
            if (PIECES >= 256 || c < PIECES) {
                constexpr int pk = D * (int) sizeof(T) / 16, pv = 64 * (int) sizeof(T) / 16;
                kr[i] = *(const bamd_u4 *) ((const unsigned char *) (kb + (size_t) (k0 + c / pk) * kstride) + (c % pk) * 16);
                vr[i] = *(const bamd_u4 *) ((const unsigned char *) (vb + (size_t) (c / pv) * ldv + k0) + (c % pv) * 16);
            }
        }
    };
    fetch(0);
    for (int k0 = 0; k0 < len; k0 += 64) {
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
        __syncthreads();
        if (k0 + 64 < len) fetch(k0 + 64);
        if (k0 > w_hi || r0 >= e.n) continue;                      // nothing in this pass for this wave
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
#pragma unroll
        for (int i = 0; i < RT; ++i) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int pos = e.pos0 + r0 + i * 16 + lq * 4 + r;
                float mx = m[i][r];
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    float v = sc[i][t][r] * a.scale;
                    if (k0 + t * 16 + lr > pos) v = -INFINITY;
                    sc[i][t][r] = v; mx = fmaxf(mx, v);
                }
                mx = fmaxf(mx, __shfl_xor(mx, 1)); mx = fmaxf(mx, __shfl_xor(mx, 2)); mx = fmaxf(mx, __shfl_xor(mx, 4)); mx = fmaxf(mx, __shfl_xor(mx, 8));
                const float al = mx == -INFINITY ? 1.f : __expf(m[i][r] - mx), ref = mx == -INFINITY ? 0.f : mx;
                float sum = 0.f;
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    const float pe = __expf(sc[i][t][r] - ref);
                    sum += pe;
                    T * d = P + (i * 16 + lq * 4 + r) * VS + t * 16 + lr;
                    const T hi = to_act<T>(pe);
                    *d = hi;
                    if constexpr (NP == 2) d[16 * RT * VS] = to_act<T>(pe - (float) hi);
                }
                sum += __shfl_xor(sum, 1); sum += __shfl_xor(sum, 2); sum += __shfl_xor(sum, 4); sum += __shfl_xor(sum, 8);
                l[i][r] = l[i][r] * al + sum; m[i][r] = mx;
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
            if (row >= e.n) continue;
            float f = 1.0f / l[i][r];
            if (a.gated) f *= sigmoid_f(a.in[(size_t) (e.row0 + row) * a.ld + a.g_off + h]);
            T * d = (T *) a.out + (size_t) (e.row0 + row) * a.ldo + h * D;
#pragma unroll
            for (int j = 0; j < NV; ++j) d[j * 16 + lr] = to_act<T>(o[i][j][r] * f);
        }
}

// ---- decoding ---------------------------------------------------------------------------------------------------------------------------------------
// block (h * parts + part, row): q of head h carried into the latent space, four 16-row tiles of it; block (heads * parts, row): the row's own latent into the cache
template <typename T> __global__ void __launch_bounds__(256) latent_absorb_kernel(bamd_batch_dev b, bamd_latent_args a, T * qp, int parts) {
    __shared__ float red[16];
    __shared__ __align__(16) float q[256];
    const int h = blockIdx.x / parts, row = blockIdx.y;
    if (h == a.heads) { latent_store_row<T>(b, a, row, red); return; }
    const int lane = threadIdx.x & 63, kt_n = a.D / 32, rt_n = a.Rp / 16, hp = (a.heads + 15) / 16 * 16, rt = (blockIdx.x % parts) * 4 + (threadIdx.x >> 6);
    bamd_u4 w[8];
#pragma unroll
    for (int kt = 0; kt < 8; ++kt) w[kt] = rt < rt_n && kt < kt_n ? *(const bamd_u4 *) (a.ukT + ((((size_t) h * rt_n + rt) * kt_n + kt) * 64 + lane) * 8) : bamd_u4{ 0, 0, 0, 0 };
    for (int i = threadIdx.x; i < 256; i += 256) q[i] = i < a.D ? a.in[(size_t) row * a.ld + a.q_off + h * a.D + i] : 0.f;
    __syncthreads();
    float v = 0.f;
#pragma unroll
    for (int kt = 0; kt < 8; ++kt) {
        const float * x = q + kt * 32 + (lane >> 4) * 8;
        v += bf_lo(w[kt].x) * x[0] + bf_hi(w[kt].x) * x[1] + bf_lo(w[kt].y) * x[2] + bf_hi(w[kt].y) * x[3] + bf_lo(w[kt].z) * x[4] + bf_hi(w[kt].z) * x[5] + bf_lo(w[kt].w) * x[6] + bf_hi(w[kt].w) * x[7];
    }
    v += __shfl_xor(v, 16); v += __shfl_xor(v, 32);
    if (lane < 16 && rt < rt_n) qp[((size_t) row * hp + h) * a.Rp + rt * 16 + lane] = to_act<T>(v);
}
// block (split, head group of 16, row).  NR: 16-column tiles of the latent per wave; KEYS: keys per pass (64, or 32 where the rows are too wide for the LDS)
template <typename T, int NR, int KEYS>
__global__ void __launch_bounds__(256) latent_decode_kernel(bamd_batch_dev b, bamd_latent_args a, const T * qp, float * part_o, float * part_ml, int splits) {
    constexpr int PAD = 16 / sizeof(T), NP = sizeof(T) == 2 ? 2 : 1, PS = KEYS + PAD;
    constexpr int JM = NR * 64 * (int) sizeof(T) / 256, JB = JM < 1 ? 1 : JM > 4 ? 4 : JM;        // pieces of a row per thread, at once
    extern __shared__ __align__(16) unsigned char lds[];
    const int S = a.Rp + PAD;
    T * Cs = (T *) lds, * Qs = Cs + KEYS * S, * Ps = Qs + 16 * S;  // [KEYS][S], [16][S], [NP][16][PS]
    __shared__ float sc[16][KEYS + 1], mx[16], ls[16], al[16];
    const int sp = blockIdx.x, hg = blockIdx.y, row = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lq = lane >> 4;
    const bamd_entry e = b.ent[row];
    const int len = e.pos0 + 1, n_pg = (len + BAMD_PAGE - 1) / BAMD_PAGE, per = (n_pg + splits - 1) / splits, pg0 = sp * per, pg1 = min(n_pg, pg0 + per);
    const int hgs = gridDim.y, rt_n = a.Rp / 16, kt_n = a.Rp / 32, pr = a.Rp * (int) sizeof(T) / 16;
    if (tid < 16) { mx[tid] = -INFINITY; ls[tid] = 0.f; }
    const T * qsrc = qp + ((size_t) row * hgs * 16 + hg * 16) * a.Rp;
    for (int i = tid; i < 16 * pr; i += 256) *(bamd_u4 *) ((unsigned char *) (Qs + (i / pr) * S) + (i % pr) * 16) = *(const bamd_u4 *) ((const unsigned char *) qsrc + (size_t) i * 16);
    bamd_v4 o[NR];
#pragma unroll
    for (int j = 0; j < NR; ++j) o[j] = bamd_v4{ 0, 0, 0, 0 };
    for (int i = pg0 * (BAMD_PAGE / KEYS); i < pg1 * (BAMD_PAGE / KEYS); ++i) {
        const int pg = i / (BAMD_PAGE / KEYS), k0 = i * KEYS, n = min(KEYS, len - k0);      // keys k0 .. k0 + n - 1
        if (n <= 0) break;
        const unsigned char * src = (const unsigned char *) ((const T *) a.cache + (size_t) b.pages[(size_t) e.seq * b.max_pages + pg] * BAMD_PAGE * a.Rp + (size_t) (k0 % BAMD_PAGE) * a.Rp);
        __syncthreads();
        // sixteen threads per row, four rows per wave and load
        for (int j0 = 0; j0 < pr; j0 += 16 * JB) {
            bamd_u4 v[KEYS / 16][JB];
#pragma unroll
            for (int r4 = 0; r4 < KEYS / 16; ++r4)
#pragma unroll
                for (int j = 0; j < JB; ++j) { const int r = (tid >> 4) + 16 * r4, c = j0 + j * 16 + (tid & 15); v[r4][j] = r < n && c < pr ? *(const bamd_u4 *) (src + ((size_t) r * pr + c) * 16) : bamd_u4{ 0, 0, 0, 0 }; }
#pragma unroll
            for (int r4 = 0; r4 < KEYS / 16; ++r4)
#pragma unroll
                for (int j = 0; j < JB; ++j) { const int r = (tid >> 4) + 16 * r4, c = j0 + j * 16 + (tid & 15); if (c < pr) *(bamd_u4 *) ((unsigned char *) (Cs + r * S) + c * 16) = v[r4][j]; }
        }
        __syncthreads();
        if (wave * 16 < KEYS) {   // scores of 16 heads x this wave's 16 keys
            bamd_v4 s = { 0, 0, 0, 0 };
            for (int k = 0; k < kt_n; ++k) {
                Frag<T> qf, cf;
                qf.load(Qs + lr * S + k * 32 + lq * 8); cf.load(Cs + (wave * 16 + lr) * S + k * 32 + lq * 8);
                s = mma(qf, cf, s);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) sc[lq * 4 + i][wave * 16 + lr] = wave * 16 + lr < n ? s[i] * a.scale : -INFINITY;
        }
        __syncthreads();
        {   // sixteen threads per head, KEYS / 16 keys each
            const int hd = tid >> 4, k = tid & 15;
            float v[KEYS / 16], m = mx[hd];
            const float m_old = m;
#pragma unroll
            for (int i = 0; i < KEYS / 16; ++i) { v[i] = sc[hd][k + 16 * i]; m = fmaxf(m, v[i]); }
            m = fmaxf(m, __shfl_xor(m, 1)); m = fmaxf(m, __shfl_xor(m, 2)); m = fmaxf(m, __shfl_xor(m, 4)); m = fmaxf(m, __shfl_xor(m, 8));
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < KEYS / 16; ++i) {
                const float p = __expf(v[i] - m);
                sum += p;
                const T hi = to_act<T>(p);
                Ps[hd * PS + k + 16 * i] = hi;
                if constexpr (NP == 2) Ps[(16 + hd) * PS + k + 16 * i] = to_act<T>(p - (float) hi);
            }
            sum += __shfl_xor(sum, 1); sum += __shfl_xor(sum, 2); sum += __shfl_xor(sum, 4); sum += __shfl_xor(sum, 8);
            if (k == 0) { const float f = __expf(m_old - m); al[hd] = f; ls[hd] = ls[hd] * f + sum; mx[hd] = m; }
        }
        __syncthreads();
        float f[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) f[i] = al[lq * 4 + i];
#pragma unroll
        for (int j = 0; j < NR; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) o[j][i] *= f[i];
#pragma unroll
        for (int k = 0; k < KEYS / 32; ++k) {
            Frag<T> pf[NP];
#pragma unroll
            for (int n2 = 0; n2 < NP; ++n2) pf[n2].load(Ps + (n2 * 16 + lr) * PS + k * 32 + lq * 8);
#pragma unroll
            for (int j = 0; j < NR; ++j) {
                const int rt = wave + 4 * j;
                if (rt < rt_n) {
                    Frag<T> cf;
                    const T * c = Cs + (k * 32 + lq * 8) * S + rt * 16 + lr;
                    if constexpr (sizeof(T) == 2) {
#pragma unroll
                        for (int i = 0; i < 8; ++i) cf.v[i] = c[i * S];
                    } else {
#pragma unroll
                        for (int i = 0; i < 4; ++i) { cf.a[i] = c[i * S]; cf.b[i] = c[(i + 4) * S]; }
                    }
#pragma unroll
                    for (int n2 = 0; n2 < NP; ++n2) o[j] = mma(pf[n2], cf, o[j]);
                }
            }
        }
    }
    __syncthreads();
    const size_t base = ((size_t) row * hgs + hg) * splits + sp;
    float * po = part_o + base * 16 * a.Rp;
#pragma unroll
    for (int j = 0; j < NR; ++j) {
        const int rt = wave + 4 * j;
        if (rt < rt_n && pg0 < pg1)
#pragma unroll
            for (int i = 0; i < 4; ++i) po[(size_t) (lq * 4 + i) * a.Rp + rt * 16 + lr] = o[j][i];
    }
    if (tid < 16) { part_ml[(base * 16 + tid) * 2] = mx[tid]; part_ml[(base * 16 + tid) * 2 + 1] = ls[tid]; }
}
// block (head, row): the parts' sums, the sink, the value up-projection, the gate
template <typename T> __global__ void __launch_bounds__(512) latent_combine_kernel(bamd_batch_dev b, bamd_latent_args a, const float * __restrict__ part_o, const float * __restrict__ part_ml, int splits) {
    extern __shared__ __align__(16) float cl[];                    // [Rp] | part sums [groups][Rp]
    __shared__ float wsp[64];
    __shared__ float inv;
    const int h = blockIdx.x, row = blockIdx.y, hgs = (a.heads + 15) / 16, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, hh = h % 16;
    const int n_pg = (b.ent[row].pos0 + BAMD_PAGE) / BAMD_PAGE, per = (n_pg + splits - 1) / splits, live = (n_pg + per - 1) / per;      // parts that hold keys
    const size_t base = ((size_t) row * hgs + h / 16) * splits;
    if (wave == 0) {
        const float snk = a.sink ? a.sink[h] : -INFINITY;
        const float ms = lane < live ? part_ml[((base + lane) * 16 + hh) * 2] : -INFINITY, ls = lane < live ? part_ml[((base + lane) * 16 + hh) * 2 + 1] : 0.f;
        float m = fmaxf(snk, ms);
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o));
        const float w = lane < live ? expf(ms - m) : 0.f;
        float sum = w * ls;
        wsp[lane] = w;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) sum += __shfl_xor(sum, o);
        if (a.sink) sum += expf(snk - m);
        if (lane == 0) inv = (a.gated ? sigmoid_f(a.in[(size_t) row * a.ld + a.g_off + h]) : 1.f) / sum;
    }
    __syncthreads();
    const int nq = a.Rp / 4, ng = 512 / nq, grp = tid / nq, q4 = (tid % nq) * 4;
    if (grp < ng) {
        bamd_v4 v = { 0, 0, 0, 0 };
        const float * src = part_o + (base * 16 + hh) * a.Rp + q4;
#pragma unroll 4
        for (int s = grp; s < live; s += ng) v = v + *(const bamd_v4 *) (src + (size_t) s * 16 * a.Rp) * wsp[s];
        *(bamd_v4 *) (cl + a.Rp * (1 + grp) + q4) = v;
    }
    __syncthreads();
    for (int r = tid; r < a.Rp; r += 512) { float v = 0.f; for (int g = 0; g < ng; ++g) v += cl[a.Rp * (1 + g) + r]; cl[r] = v; }
    __syncthreads();
    const int kt_n = a.Rp / 32, vt_n = a.D / 16;
    for (int t = wave; t < vt_n; t += 8) {
        float v = 0.f;
        const bamd_u4 * wv = (const bamd_u4 *) (a.uv.w + (((size_t) h * vt_n + t) * kt_n * 64 + lane) * 8);
#pragma unroll 8
        for (int kt = 0; kt < kt_n; ++kt) {
            const bamd_u4 w = wv[(size_t) kt * 64];
            const float * x = cl + kt * 32 + (lane >> 4) * 8;
            v += bf_lo(w.x) * x[0] + bf_hi(w.x) * x[1] + bf_lo(w.y) * x[2] + bf_hi(w.y) * x[3] + bf_lo(w.z) * x[4] + bf_hi(w.z) * x[5] + bf_lo(w.w) * x[6] + bf_hi(w.w) * x[7];
        }
        v += __shfl_xor(v, 16); v += __shfl_xor(v, 32);
        if (lane < 16) ((T *) a.out)[(size_t) row * a.ldo + h * a.D + t * 16 + lane] = to_act<T>(v * inv);
    }
}

// ---- launches ---------------------------------------------------------------------------------------------------------------------------------------
void bamd_launch_latent_store(int act, const bamd_batch_dev & b, const bamd_latent_args & a, hipStream_t s) {
    if (act == BAMD_ACT_F32) hipLaunchKernelGGL(latent_store_kernel<float>, dim3(b.rows), dim3(256), 0, s, b, a);
    else hipLaunchKernelGGL(latent_store_kernel<bamd_bf>, dim3(b.rows), dim3(256), 0, s, b, a);
}
void bamd_launch_latent_gather(int act, const bamd_batch_dev & b, const bamd_latent_args & a, const int32_t * k_entry, int k_rows, void * dst, hipStream_t s) {
    if (act == BAMD_ACT_F32) hipLaunchKernelGGL(latent_gather_kernel<float>, dim3(k_rows / BAMD_PAGE), dim3(256), 0, s, b, a, k_entry, (float *) dst);
    else hipLaunchKernelGGL(latent_gather_kernel<bamd_bf>, dim3(k_rows / BAMD_PAGE), dim3(256), 0, s, b, a, k_entry, (bamd_bf *) dst);
}
static int prompt_rt(int act, int D) { return act == BAMD_ACT_F32 ? 1 : D <= 128 ? 2 : 1; }
int bamd_latent_prompt_rows(int act, int D) { return 64 * prompt_rt(act, D); }
template <typename T, int ND, int RT>
static void prompt_go(const bamd_batch_dev & b, const bamd_latent_args & a, const bamd_qtile * tiles, int n, const void * k, const void * vt, int ldv, hipStream_t s) {
    constexpr int D = ND * 32, KS = D + 16 / sizeof(T), VS = 64 + 16 / sizeof(T), NP = sizeof(T) == 2 ? 2 : 1;
    const size_t lds = sizeof(T) * ((size_t) 64 * KS + (size_t) D * VS + (size_t) 4 * NP * 16 * RT * VS);
    hipLaunchKernelGGL((latent_prompt_kernel<T, ND, RT>), dim3(n * a.heads), dim3(256), lds, s, b, a, tiles, a.heads, (const T *) k, (const T *) vt, ldv);
}
int bamd_launch_latent_prompt(int act, const bamd_batch_dev & b, const bamd_latent_args & a, const bamd_qtile * tiles, int n, const void * k, const void * vt, int ldv, hipStream_t s) {
    if (n < 1 || (ldv & 63)) return 1;
    if (act == BAMD_ACT_F32) switch (a.D) {
        case 32: prompt_go<float, 1, 1>(b, a, tiles, n, k, vt, ldv, s); return 0;
        case 64: prompt_go<float, 2, 1>(b, a, tiles, n, k, vt, ldv, s); return 0;
        case 128: prompt_go<float, 4, 1>(b, a, tiles, n, k, vt, ldv, s); return 0;
        case 256: prompt_go<float, 8, 1>(b, a, tiles, n, k, vt, ldv, s); return 0;
    } else switch (a.D) {
        case 32: prompt_go<bamd_bf, 1, 2>(b, a, tiles, n, k, vt, ldv, s); return 0;
        case 64: prompt_go<bamd_bf, 2, 2>(b, a, tiles, n, k, vt, ldv, s); return 0;
        case 128: prompt_go<bamd_bf, 4, 2>(b, a, tiles, n, k, vt, ldv, s); return 0;
        case 256: prompt_go<bamd_bf, 8, 1>(b, a, tiles, n, k, vt, ldv, s); return 0;
    }
    return 1;
}
template <typename T> static size_t decode_lds(int Rp, int keys) { return sizeof(T) * ((size_t) (keys + 16) * (Rp + 16 / sizeof(T)) + 2 * 16 * (keys + 16 / sizeof(T))); }
#define DECODE_LDS (152 * 1024)
int bamd_latent_max_rank(int act) {                                // widest latent row with a decoding kernel
    int rp = 1024;
    while ((act == BAMD_ACT_F32 ? decode_lds<float>(rp, 32) : decode_lds<bamd_bf>(rp, 32)) > DECODE_LDS) rp -= 32;
    return rp;
}
template <typename T, int KEYS>
static void decode_pick(const bamd_batch_dev & b, const bamd_latent_args & a, const T * qp, float * po, float * pm, int splits, hipStream_t s) {
    const dim3 grid(splits, (a.heads + 15) / 16, b.rows);
    const size_t lds = decode_lds<T>(a.Rp, KEYS);
    const int nr = (a.Rp / 16 + 3) / 4;
    if (nr <= 1) hipLaunchKernelGGL((latent_decode_kernel<T, 1, KEYS>), grid, dim3(256), lds, s, b, a, qp, po, pm, splits);
    else if (nr <= 2) hipLaunchKernelGGL((latent_decode_kernel<T, 2, KEYS>), grid, dim3(256), lds, s, b, a, qp, po, pm, splits);
    else if (nr <= 4) hipLaunchKernelGGL((latent_decode_kernel<T, 4, KEYS>), grid, dim3(256), lds, s, b, a, qp, po, pm, splits);
    else if (nr <= 8) hipLaunchKernelGGL((latent_decode_kernel<T, 8, KEYS>), grid, dim3(256), lds, s, b, a, qp, po, pm, splits);
    else hipLaunchKernelGGL((latent_decode_kernel<T, 16, KEYS>), grid, dim3(256), lds, s, b, a, qp, po, pm, splits);
}
template <typename T>
static int decode_go(const bamd_batch_dev & b, const bamd_latent_args & a, void * qp, float * part_o, float * part_ml, int splits, hipStream_t s) {
    if (splits < 1 || splits > 64 || a.Rp > 1024 || decode_lds<T>(a.Rp, 32) > DECODE_LDS) return 1;
    const int parts = (a.Rp / 16 + 3) / 4;
    hipLaunchKernelGGL(latent_absorb_kernel<T>, dim3(a.heads * parts + 1, b.rows), dim3(256), 0, s, b, a, (T *) qp, parts);
    if (decode_lds<T>(a.Rp, 64) <= DECODE_LDS) decode_pick<T, 64>(b, a, (const T *) qp, part_o, part_ml, splits, s);
    else decode_pick<T, 32>(b, a, (const T *) qp, part_o, part_ml, splits, s);
    hipLaunchKernelGGL(latent_combine_kernel<T>, dim3(a.heads, b.rows), dim3(512), ((size_t) a.Rp + 2048) * 4, s, b, a, part_o, part_ml, splits);
    return 0;
}
int bamd_launch_latent_decode(int act, const bamd_batch_dev & b, const bamd_latent_args & a, void * qp, float * part_o, float * part_ml, int splits, hipStream_t s) {
    return act == BAMD_ACT_F32 ? decode_go<float>(b, a, qp, part_o, part_ml, splits, s) : decode_go<bamd_bf>(b, a, qp, part_o, part_ml, splits, s);
}
