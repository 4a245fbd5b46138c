// bamd_gla_device.h — the scan of gated linear attention (bamd_gla.hip) as a device function: one block walks PT value columns of one head over consecutive tokens.
//
// A lane keeps four columns of NPL state rows in registers (lane = column quad + group of state rows); what a token brings — v of the block's columns, k, alpha and q of
// the head's channels — is read from LDS, where a chunk of CT tokens lies while the next one is on its way in registers.  o is summed over a lane's rows at once and over the row
// groups once per chunk.
#pragma once
#include "bamd_dense_device.h"

enum { GLA_STEP = 0, GLA_SCAN = 1, GLA_STATE = 2 };                // one decoded token (alpha computed here) | outputs and final state | final state and product of the decays only
// sigmoid(z)^(1 / tau): log2 of the sigmoid is min(z, 0) log2(e) - log2(1 + exp(-|z|)), right to an ulp of 1 + exp(-|z|), which is an ulp of the result
__device__ __forceinline__ float gla_alpha(float z, float inv_tau) {
    const float l = 1.4426950408889634f;
    return __builtin_amdgcn_exp2f((fminf(z, 0.f) * l - __builtin_amdgcn_logf(1.f + __builtin_amdgcn_exp2f(-fabsf(z) * l))) * inv_tau);
}

template <int PT, int NPL, int MODE> struct GlaShape {
    static constexpr int Q = PT / 4, NG = 64 / Q, GROUPS = 4 * NG, NP = GROUPS * NPL, CT = MODE == GLA_STEP ? 1 : 8;      // NP >= Np state rows
    static constexpr int OPS = CT * (PT + 3 * NP), YP = MODE == GLA_STATE ? 0 : CT * GROUPS * PT;
    static constexpr size_t lds = ((size_t) OPS + YP) * 4;
};
// init: state at the first token (null: zero); fin: where the last one goes; prod: product of the decays (GLA_STATE).  All at this head.  row0: the first token's row
template <int PT, int NPL, int MODE>
__device__ __forceinline__ void gla_scan_block(const bamd_gla_args & a, int h, int p0, int row0, int n, const float * init, float * fin, float * prod, unsigned char * lds) {
    typedef GlaShape<PT, NPL, MODE> G;
    constexpr int Q = G::Q, NG = G::NG, GROUPS = G::GROUPS, NP = G::NP, CT = G::CT;
    constexpr int PF = MODE == GLA_STEP ? 1 : (CT * (PT + 3 * NP) / 4 + 255) / 256;
    float * ops = (float *) lds, * yp = ops + G::OPS;              // [v: CT x PT | k, alpha, q: CT x NP each], [CT][GROUPS][PT]
    float * vs = ops, * ks = ops + CT * PT, * as = ks + CT * NP, * qs = as + CT * NP;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, quad = lane % Q, grp = wave * NG + lane / Q, Np = a.Np, Pp = a.Pp, pw = min(PT, Pp - p0);
    const float * in = a.in + (size_t) row0 * a.ld;
    float s[NPL][4], dec[NPL];
#pragma unroll
    for (int j = 0; j < NPL; ++j) {
        const int r = grp * NPL + j;
        const bamd_v4 v = init && r < Np && quad * 4 < pw ? *(const bamd_v4 *) (init + (size_t) r * Pp + p0 + quad * 4) : bamd_v4{ 0, 0, 0, 0 };
#pragma unroll
        for (int k = 0; k < 4; ++k) s[j][k] = v[k];
        dec[j] = 1.f;
    }
    for (int i = tid; i < G::OPS; i += 256) ops[i] = 0.f;
    // this thread's share of a chunk, four floats each: place behind the chunk's first row, place in LDS; the kind: 0 projection, 1 alpha, -1 none
    int src[PF], dst[PF], tok[PF], kind[PF];
    bamd_v4 pf[PF];
    const size_t aw = (size_t) a.heads * Np;
    if constexpr (MODE != GLA_STEP) {
        const int vq = (pw + 3) / 4, nq = Np / 4, per = vq + (MODE == GLA_STATE ? 2 : 3) * nq;
#pragma unroll
        for (int i = 0; i < PF; ++i) {
            const int k = tid + 256 * i, t = k / per, c = k % per;
            tok[i] = t; kind[i] = t < CT ? 0 : -1; src[i] = 0; dst[i] = 0;
            if (t >= CT) continue;
            if (c < vq) { src[i] = t * a.ld + a.v_off + h * Pp + p0 + c * 4; dst[i] = t * PT + c * 4; }
            else {
                const int w = (c - vq) / nq, m = (c - vq) % nq * 4;
                dst[i] = CT * PT + w * CT * NP + t * NP + m;
                if (w == 1) { kind[i] = 1; src[i] = t * (int) aw + h * Np + m; }
                else src[i] = t * a.ld + (w == 0 ? a.k_off : a.q_off) + h * Np + m;
            }
        }
    }
    auto request = [&](int t0) {
        const float * pi = in + (size_t) t0 * a.ld, * pa = a.alpha + (size_t) (row0 + t0) * aw;
#pragma unroll
        for (int i = 0; i < PF; ++i) if (kind[i] >= 0 && t0 + tok[i] < n) pf[i] = *(const bamd_v4 *) ((kind[i] ? pa : pi) + src[i]);
    };
    if constexpr (MODE != GLA_STEP) request(0);
    for (int t0 = 0; t0 < n; t0 += CT) {
        const int nt = min(CT, n - t0);
        __syncthreads();                                           // zeroes are in, or the chunk before is done with LDS
        if constexpr (MODE != GLA_STEP) {
#pragma unroll
            for (int i = 0; i < PF; ++i) if (kind[i] >= 0 && tok[i] < nt) *(bamd_v4 *) (ops + dst[i]) = pf[i];
        } else {
            for (int c = tid; c < pw; c += 256) vs[c] = in[a.v_off + h * Pp + p0 + c];
            for (int c = tid; c < Np; c += 256) {
                ks[c] = in[a.k_off + h * Np + c]; qs[c] = in[a.q_off + h * Np + c];
                float z = a.a2b[h * Np + c];
                for (int r0 = 0; r0 < a.rank; r0 += 16) {          // sixteen factors on their way at once
                    float w[16], t[16];
#pragma unroll
                    for (int r = 0; r < 16; ++r) { const int i = min(r0 + r, a.rank - 1); w[r] = bf_f(a.a2[(size_t) i * aw + h * Np + c]); t[r] = in[a.t_off + i]; }
#pragma unroll
                    for (int r = 0; r < 16; ++r) z = fmaf(r0 + r < a.rank ? w[r] : 0.f, t[r], z);
                }
                as[c] = gla_alpha(z, a.inv_tau);
            }
        }
        __syncthreads();
        if constexpr (MODE != GLA_STEP) if (t0 + CT < n) request(t0 + CT);
        auto token = [&](int t) {
            const bamd_v4 v = *(const bamd_v4 *) (vs + t * PT + quad * 4);
            float y[4] = { 0.f, 0.f, 0.f, 0.f };
#pragma unroll
            for (int j = 0; j < NPL; ++j) {
                const float k = ks[t * NP + grp * NPL + j], al = as[t * NP + grp * NPL + j];
#pragma unroll
                for (int c = 0; c < 4; ++c) s[j][c] = fmaf(al, s[j][c], k * v[c]);
                if constexpr (MODE == GLA_STATE) dec[j] *= al;
                else {
                    const float q = qs[t * NP + grp * NPL + j];
#pragma unroll
                    for (int c = 0; c < 4; ++c) y[c] = fmaf(q, s[j][c], y[c]);
                }
            }
            if constexpr (MODE != GLA_STATE) *(bamd_v4 *) (yp + (t * GROUPS + grp) * PT + quad * 4) = bamd_v4{ y[0], y[1], y[2], y[3] };
        };
        if (nt == CT) {                                            // a whole chunk: unrolled, the next token's operands are read under this one's arithmetic
#pragma unroll
            for (int t = 0; t < CT; ++t) token(t);
        } else for (int t = 0; t < nt; ++t) token(t);
        if constexpr (MODE != GLA_STATE) {
            __syncthreads();
            for (int i = tid; i < nt * PT; i += 256) {
                const int t = i / PT, c = i % PT;
                if (c >= pw) continue;
                float y[4] = { 0.f, 0.f, 0.f, 0.f };
#pragma unroll
                for (int g = 0; g < GROUPS; ++g) y[g & 3] += yp[(t * GROUPS + g) * PT + c];
                a.y[(size_t) (row0 + t0 + t) * a.ldy + h * Pp + p0 + c] = ((y[0] + y[1]) + (y[2] + y[3])) * a.q_scale;
            }
        }
    }
#pragma unroll
    for (int j = 0; j < NPL; ++j) {
        const int r = grp * NPL + j;
        if (r >= Np) continue;
        if (quad * 4 < pw) *(bamd_v4 *) (fin + (size_t) r * Pp + p0 + quad * 4) = bamd_v4{ s[j][0], s[j][1], s[j][2], s[j][3] };
        if constexpr (MODE == GLA_STATE) if (p0 == 0 && quad == 0) prod[r] = dec[j];
    }
}
// sixteen heads of a row from h0 on, sixteen lanes each: norm over a head's columns, gate; a whole block of 256
template <typename T> __device__ __forceinline__ void gla_norm_block(const bamd_gla_args & a, int h0, int row) {
    constexpr int RC = 4;
    const int h = h0 + (threadIdx.x >> 4), l = (threadIdx.x & 15) * 4;
    T * out = (T *) a.out + (size_t) row * a.ldo + a.out_off;
    if (h < a.heads) {
        const float * y = a.y + (size_t) row * a.ldy + h * a.Pp, * g = a.g_off >= 0 ? a.in + (size_t) row * a.ld + a.g_off + h * a.Pp : nullptr;
        bamd_v4 v[RC], gv[RC];
        float ss = 0.f;
#pragma unroll
        for (int c = 0; c < RC; ++c) {
            const int i = l + c * 64;
            v[c] = i < a.Pp ? *(const bamd_v4 *) (y + i) : bamd_v4{ 0, 0, 0, 0 };
            if (g) gv[c] = i < a.Pp ? *(const bamd_v4 *) (g + i) : bamd_v4{ 0, 0, 0, 0 };
#pragma unroll
            for (int k = 0; k < 4; ++k) ss += v[c][k] * v[c][k];
        }
        for (int i = l + RC * 64; i < a.Pp; i += 64) { const bamd_v4 t = *(const bamd_v4 *) (y + i); for (int k = 0; k < 4; ++k) ss += t[k] * t[k]; }
        const float r = 1.0f / sqrtf(row_sum16(ss) / (float) a.P + a.eps);
        auto put = [&](int i, bamd_v4 t, bamd_v4 gate) {
            t = t * r * *(const bamd_v4 *) (a.norm + i);
            if (g)
#pragma unroll
                for (int k = 0; k < 4; ++k) t[k] *= gate[k] / (1.0f + __expf(-gate[k]));
            store4<T>(out + h * a.Pp + i, t);
        };
#pragma unroll
        for (int c = 0; c < RC; ++c) if (l + c * 64 < a.Pp) put(l + c * 64, v[c], gv[c]);
        for (int i = l + RC * 64; i < a.Pp; i += 64) put(i, *(const bamd_v4 *) (y + i), g ? *(const bamd_v4 *) (g + i) : bamd_v4{ 0, 0, 0, 0 });
    }
    if (h0 + 16 >= a.heads) for (int c = a.heads * a.Pp + threadIdx.x; c < a.out_cols; c += 256) out[c] = to_act<T>(0.f);
}
