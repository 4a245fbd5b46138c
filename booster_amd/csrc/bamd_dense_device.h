// bamd_dense_device.h — device-side pieces shared by the kernels of the configured layer stacks: operand fragments and their matrix-core products for both
// activation types, block reductions, and the row mechanisms in the form that both the row kernels and the prologues of the few-row product use.
#pragma once
#include "bamd_dense.h"

typedef __bf16 bamd_bf;
typedef __bf16 bamd_bf8 __attribute__((ext_vector_type(8)));
typedef float bamd_v4 __attribute__((ext_vector_type(4)));
typedef unsigned int bamd_u4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float bf_lo(uint32_t u) { return __uint_as_float(u << 16); }
__device__ __forceinline__ float bf_hi(uint32_t u) { return __uint_as_float(u & 0xffff0000u); }
__device__ __forceinline__ float bf_f(uint16_t u) { return __uint_as_float((uint32_t) u << 16); }

// eight consecutive k of one row / column
template <typename T> struct Frag;
template <> struct Frag<bamd_bf> {
    bamd_bf8 v;
    __device__ __forceinline__ void zero() { v = __builtin_bit_cast(bamd_bf8, bamd_u4{ 0, 0, 0, 0 }); }
    __device__ __forceinline__ void load(const bamd_bf * p) { v = *(const bamd_bf8 *) p; }
    __device__ __forceinline__ void weight(bamd_u4 w) { v = __builtin_bit_cast(bamd_bf8, w); }
    __device__ __forceinline__ void set(int i, float f) { v[i] = (bamd_bf) f; }
    __device__ __forceinline__ void store(bamd_bf * p) const { *(bamd_bf8 *) p = v; }
};
template <> struct Frag<float> {
    bamd_v4 a, b;
    __device__ __forceinline__ void zero() { a = bamd_v4{ 0, 0, 0, 0 }; b = a; }
    __device__ __forceinline__ void load(const float * p) { a = *(const bamd_v4 *) p; b = *(const bamd_v4 *) (p + 4); }
    __device__ __forceinline__ void weight(bamd_u4 w) { a = bamd_v4{ bf_lo(w.x), bf_hi(w.x), bf_lo(w.y), bf_hi(w.y) }; b = bamd_v4{ bf_lo(w.z), bf_hi(w.z), bf_lo(w.w), bf_hi(w.w) }; }
    __device__ __forceinline__ void set(int i, float f) { if (i < 4) a[i] = f; else b[i - 4] = f; }
    __device__ __forceinline__ void store(float * p) const { *(bamd_v4 *) p = a; *(bamd_v4 *) (p + 4) = b; }
};
// D[row = (lane / 16) * 4 + i][col = lane % 16] += sum over 32 k of A[row][k] B[k][col]
__device__ __forceinline__ bamd_v4 mma(const Frag<bamd_bf> & a, const Frag<bamd_bf> & b, bamd_v4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0); }
__device__ __forceinline__ bamd_v4 mma(const Frag<float> & a, const Frag<float> & b, bamd_v4 c) {
#pragma unroll
    for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.a[i], b.a[i], c, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.b[i], b.b[i], c, 0, 0, 0);
    return c;
}
template <typename T> __device__ __forceinline__ T to_act(float f) { return (T) f; }

__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float silu_f(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.0f) + log1pf(expf(-fabsf(x))); }

// sum over the wave, the same in every lane: rows of sixteen lanes by data-parallel moves, then the four rows
__device__ __forceinline__ float wave_sum(float v) {
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xb1, 0xf, 0xf, true));      // lane ^ 1
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4e, 0xf, 0xf, true));      // lane ^ 2
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x141, 0xf, 0xf, true));     // the other four of eight
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x140, 0xf, 0xf, true));     // the other eight of sixteen
    const int i = __float_as_int(v);
    return (__int_as_float(__builtin_amdgcn_readlane(i, 0)) + __int_as_float(__builtin_amdgcn_readlane(i, 16))) + (__int_as_float(__builtin_amdgcn_readlane(i, 32)) + __int_as_float(__builtin_amdgcn_readlane(i, 48)));
}
// maximum and sum over the sixteen lanes of a row
__device__ __forceinline__ float row_sum16(float v) {
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xb1, 0xf, 0xf, true));
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4e, 0xf, 0xf, true));
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x141, 0xf, 0xf, true));
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x140, 0xf, 0xf, true));
    return v;
}
__device__ __forceinline__ float row_max16(float v) {
    v = fmaxf(v, __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xb1, 0xf, 0xf, true)));
    v = fmaxf(v, __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4e, 0xf, 0xf, true)));
    v = fmaxf(v, __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x141, 0xf, 0xf, true)));
    v = fmaxf(v, __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x140, 0xf, 0xf, true)));
    return v;
}
__device__ __forceinline__ void wave_lds_fence() { __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront"); __builtin_amdgcn_wave_barrier(); }

// sums of NV values over the block; red: NV * 16 floats of LDS.  Every thread gets the result
template <int NV> __device__ __forceinline__ void block_sum(float (&v)[NV], float * red) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
#pragma unroll
    for (int i = 0; i < NV; ++i) v[i] = wave_sum(v[i]);
    __syncthreads();
    if (lane == 0)
#pragma unroll
        for (int i = 0; i < NV; ++i) red[i * 16 + wave] = v[i];
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NV; ++i) { float t = 0.f; for (int w = 0; w < nw; ++w) t += red[i * 16 + w]; v[i] = t; }
}

// A row of n floats spread over the block four at a time, kept in registers between the passes over it: `fits` rows (n a multiple of four, at most RC pieces per
// thread) take this path, others re-read memory.
template <int RC> struct RowRegs {
    bamd_v4 v[RC];
    static __device__ __forceinline__ bool fits(int n) { return (n & 3) == 0 && n <= (int) blockDim.x * 4 * RC; }
    static __device__ __forceinline__ int at(int c) { return ((int) threadIdx.x + c * (int) blockDim.x) * 4; }
    __device__ __forceinline__ void load(const float * p, int n) {
#pragma unroll
        for (int c = 0; c < RC; ++c) v[c] = at(c) < n ? *(const bamd_v4 *) (p + at(c)) : bamd_v4{ 0, 0, 0, 0 };
    }
    __device__ __forceinline__ void clear() {
#pragma unroll
        for (int c = 0; c < RC; ++c) v[c] = bamd_v4{ 0, 0, 0, 0 };
    }
    __device__ __forceinline__ float squares() const {
        float t = 0.f;
#pragma unroll
        for (int c = 0; c < RC; ++c)
#pragma unroll
            for (int k = 0; k < 4; ++k) t += v[c][k] * v[c][k];
        return t;
    }
};
template <typename T> __device__ __forceinline__ void store4(T * h, bamd_v4 v);
template <> __device__ __forceinline__ void store4<float>(float * h, bamd_v4 v) { *(bamd_v4 *) h = v; }
template <> __device__ __forceinline__ void store4<bamd_bf>(bamd_bf * h, bamd_v4 v) {
    typedef __bf16 bf4 __attribute__((ext_vector_type(4)));
    *(bf4 *) h = bf4{ (bamd_bf) v[0], (bamd_bf) v[1], (bamd_bf) v[2], (bamd_bf) v[3] };
}
template <typename T> __device__ __forceinline__ void zero_tail(T * h, int n, int ld) { for (int i = n + threadIdx.x; i < ld; i += blockDim.x) h[i] = to_act<T>(0.f); }

// mean and variance (mean of the squared deviations) of a row in registers: per wave around its own mean, then over the waves.  red: 48 floats of LDS
template <int RC> __device__ __forceinline__ void row_moments(const RowRegs<RC> & r, int n, float * red, float & mean, float & var) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    float s = 0.f, c = 0.f, q = 0.f;
#pragma unroll
    for (int i = 0; i < RC; ++i) if (RowRegs<RC>::at(i) < n) { s += (r.v[i][0] + r.v[i][1]) + (r.v[i][2] + r.v[i][3]); c += 4.f; }
    s = wave_sum(s); c = wave_sum(c);
    const float m = c > 0.f ? s / c : 0.f;
#pragma unroll
    for (int i = 0; i < RC; ++i) if (RowRegs<RC>::at(i) < n)
#pragma unroll
        for (int k = 0; k < 4; ++k) { const float d = r.v[i][k] - m; q += d * d; }
    q = wave_sum(q);
    __syncthreads();
    if (lane == 0) { red[wave] = m; red[16 + wave] = q; red[32 + wave] = c; }
    __syncthreads();
    mean = 0.f; var = 0.f;
    for (int w = 0; w < nw; ++w) mean += red[w] * red[32 + w];
    mean /= (float) n;
    for (int w = 0; w < nw; ++w) { const float d = red[w] - mean; var += red[16 + w] + red[32 + w] * d * d; }
    var /= (float) n;
}
// residual sum with the layer norm of the sublayer's output, and the layer norm (gain gi, null: none) the next sublayer reads, of one row by the whole block
template <typename T>
__device__ __forceinline__ void layer_row(const bamd_residual_args & a, int row, const float * gi, T * h, bool write, float * red) {
    constexpr int RC = 2;
    const int E = a.E;
    const float * x = a.x + (size_t) row * E, * y = a.y ? a.y + (size_t) row * a.ldy : nullptr;
    float * xo = a.xo + (size_t) row * E;
    if (RowRegs<RC>::fits(E)) {
        RowRegs<RC> xr, yr;
        bamd_v4 g[RC], w[RC];
        xr.load(x, E);
        if (y) yr.load(y, E);
#pragma unroll
        for (int c = 0; c < RC; ++c) {
            const int i = RowRegs<RC>::at(c);
            if (y) g[c] = i < E ? *(const bamd_v4 *) (a.g + i) : bamd_v4{ 0, 0, 0, 0 };
            if (gi) w[c] = i < E ? *(const bamd_v4 *) (gi + i) : bamd_v4{ 0, 0, 0, 0 };
        }
        float mean, var;
        if (y) {
            row_moments<RC>(yr, E, red, mean, var);
            const float r = 1.0f / sqrtf(var + a.eps);
#pragma unroll
            for (int c = 0; c < RC; ++c) xr.v[c] = xr.v[c] + (yr.v[c] - mean) * r * g[c];
        }
        if (write)
#pragma unroll
            for (int c = 0; c < RC; ++c) { const int i = RowRegs<RC>::at(c); if (i < E) *(bamd_v4 *) (xo + i) = xr.v[c]; }
        if (!h) return;
        float r = 1.f;
        mean = 0.f;
        if (gi) { row_moments<RC>(xr, E, red, mean, var); r = 1.0f / sqrtf(var + a.eps); }
#pragma unroll
        for (int c = 0; c < RC; ++c) { const int i = RowRegs<RC>::at(c); if (i < E) store4<T>(h + i, gi ? (xr.v[c] - mean) * r * w[c] : xr.v[c]); }
        zero_tail(h, E, a.ldh);
        return;
    }
    float my = 0.f, ry = 0.f, v[1];
    if (y) {
        v[0] = 0.f;
        for (int i = threadIdx.x; i < E; i += blockDim.x) v[0] += y[i];
        block_sum<1>(v, red);
        my = v[0] / (float) E; v[0] = 0.f;
        for (int i = threadIdx.x; i < E; i += blockDim.x) { const float d = y[i] - my; v[0] += d * d; }
        block_sum<1>(v, red);
        ry = 1.0f / sqrtf(v[0] / (float) E + a.eps);
    }
    auto at = [&](int i) { return y ? x[i] + (y[i] - my) * ry * a.g[i] : x[i]; };
    float mx = 0.f, rx = 1.f;
    if (gi && h) {
        v[0] = 0.f;
        for (int i = threadIdx.x; i < E; i += blockDim.x) v[0] += at(i);
        block_sum<1>(v, red);
        mx = v[0] / (float) E; v[0] = 0.f;
        for (int i = threadIdx.x; i < E; i += blockDim.x) { const float d = at(i) - mx; v[0] += d * d; }
        block_sum<1>(v, red);
        rx = 1.0f / sqrtf(v[0] / (float) E + a.eps);
    }
    for (int i = threadIdx.x; i < E; i += blockDim.x) {
        const float xn = at(i);
        if (write) xo[i] = xn;
        if (h) h[i] = to_act<T>(gi ? (xn - mx) * rx * gi[i] : xn);
    }
    if (h) zero_tail(h, E, a.ldh);
}
__device__ __forceinline__ float clamped_glu(float gate, float up, float limit) {
    const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
    return g / (1.0f + __expf(-1.702f * g)) * (u + 1.0f);
}
// columns [from, to) of a row
template <typename T>
__device__ __forceinline__ void glu_row(const bamd_glu_args & a, int row, T * h, int from, int to) {
    const float * z = a.z + (size_t) row * a.ldz;
    for (int i = from + threadIdx.x * 4; i < to; i += blockDim.x * 4) {
        const bamd_v4 g = *(const bamd_v4 *) (z + (i >> 4) * 32 + (i & 15)), u = *(const bamd_v4 *) (z + (i >> 4) * 32 + 16 + (i & 15));
        store4<T>(h + i, bamd_v4{ clamped_glu(g[0], u[0], a.limit), clamped_glu(g[1], u[1], a.limit), clamped_glu(g[2], u[2], a.limit), clamped_glu(g[3], u[3], a.limit) });
    }
}

// residual sum, norm of the sublayer's output and token shift of one row by the whole block.  h: LDS or global row (null: none).  write: this block also stores x' and the
// state.  SINGLE: the step has one row
template <typename T, bool SINGLE>
__device__ __forceinline__ void residual_row(const bamd_batch_dev & b, const bamd_residual_args & a, int row, T * h, bool write, float * red) {
    constexpr int RC = 2;
    const bool shifted = a.mu != nullptr;
    const int E = a.E;
    const float * x = a.x + (size_t) row * E, * y = a.y ? a.y + (size_t) row * a.ldy : nullptr;
    bamd_entry e; bool first = true, last = true;
    if (shifted) {
        e = b.ent[SINGLE ? 0 : b.row_entry[row]];
        if (!SINGLE) { first = row == e.row0; last = row == e.row0 + e.n - 1; }
    }
    const bool before = !SINGLE && shifted && !first;            // x' of the row in front is rebuilt here: another block may be the one that stores it
    const float * xp = before ? x - E : nullptr, * yp = before && y ? y - a.ldy : nullptr;
    const float * sp = shifted && first && e.pos0 > 0 ? a.prev + ((size_t) e.par * b.n_seq + e.seq) * E : nullptr;
    float * so = shifted && last && write ? a.prev + ((size_t) (e.par ^ 1) * b.n_seq + e.seq) * E : nullptr;
    if (RowRegs<RC>::fits(E)) {
        RowRegs<RC> xr, yr, pr, qr, mu;
        xr.load(x, E);
        if (y) yr.load(y, E);
        if (shifted) { mu.load(a.mu, E); if (before) { pr.load(xp, E); if (yp) qr.load(yp, E); } else if (sp) pr.load(sp, E); else pr.clear(); }
        float r = 0.f, rp = 0.f;
        if (y) {
            const float g = a.g[0];
            if constexpr (SINGLE) { float v[1] = { yr.squares() }; block_sum<1>(v, red); r = g / sqrtf(v[0] / (float) E + a.eps); }
            else { float v[2] = { yr.squares(), yp ? qr.squares() : 0.f }; block_sum<2>(v, red); r = g / sqrtf(v[0] / (float) E + a.eps); rp = g / sqrtf(v[1] / (float) E + a.eps); }
        }
#pragma unroll
        for (int c = 0; c < RC; ++c) {
            const int i = RowRegs<RC>::at(c);
            if (i >= E) continue;
            bamd_v4 xn = xr.v[c], hn;
            if (y) xn = xn + yr.v[c] * r;
            hn = xn;
            if (shifted) { bamd_v4 pv = pr.v[c]; if (yp) pv = pv + qr.v[c] * rp; hn = xn + (pv - xn) * mu.v[c]; }
            if (write) { *(bamd_v4 *) (a.xo + (size_t) row * E + i) = xn; if (so) *(bamd_v4 *) (so + i) = xn; }
            if (h) store4<T>(h + i, hn);
        }
        if (h) zero_tail(h, E, a.ldh);
        return;
    }
    float r = 0.f, rp = 0.f;
    if (y) {
        float v[2] = { 0.f, 0.f };
        for (int i = threadIdx.x; i < E; i += blockDim.x) { const float t = y[i]; v[0] += t * t; if (yp) { const float u = yp[i]; v[1] += u * u; } }
        block_sum<2>(v, red);
        const float g = a.g[0];
        r = g / sqrtf(v[0] / (float) E + a.eps); rp = g / sqrtf(v[1] / (float) E + a.eps);
    }
    for (int i = threadIdx.x; i < E; i += blockDim.x) {
        const float xn = y ? x[i] + y[i] * r : x[i];
        float hn = xn;
        if (shifted) {
            const float pv = before ? (yp ? xp[i] + yp[i] * rp : xp[i]) : (sp ? sp[i] : 0.f);
            hn = xn + (pv - xn) * a.mu[i];
        }
        if (write) { a.xo[(size_t) row * E + i] = xn; if (so) so[i] = xn; }
        if (h) h[i] = to_act<T>(hn);
    }
    if (h) zero_tail(h, E, a.ldh);
}
template <typename T>
__device__ __forceinline__ void final_row(const bamd_residual_args & a, int row, const float * gf, T * h, float * red) {
    constexpr int RC = 4;
    const int E = a.E;
    const float * x = a.x + (size_t) row * E, * y = a.y ? a.y + (size_t) row * a.ldy : nullptr;
    float v[1] = { 0.f }, w[1] = { 0.f };
    if (RowRegs<RC>::fits(E)) {
        RowRegs<RC> xr, yr;
        xr.load(x, E);
        if (y) {
            yr.load(y, E);
            v[0] = yr.squares();
            block_sum<1>(v, red);
            const float r = a.g[0] / sqrtf(v[0] / (float) E + a.eps);
#pragma unroll
            for (int c = 0; c < RC; ++c) xr.v[c] = xr.v[c] + yr.v[c] * r;
        }
        w[0] = xr.squares();
        block_sum<1>(w, red);
        const float rf = gf[0] / sqrtf(w[0] / (float) E + a.eps);
#pragma unroll
        for (int c = 0; c < RC; ++c) { const int i = RowRegs<RC>::at(c); if (i < E) store4<T>(h + i, xr.v[c] * rf); }
        zero_tail(h, E, a.ldh);
        return;
    }
    float r = 0.f;
    if (y) {
        for (int i = threadIdx.x; i < E; i += blockDim.x) v[0] += y[i] * y[i];
        block_sum<1>(v, red);
        r = a.g[0] / sqrtf(v[0] / (float) E + a.eps);
    }
    for (int i = threadIdx.x; i < E; i += blockDim.x) { const float xn = y ? x[i] + y[i] * r : x[i]; w[0] += xn * xn; }
    block_sum<1>(w, red);
    const float rf = gf[0] / sqrtf(w[0] / (float) E + a.eps);
    for (int i = threadIdx.x; i < E; i += blockDim.x) h[i] = to_act<T>((y ? x[i] + y[i] * r : x[i]) * rf);
    zero_tail(h, E, a.ldh);
}
template <typename T>
__device__ __forceinline__ void poly_row(const bamd_poly_args & a, int row, T * h, float * red) {
    constexpr int RC = 8;
    const float * z = a.z + (size_t) row * a.ldz;
    const bool fits = RowRegs<RC>::fits(a.F);
    RowRegs<RC> zr;
    float v[3] = { 0.f, 0.f, 0.f };
    if (fits) {
        zr.load(z, a.F);
#pragma unroll
        for (int c = 0; c < RC; ++c)
#pragma unroll
            for (int k = 0; k < 4; ++k) { const float t = zr.v[c][k], t2 = t * t, t3 = t2 * t; v[0] += t2; v[1] += t2 * t2; v[2] += t3 * t3; }
    } else for (int i = threadIdx.x; i < a.F; i += blockDim.x) { const float t = z[i], t2 = t * t, t3 = t2 * t; v[0] += t2; v[1] += t2 * t2; v[2] += t3 * t3; }
    block_sum<3>(v, red);
    const float n = (float) a.F;
    const float c1 = a.coef[0] / sqrtf(v[0] / n + a.eps), c2 = a.coef[1] / sqrtf(v[1] / n + a.eps), c3 = a.coef[2] / sqrtf(v[2] / n + a.eps), c0 = a.coef[3];
    if (fits) {
#pragma unroll
        for (int c = 0; c < RC; ++c) {
            const int i = RowRegs<RC>::at(c);
            if (i >= a.F) continue;
            bamd_v4 o;
#pragma unroll
            for (int k = 0; k < 4; ++k) { const float t = zr.v[c][k], t2 = t * t; o[k] = c1 * t + c2 * t2 + c3 * (t2 * t) + c0; }
            store4<T>(h + i, o);
        }
    } else for (int i = threadIdx.x; i < a.F; i += blockDim.x) { const float t = z[i], t2 = t * t; h[i] = to_act<T>(c1 * t + c2 * t2 + c3 * (t2 * t) + c0); }
    zero_tail(h, a.F, a.ldh);
}
// inv: LDS, one float per part and 16 more
template <typename T>
__device__ __forceinline__ void group_norm_row(const bamd_group_norm_args & a, int row, T * h, float * inv) {
    constexpr int RC = 4;
    const float * y = a.y + (size_t) row * a.ldy;
    const int per = a.n / a.groups, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6, wp = nw / a.groups;      // wp: waves per part
    if (wp >= 1 && nw % a.groups == 0 && (per & 3) == 0 && per <= wp * 256 * RC) {
        const int g = wave / wp, base = g * per, at0 = ((wave % wp) * 64 + lane) * 4, by = wp * 256;
        bamd_v4 v[RC]; float t = 0.f;
#pragma unroll
        for (int c = 0; c < RC; ++c) {
            v[c] = at0 + c * by < per ? *(const bamd_v4 *) (y + base + at0 + c * by) : bamd_v4{ 0, 0, 0, 0 };
#pragma unroll
            for (int k = 0; k < 4; ++k) t += v[c][k] * v[c][k];
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) t += __shfl_xor(t, o);
        __syncthreads();
        if (lane == 0) inv[wave] = t;
        __syncthreads();
        float sum = 0.f;
        for (int w = 0; w < wp; ++w) sum += inv[g * wp + w];
        const float r = 1.0f / sqrtf(sum / (float) per + a.eps);
#pragma unroll
        for (int c = 0; c < RC; ++c) { const int i = at0 + c * by; if (i < per) store4<T>(h + base + i, v[c] * r * *(const bamd_v4 *) (a.w + base + i)); }
        zero_tail(h, a.n, a.ldh);
        return;
    }
    if (a.groups >= nw) {                                        // parts are taken by waves in turn
        for (int g = wave; g < a.groups; g += nw) {
            float v = 0.f;
            for (int i = lane; i < per; i += 64) { const float t = y[g * per + i]; v += t * t; }
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
            if (lane == 0) inv[g] = 1.0f / sqrtf(v / (float) per + a.eps);
        }
        __syncthreads();
    } else {
        for (int g = 0; g < a.groups; ++g) {
            float v[1] = { 0.f };
            for (int i = threadIdx.x; i < per; i += blockDim.x) { const float t = y[g * per + i]; v[0] += t * t; }
            block_sum<1>(v, inv + a.groups);
            if (threadIdx.x == 0) inv[g] = 1.0f / sqrtf(v[0] / (float) per + a.eps);
        }
        __syncthreads();
    }
    for (int i = threadIdx.x; i < a.n; i += blockDim.x) h[i] = to_act<T>(y[i] * inv[i / per] * a.w[i]);
    zero_tail(h, a.n, a.ldh);
}
