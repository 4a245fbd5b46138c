// bamd_rows.hip — row-wise mechanisms of the configured layer stacks, one block per row: embedding with learned positions, residual sum with the norm of the
// sublayer's output and token shift (or layer norms in front and behind), PolyNorm, clamped gated unit, grouped norm, the model's last norm, arg-max, and the device side of the greedy loop.  With a single row the same
// device functions run as the prologue of the product behind them (bamd_dense.hip).
#include "bamd_dense_device.h"

// block (1024 columns, row)
__global__ void __launch_bounds__(256) embed_rows_kernel(bamd_batch_dev b, const uint16_t * __restrict__ embd, const uint16_t * __restrict__ pos, float scale, int E, int V, float * __restrict__ x) {
    const int row = blockIdx.y, i0 = blockIdx.x * 1024 + threadIdx.x * 4;
    int t = b.tokens[row]; t = t < 0 ? 0 : t >= V ? V - 1 : t;
    const bamd_entry e = b.ent[b.row_entry[row]];
    const int p = e.pos0 + (row - e.row0);
    const uint16_t * er = embd + (size_t) t * E, * pr = pos ? pos + (size_t) p * E : nullptr;
    if (i0 + 3 < E && (E & 3) == 0) {
        const uint2 u = *(const uint2 *) (er + i0), w = pr ? *(const uint2 *) (pr + i0) : uint2{ 0, 0 };
        *(bamd_v4 *) (x + (size_t) row * E + i0) = bamd_v4{ bf_lo(u.x) * scale + bf_lo(w.x), bf_hi(u.x) * scale + bf_hi(w.x), bf_lo(u.y) * scale + bf_lo(w.y), bf_hi(u.y) * scale + bf_hi(w.y) };
    } else for (int i = i0; i < min(i0 + 4, E); ++i) x[(size_t) row * E + i] = bf_f(er[i]) * scale + (pr ? bf_f(pr[i]) : 0.f);
}
template <typename T> __global__ void __launch_bounds__(1024) residual_rows_kernel(bamd_batch_dev b, bamd_residual_args a) {
    __shared__ float red[64];
    residual_row<T, false>(b, a, blockIdx.x, a.h ? (T *) a.h + (size_t) blockIdx.x * a.ldh : nullptr, true, red);
}
template <typename T> __global__ void __launch_bounds__(1024) final_rows_kernel(bamd_residual_args a, const int32_t * want, const float * gf) {
    __shared__ float red[64];
    final_row<T>(a, want[blockIdx.x], gf, (T *) a.h + (size_t) blockIdx.x * a.ldh, red);
}
template <typename T> __global__ void __launch_bounds__(1024) layer_rows_kernel(bamd_residual_args a, const int32_t * want, const float * gi) {
    __shared__ float red[64];
    const int row = want ? want[blockIdx.x] : blockIdx.x;
    layer_row<T>(a, row, gi, a.h ? (T *) a.h + (size_t) blockIdx.x * a.ldh : nullptr, !want, red);
}
// block (1024 columns, row)
template <typename T> __global__ void __launch_bounds__(256) glu_rows_kernel(bamd_glu_args a) { glu_row<T>(a, blockIdx.y, (T *) a.h + (size_t) blockIdx.y * a.ldh, blockIdx.x * 1024, min(a.ldh, (int) blockIdx.x * 1024 + 1024)); }
template <typename T> __global__ void __launch_bounds__(1024) poly_rows_kernel(bamd_poly_args a) {
    __shared__ float red[64];
    poly_row<T>(a, blockIdx.x, (T *) a.h + (size_t) blockIdx.x * a.ldh, red);
}
template <typename T> __global__ void __launch_bounds__(1024) group_norm_rows_kernel(bamd_group_norm_args a) {
    __shared__ float inv[BAMD_MAX_NORM_GROUPS + 16];
    group_norm_row<T>(a, blockIdx.x, (T *) a.h + (size_t) blockIdx.x * a.ldh, inv);
}
// block (part, row); keys must be zero
__global__ void __launch_bounds__(256) argmax_rows_kernel(const float * __restrict__ logits, int V, unsigned long long * keys) {
    __shared__ unsigned long long wk[4];
    const float * l = logits + (size_t) blockIdx.y * V;
    unsigned long long best = 0ull;
    for (int i = blockIdx.x * 256 + threadIdx.x; i < V; i += gridDim.x * 256) {
        const float f = l[i];
        if (f != f) continue;
        const unsigned int u = __float_as_uint(f), o = (u & 0x80000000u) ? ~u : (u | 0x80000000u);
        const unsigned long long k = ((unsigned long long) o << 32) | (0xffffffffu - (unsigned int) i);
        best = k > best ? k : best;
    }
    for (int o = 32; o > 0; o >>= 1) { const unsigned long long k = __shfl_xor(best, o); best = k > best ? k : best; }
    if ((threadIdx.x & 63) == 0) wk[threadIdx.x >> 6] = best;
    __syncthreads();
    if (threadIdx.x == 0) { for (int w = 1; w < 4; ++w) best = wk[w] > best ? wk[w] : best; if (best) atomicMax(keys + blockIdx.y, best); }
}
__global__ void __launch_bounds__(64) clear_keys_kernel(unsigned long long * keys, int n) { for (int i = threadIdx.x; i < n; i += 64) keys[i] = 0ull; }
__global__ void __launch_bounds__(64) advance_kernel(bamd_entry * ent, int32_t * tokens, unsigned long long * keys, int n, int32_t * out, int ldo, int32_t * step, int advance, int V) {
    const int i = threadIdx.x, at = step ? *step : 0;
    for (int j = i; j < n; j += 64) {
        const uint32_t id = 0xffffffffu - (uint32_t) (keys[j] & 0xffffffffull);
        const int t = id < (uint32_t) V ? (int) id : 0;
        if (out && at < ldo) out[(size_t) j * ldo + at] = t;
        if (tokens) tokens[j] = t;
        if (advance) keys[j] = 0ull;                              // for the arg-max at this step's end
        if (advance) { if (at > 0) { ent[j].pos0 += 1; ent[j].par ^= 1; } }
    }
    __syncthreads();
    if (i == 0 && step) *step = at + 1;
}

static dim3 row_block(int n) { return dim3(n > 1024 ? 1024 : 256); }
void bamd_launch_embed_rows(const bamd_batch_dev & b, const uint16_t * embd, const uint16_t * pos, float scale, int E, int V, float * x, hipStream_t s) {
    hipLaunchKernelGGL(embed_rows_kernel, dim3((E + 1023) / 1024, b.rows), dim3(256), 0, s, b, embd, pos, scale, E, V, x);
}
void bamd_launch_residual_rows(int act, const bamd_batch_dev & b, const bamd_residual_args & a, hipStream_t s) {
    if (a.norm == BAMD_NORM_LAYER) {
        if (act == BAMD_ACT_F32) hipLaunchKernelGGL(layer_rows_kernel<float>, dim3(b.rows), row_block(a.E), 0, s, a, nullptr, a.gi);
        else hipLaunchKernelGGL(layer_rows_kernel<bamd_bf>, dim3(b.rows), row_block(a.E), 0, s, a, nullptr, a.gi);
    } else if (act == BAMD_ACT_F32) hipLaunchKernelGGL(residual_rows_kernel<float>, dim3(b.rows), row_block(a.E), 0, s, b, a);
    else hipLaunchKernelGGL(residual_rows_kernel<bamd_bf>, dim3(b.rows), row_block(a.E), 0, s, b, a);
}
void bamd_launch_final_rows(int act, const bamd_residual_args & a, const int32_t * want, int n_want, const float * gf, hipStream_t s) {
    if (a.norm == BAMD_NORM_LAYER) {
        if (act == BAMD_ACT_F32) hipLaunchKernelGGL(layer_rows_kernel<float>, dim3(n_want), row_block(a.E), 0, s, a, want, gf);
        else hipLaunchKernelGGL(layer_rows_kernel<bamd_bf>, dim3(n_want), row_block(a.E), 0, s, a, want, gf);
    } else if (act == BAMD_ACT_F32) hipLaunchKernelGGL(final_rows_kernel<float>, dim3(n_want), row_block(a.E), 0, s, a, want, gf);
    else hipLaunchKernelGGL(final_rows_kernel<bamd_bf>, dim3(n_want), row_block(a.E), 0, s, a, want, gf);
}
void bamd_launch_poly_rows(int act, int rows, const bamd_poly_args & a, hipStream_t s) {
    if (act == BAMD_ACT_F32) hipLaunchKernelGGL(poly_rows_kernel<float>, dim3(rows), row_block(a.F), 0, s, a);
    else hipLaunchKernelGGL(poly_rows_kernel<bamd_bf>, dim3(rows), row_block(a.F), 0, s, a);
}
void bamd_launch_glu_rows(int act, int rows, const bamd_glu_args & a, hipStream_t s) {
    if (act == BAMD_ACT_F32) hipLaunchKernelGGL(glu_rows_kernel<float>, dim3((a.ldh + 1023) / 1024, rows), dim3(256), 0, s, a);
    else hipLaunchKernelGGL(glu_rows_kernel<bamd_bf>, dim3((a.ldh + 1023) / 1024, rows), dim3(256), 0, s, a);
}
void bamd_launch_group_norm_rows(int act, int rows, const bamd_group_norm_args & a, hipStream_t s) {
    if (act == BAMD_ACT_F32) hipLaunchKernelGGL(group_norm_rows_kernel<float>, dim3(rows), row_block(a.n), 0, s, a);
    else hipLaunchKernelGGL(group_norm_rows_kernel<bamd_bf>, dim3(rows), row_block(a.n), 0, s, a);
}
void bamd_launch_argmax_rows(const float * logits, int n, int V, unsigned long long * keys, bool clear, hipStream_t s) {
    if (clear) hipLaunchKernelGGL(clear_keys_kernel, dim3(1), dim3(64), 0, s, keys, n);
    hipLaunchKernelGGL(argmax_rows_kernel, dim3(V > 8192 ? 32 : 4, n), dim3(256), 0, s, logits, V, keys);
}
void bamd_launch_advance(bamd_entry * ent, int32_t * tokens, unsigned long long * keys, int n, int32_t * out, int ldo, int32_t * step, int advance, int V, hipStream_t s) {
    hipLaunchKernelGGL(advance_kernel, dim3(1), dim3(64), 0, s, ent, tokens, keys, n, out, ldo, step, advance, V);
}
