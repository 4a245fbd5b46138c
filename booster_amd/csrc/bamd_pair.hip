// bamd_pair.hip — one decoded token through two mixers side by side, attention over cached keys and values (bamd_kv_device.h) and gated linear attention (bamd_gla_device.h): each is
// a chain of dependent reads that leaves most of the chip idle, so that their blocks share a launch — the shares of the keys and the state updates first, then the sums over
// the shares and the norms of the heads.
#include "bamd_kv_device.h"
#include "bamd_gla_device.h"

#define PAIR_PT 16
// block (attention shares x groups, then value columns x heads; row)
template <typename T, int ND, int NPL>
__global__ void __launch_bounds__(256, ND <= 4 ? 2 : 1) kv_gla_step_kernel(bamd_batch_dev b, bamd_kv_args kv, bamd_gla_args gla, float * part_o, float * part_ml, int splits, int attn) {
    extern __shared__ __align__(16) unsigned char lds[];
    const int x = blockIdx.x, row = blockIdx.y;
    if (x < attn) { kv_decode_block<T, ND>(b, kv, x / (attn / splits), splits, x % (attn / splits), row, part_o, part_ml, lds); return; }
    const int cols = (gla.Pp + PAIR_PT - 1) / PAIR_PT, i = x - attn, h = i / cols;
    const bamd_entry e = b.ent[row];
    float * st = gla.state + ((size_t) e.seq * gla.heads + h) * gla.Np * gla.Pp;
    gla_scan_block<PAIR_PT, NPL, GLA_STEP>(gla, h, (i % cols) * PAIR_PT, row, 1, e.pos0 > 0 ? st : nullptr, st, nullptr, lds);
}
// block (head of the attention, then sixteen heads of the recurrence; row)
template <typename T> __global__ void __launch_bounds__(256) kv_gla_finish_kernel(bamd_kv_args kv, bamd_gla_args gla, const float * part_o, const float * part_ml, int splits) {
    if ((int) blockIdx.x < kv.heads) kv_combine_block<T>(kv, blockIdx.x, blockIdx.y, part_o, part_ml, splits);
    else gla_norm_block<T>(gla, (blockIdx.x - kv.heads) * 16, blockIdx.y);
}

template <typename T, int ND, int NPL>
static int pair_go(const bamd_batch_dev & b, const bamd_kv_args & kv, const bamd_gla_args & gla, float * po, float * pm, int splits, hipStream_t s) {
    constexpr size_t lk = KvDecodeLds<T, ND>::bytes, lg = GlaShape<PAIR_PT, NPL, GLA_STEP>::lds, lds = lk > lg ? lk : lg;
    const int attn = splits * bamd_kv_groups(kv), cols = (gla.Pp + PAIR_PT - 1) / PAIR_PT;
    hipLaunchKernelGGL((kv_gla_step_kernel<T, ND, NPL>), dim3(attn + gla.heads * cols, b.rows), dim3(256), lds, s, b, kv, gla, po, pm, splits, attn);
    hipLaunchKernelGGL(kv_gla_finish_kernel<T>, dim3(kv.heads + (gla.heads + 15) / 16, b.rows), dim3(256), 0, s, kv, gla, po, pm, splits);
    return 0;
}
template <typename T, int ND>
static int pair_npl(const bamd_batch_dev & b, const bamd_kv_args & kv, const bamd_gla_args & gla, float * po, float * pm, int splits, hipStream_t s) {
    if (gla.Np <= 64) return pair_go<T, ND, 1>(b, kv, gla, po, pm, splits, s);
    if (gla.Np <= 128) return pair_go<T, ND, 2>(b, kv, gla, po, pm, splits, s);
    return pair_go<T, ND, 4>(b, kv, gla, po, pm, splits, s);
}
template <typename T>
static int pair_nd(const bamd_batch_dev & b, const bamd_kv_args & kv, const bamd_gla_args & gla, float * po, float * pm, int splits, hipStream_t s) {
    switch (kv.D) {
        case 32: return pair_npl<T, 1>(b, kv, gla, po, pm, splits, s);
        case 64: return pair_npl<T, 2>(b, kv, gla, po, pm, splits, s);
        case 128: return pair_npl<T, 4>(b, kv, gla, po, pm, splits, s);
        case 256: return pair_npl<T, 8>(b, kv, gla, po, pm, splits, s);
    }
    return 1;
}
int bamd_launch_kv_gla_decode(int act, const bamd_batch_dev & b, const bamd_kv_args & kv, const bamd_gla_args & gla, float * po, float * pm, int splits, hipStream_t s) {
    if (splits < 1 || splits > 64 || b.rows != b.n_entries || !bamd_kv_valid(kv) || !bamd_gla_valid(gla)) return 1;
    return act == BAMD_ACT_F32 ? pair_nd<float>(b, kv, gla, po, pm, splits, s) : pair_nd<bamd_bf>(b, kv, gla, po, pm, splits, s);
}
