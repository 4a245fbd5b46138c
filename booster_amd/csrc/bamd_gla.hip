// bamd_gla.hip — gated linear attention: per head a state S [key channels][value columns], S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, everything in 32-bit.
//   decoding: one launch; a block owns some value columns of a head's state, computes the head's decays and reads and writes its part of the state once;
//   prompts: the decays of all tokens (gla_alpha_kernel), then scans.  The tokens of a sequence are a dependent chain, so that a long portion is cut into segments: every segment but
//     the last is scanned alone without outputs (gla_segment_kernel), the states at the segments' starts follow from the segments' results and decay products
//     (gla_join_kernel), and all segments are scanned at once from those (gla_scan_kernel).
#include "bamd_gla_device.h"

// alpha [rows][heads x Np]; block (256 channels, eight rows)
#define GLA_STRIP 8
__global__ void __launch_bounds__(256) gla_alpha_kernel(bamd_gla_args a, int rows) {
    extern __shared__ __align__(16) float low[];                   // [rank][GLA_STRIP]
    const int ch = a.heads * a.Np, c = blockIdx.x * 256 + threadIdx.x, row0 = blockIdx.y * GLA_STRIP;
    for (int i = threadIdx.x; i < a.rank * GLA_STRIP; i += 256) { const int r = i / GLA_STRIP, row = row0 + i % GLA_STRIP; low[i] = row < rows ? a.in[(size_t) row * a.ld + a.t_off + r] : 0.f; }
    __syncthreads();
    if (c >= ch) return;
    float z[GLA_STRIP];
    const float bias = a.a2b[c];
#pragma unroll
    for (int i = 0; i < GLA_STRIP; ++i) z[i] = bias;
    for (int r = 0; r < a.rank; ++r) {
        const float w = bf_f(a.a2[(size_t) r * ch + c]);
#pragma unroll
        for (int i = 0; i < GLA_STRIP; ++i) z[i] = fmaf(w, low[r * GLA_STRIP + i], z[i]);
    }
#pragma unroll
    for (int i = 0; i < GLA_STRIP; ++i) if (row0 + i < rows) a.alpha[(size_t) (row0 + i) * ch + c] = gla_alpha(z[i], a.inv_tau);
}
__device__ __forceinline__ size_t gla_head(const bamd_gla_args & a, size_t i, int h) { return (i * a.heads + h) * a.Np * a.Pp; }
// block (column block, head, segment).  many: the segments' first states lie in seg_state
template <int PT, int NPL, int MODE>
__global__ void __launch_bounds__(256) gla_scan_kernel(bamd_batch_dev b, bamd_gla_args a, const bamd_segment * segs, int many) {
    extern __shared__ __align__(16) unsigned char lds[];
    const int h = blockIdx.y, p0 = blockIdx.x * PT, z = blockIdx.z;
    const bamd_segment sg = MODE == GLA_STEP || !many ? bamd_segment{ z, 0, b.ent[z].n, z, z } : segs[z];
    const bamd_entry e = b.ent[sg.entry];
    float * st = a.state + gla_head(a, e.seq, h);
    if constexpr (MODE == GLA_STATE) {
        if (z == sg.last) return;
        gla_scan_block<PT, NPL, MODE>(a, h, p0, e.row0 + sg.t0, sg.n, sg.t0 == 0 && e.pos0 > 0 ? st : nullptr, a.seg_state + gla_head(a, z, h), a.seg_decay + ((size_t) z * a.heads + h) * a.Np, lds);
    } else {
        // a segment in front of others starts from its own place and leaves the sequence's state alone
        const bool own = sg.first == sg.last;
        const float * init = own ? (e.pos0 > 0 ? st : nullptr) : a.seg_state + gla_head(a, z, h);
        gla_scan_block<PT, NPL, MODE>(a, h, p0, e.row0 + sg.t0, sg.n, init, z == sg.last ? st : a.seg_state + gla_head(a, z, h), nullptr, lds);
    }
}
// block (1024 values of a head's state, head, first segment of an entry): seg_state becomes the state at every segment's start
__global__ void __launch_bounds__(256) gla_join_kernel(bamd_batch_dev b, bamd_gla_args a, const bamd_segment * segs) {
    const bamd_segment sg = segs[blockIdx.z];
    if ((int) blockIdx.z != sg.first || sg.first == sg.last) return;
    const bamd_entry e = b.ent[sg.entry];
    const int h = blockIdx.y, i = (blockIdx.x * 256 + threadIdx.x) * 4, n = a.Np * a.Pp;
    if (i >= n) return;
    const int r = i / a.Pp;
    bamd_v4 s = e.pos0 > 0 ? *(const bamd_v4 *) (a.state + gla_head(a, e.seq, h) + i) : bamd_v4{ 0, 0, 0, 0 };
    for (int z = sg.first; z <= sg.last; ++z) {
        bamd_v4 * p = (bamd_v4 *) (a.seg_state + gla_head(a, z, h) + i);
        bamd_v4 next = s;
        if (z < sg.last) {
            next = *p;                                             // (the first segment's scan began with the sequence's state, the others' with zero)
            if (z > sg.first) next = next + s * a.seg_decay[((size_t) z * a.heads + h) * a.Np + r];
        }
        *p = s;
        s = next;
    }
}
// block (sixteen heads, row)
template <typename T> __global__ void __launch_bounds__(256) gla_norm_kernel(bamd_gla_args a) { gla_norm_block<T>(a, blockIdx.x * 16, blockIdx.y); }
void bamd_launch_gla_norm(int act, const bamd_gla_args & a, int rows, hipStream_t s) {
    const dim3 grid((a.heads + 15) / 16, rows);
    if (act == BAMD_ACT_F32) hipLaunchKernelGGL(gla_norm_kernel<float>, grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL(gla_norm_kernel<bamd_bf>, grid, dim3(256), 0, s, a);
}

template <int PT, int MODE> static int scan_go(const bamd_batch_dev & b, const bamd_gla_args & a, const bamd_segment * segs, int n_segs, bool many, hipStream_t s) {
    constexpr int GROUPS = 4 * 64 / (PT / 4);                      // 16 (64 columns), 32, 64
    const dim3 grid((a.Pp + PT - 1) / PT, a.heads, n_segs);
    const int npl = (a.Np + GROUPS - 1) / GROUPS;
#define GLA_GO(N) do { constexpr size_t lds = GlaShape<PT, N, MODE>::lds; hipLaunchKernelGGL((gla_scan_kernel<PT, N, MODE>), grid, dim3(256), lds, s, b, a, segs, many ? 1 : 0); return 0; } while (0)
    if (npl <= 1) GLA_GO(1);
    if (npl <= 2) GLA_GO(2);
    if (npl <= 4) GLA_GO(4);
    if constexpr (PT >= 32) {
        if (npl <= 8) GLA_GO(8);
        if constexpr (PT >= 64) if (npl <= 16) GLA_GO(16);
    }
#undef GLA_GO
    return 1;
}
template <int MODE> static int scan_pick(int pt, const bamd_batch_dev & b, const bamd_gla_args & a, const bamd_segment * segs, int n_segs, bool many, hipStream_t s) {
    return pt == 16 ? scan_go<16, MODE>(b, a, segs, n_segs, many, s) : pt == 32 ? scan_go<32, MODE>(b, a, segs, n_segs, many, s) : scan_go<64, MODE>(b, a, segs, n_segs, many, s);
}
int bamd_gla_blocks(int heads, int Pp) { return (Pp + 63) / 64 * heads; }
bool bamd_gla_valid(const bamd_gla_args & a) {
    return a.Np >= 4 && a.Np <= 256 && !(a.Np & 3) && a.Pp >= 4 && !(a.Pp & 3) && a.heads >= 1 && a.rank >= 1 && a.rank <= 1024 && !((a.ld | a.q_off | a.k_off | a.v_off) & 3) && (a.g_off < 0 || !(a.g_off & 3)) && !((a.ldo | a.out_off) & 3);
}
int bamd_launch_gla(const bamd_batch_dev & b, const bamd_gla_args & a, int max_n, const bamd_segment * segs, int n_segs, hipStream_t s) {
    if (!bamd_gla_valid(a) || max_n < 1) return 1;
    // enough blocks for the chip; narrower blocks only as far as they are filled
    const long wide = (long) bamd_gla_blocks(a.heads, a.Pp) * (max_n == 1 ? b.n_entries : n_segs);
    const int pt = a.Pp <= 16 || (max_n == 1 && wide * 2 < 256) ? 16 : a.Pp <= 32 || wide < 256 ? 32 : 64;
    if (max_n == 1) return scan_pick<GLA_STEP>(pt, b, a, nullptr, b.n_entries, false, s);
    if (!a.alpha) return 1;
    const bool many = n_segs > b.n_entries;
    if (many && (!segs || !a.seg_state || !a.seg_decay)) return 1;
    hipLaunchKernelGGL(gla_alpha_kernel, dim3((a.heads * a.Np + 255) / 256, (b.rows + GLA_STRIP - 1) / GLA_STRIP), dim3(256), (size_t) a.rank * GLA_STRIP * 4, s, a, b.rows);
    if (many) {
        if (scan_pick<GLA_STATE>(pt, b, a, segs, n_segs, true, s)) return 1;
        hipLaunchKernelGGL(gla_join_kernel, dim3((a.Np * a.Pp / 4 + 255) / 256, a.heads, n_segs), dim3(256), 0, s, b, a, segs);
    }
    return scan_pick<GLA_SCAN>(pt, b, a, segs, many ? n_segs : b.n_entries, many, s);
}
