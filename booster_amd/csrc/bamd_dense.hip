// bamd_dense.hip — products with dense bfloat16 matrices in the packed layout of bamd_dense.h.
//   dense_gemm_kernel: many rows (prompts).  Weight and activation tiles through two LDS stages in operand order (every LDS access is one contiguous kilobyte per
//     wave), the next stage's global loads in flight under the matrix instructions.
//   dense_mv_kernel: few rows (decoding).  The eight or sixteen waves of a block split K; every wave streams its share of a 16-row tile straight from HBM into matrix operands.  With
//     a single row the mechanism in front of the product (residual + norm + token shift or layer norms, PolyNorm, clamped gated unit, grouped norm, last norm) runs as its prologue, its weights
//     already requested.
#include "bamd_dense_device.h"

// ---- packing at load: value (row, col) of the packed matrix = src[row_off[row] + col_off[col]], zero where either is negative; row tiles go to every step-th row tile of
// a matrix of ld column blocks ------------------------------------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(64) pack_kernel(const uint16_t * src, const int32_t * row_off, const int32_t * col_off, int k_tiles, uint16_t * dst, int step, int ld) {
    const int lane = threadIdx.x, kt = blockIdx.x % k_tiles, rt = blockIdx.x / k_tiles;
    const int ro = row_off[rt * 16 + (lane & 15)];
    uint16_t * d = dst + (((size_t) rt * step * ld + kt) * 64 + lane) * 8;
    for (int i = 0; i < 8; ++i) { const int co = col_off[kt * 32 + (lane >> 4) * 8 + i]; d[i] = ro < 0 || co < 0 ? 0 : src[(size_t) ro + co]; }
}
void bamd_launch_pack(const uint16_t * src, const int32_t * row_off, const int32_t * col_off, int row_tiles, int k_tiles, uint16_t * dst, int step, int ld, hipStream_t s) {
    hipLaunchKernelGGL(pack_kernel, dim3(row_tiles * k_tiles), dim3(64), 0, s, src, row_off, col_off, k_tiles, dst, step, ld);
}

// ---- many rows --------------------------------------------------------------------------------------------------------------------------------------
// TM activation rows x TN matrix rows per block of four waves (2 x 2); KT 32-column blocks per stage
template <typename T, int TM, int TN, int KT, int OUT>
__global__ void __launch_bounds__(256) dense_gemm_kernel(bamd_dense w, const T * x, int ldx, int rows, void * out, int ldo, int n_mt, int n_nt, float limit) {
    constexpr int FB = 64 * 8 * sizeof(T);                        // bytes of one operand block (16 rows x 32 columns)
    constexpr int XT = TM / 16, WT = TN / 16, XC = XT * KT * FB / 4096, WC = WT * KT * 1024 / 4096;   // 16-byte pieces per thread and stage
    constexpr int WF = 1024;                                      // weights stay bfloat16 in LDS
    constexpr int STAGE = XT * KT * FB + WT * KT * WF;
    extern __shared__ __align__(16) unsigned char lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    // blocks of one XCD (every eighth) take neighbouring tiles: the row tiles of one column strip follow one another, so the strip's weights stay in that XCD's L2
    const int total = n_mt * n_nt;
    int id = blockIdx.x;
    { const int per = (total + 7) / 8, xcd = id & 7, k = id >> 3; id = xcd * per + k; if (k >= per || id >= total) return; }
    const int mt = id % n_mt, nt = id / n_mt, m0 = mt * TM, n0t = nt * WT;
    bamd_u4 xr[XC], wr[WC];
    auto fetch = [&](int ks) {
#pragma unroll
        for (int i = 0; i < XC; ++i) {
            const int c = tid + 256 * i, per = FB / 16, blk = c / per, in = c % per;        // piece `in` of operand block blk
            const int l = in & 63, half = in >> 6, tile = blk / KT, kt = ks * KT + blk % KT;
            int row = m0 + tile * 16 + (l & 15); row = row < rows ? row : rows - 1;
            const int k = kt * 32 + (l >> 4) * 8 + half * 4;
            xr[i] = kt < w.k_tiles ? *(const bamd_u4 *) (x + (size_t) row * ldx + k) : bamd_u4{ 0, 0, 0, 0 };
        }
#pragma unroll
        for (int i = 0; i < WC; ++i) {
            const int c = tid + 256 * i, blk = c >> 6, l = c & 63, kt = ks * KT + blk % KT;
            int tile = n0t + blk / KT; tile = tile < w.row_tiles ? tile : w.row_tiles - 1;
            wr[i] = kt < w.k_tiles ? *(const bamd_u4 *) (w.w + (((size_t) tile * w.k_tiles + kt) * 64 + l) * 8) : bamd_u4{ 0, 0, 0, 0 };
        }
    };
    auto put = [&](int st) {
        unsigned char * base = lds + st * STAGE;
#pragma unroll
        for (int i = 0; i < XC; ++i) *(bamd_u4 *) (base + (tid + 256 * i) * 16) = xr[i];
#pragma unroll
        for (int i = 0; i < WC; ++i) *(bamd_u4 *) (base + XT * KT * FB + (tid + 256 * i) * 16) = wr[i];
    };
    constexpr int MI = XT / 2, NI = WT / 2;
    const int wm = wave & 1, wn = wave >> 1;
    bamd_v4 acc[MI][NI];
#pragma unroll
    for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < NI; ++j) acc[i][j] = bamd_v4{ 0, 0, 0, 0 };
    const int nks = (w.k_tiles + KT - 1) / KT;
    fetch(0); put(0);
    __syncthreads();
    for (int ks = 0; ks < nks; ++ks) {
        if (ks + 1 < nks) fetch(ks + 1);
        const unsigned char * base = lds + (ks & 1) * STAGE;
#pragma unroll
        for (int h = 0; h < KT; ++h) {
            Frag<T> xf[MI], wf[NI];
#pragma unroll
            for (int i = 0; i < MI; ++i) {
                const unsigned char * p = base + ((wm * MI + i) * KT + h) * FB;
                if constexpr (sizeof(T) == 2) xf[i].load((const T *) (p + lane * 16));
                else { xf[i].a = *(const bamd_v4 *) (p + lane * 16); xf[i].b = *(const bamd_v4 *) (p + 1024 + lane * 16); }
            }
#pragma unroll
            for (int j = 0; j < NI; ++j) wf[j].weight(*(const bamd_u4 *) (base + XT * KT * FB + ((wn * NI + j) * KT + h) * WF + lane * 16));
#pragma unroll
            for (int i = 0; i < MI; ++i)
#pragma unroll
                for (int j = 0; j < NI; ++j) {
                    if constexpr (OUT == BAMD_OUT_ACT_T) acc[i][j] = mma(xf[i], wf[j], acc[i][j]);     // lane: four activation rows of one matrix row
                    else acc[i][j] = mma(wf[j], xf[i], acc[i][j]);                                      // lane: four matrix rows of one activation row
                }
        }
        if (ks + 1 < nks) put((ks + 1) & 1);
        __syncthreads();
    }
    const int n_lim = w.row_tiles * 16;
#pragma unroll
    for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < NI; ++j) {
            const int mb = m0 + (wm * MI + i) * 16, nb = (n0t + wn * NI + j) * 16;
            if (nb >= n_lim) continue;
            if constexpr (OUT == BAMD_OUT_ACT_T) {
                const int n = nb + (lane & 15), m = mb + (lane >> 4) * 4;
                if (n >= w.rows) continue;
#pragma unroll
                for (int k = 0; k < 4; ++k) if (m + k < rows) ((T *) out)[(size_t) n * ldo + m + k] = to_act<T>(acc[i][j][k]);
            } else if constexpr (OUT == BAMD_OUT_GLU) {           // tiles in turn: gate, up
                const int n = (nb >> 1) + (lane >> 4) * 4, m = mb + (lane & 15);
                if ((j & 1) || m >= rows) continue;
                bamd_v4 o;
#pragma unroll
                for (int k = 0; k < 4; ++k) o[k] = clamped_glu(acc[i][j][k], acc[i][j | 1][k], limit);
                store4<T>((T *) out + (size_t) m * ldo + n, o);
            } else {
                const int n = nb + (lane >> 4) * 4, m = mb + (lane & 15);
                if (m >= rows) continue;
                if constexpr (OUT == BAMD_OUT_F32) {
                    float * o = (float *) out + (size_t) m * ldo + n;
                    if (n + 3 < w.rows) *(bamd_v4 *) o = acc[i][j];
                    else for (int k = 0; k < 4; ++k) if (n + k < w.rows) o[k] = acc[i][j][k];
                } else {
                    T * o = (T *) out + (size_t) m * ldo + n;
#pragma unroll
                    for (int k = 0; k < 4; ++k) if (n + k < w.rows) o[k] = to_act<T>(acc[i][j][k]);
                }
            }
        }
}
template <typename T, int TM, int TN, int KT, int OUT>
static int gemm_go(const bamd_dense & w, const void * x, int ldx, int rows, void * out, int ldo, float limit, hipStream_t s) {
    const int n_mt = (rows + TM - 1) / TM, n_nt = (w.row_tiles + TN / 16 - 1) / (TN / 16), per = (n_mt * n_nt + 7) / 8;
    const size_t lds = 2 * ((size_t) TM / 16 * KT * 64 * 8 * sizeof(T) + (size_t) TN / 16 * KT * 1024);
    hipLaunchKernelGGL((dense_gemm_kernel<T, TM, TN, KT, OUT>), dim3(per * 8), dim3(256), lds, s, w, (const T *) x, ldx, rows, out, ldo, n_mt, n_nt, limit);
    return 0;
}
template <typename T, int OUT>
static int gemm_tiles(const bamd_dense & w, const void * x, int ldx, int rows, void * out, int ldo, float limit, hipStream_t s) {
    if constexpr (sizeof(T) == 2) if ((long) ((rows + 127) / 128) * ((w.row_tiles + 7) / 8) >= 192) return gemm_go<T, 128, 128, 2, OUT>(w, x, ldx, rows, out, ldo, limit, s);
    return gemm_go<T, 64, 64, sizeof(T) == 2 ? 4 : 2, OUT>(w, x, ldx, rows, out, ldo, limit, s);
}
// f32 rows are stored four matrix rows at a time: ldo % 4 == 0; x rows start on 16 bytes and hold k_tiles * 32 columns
template <typename T>
static int gemm_out(const bamd_dense & w, const void * x, int ldx, int rows, void * out, int ldo, int kind, float limit, hipStream_t s) {
    switch (kind) {
        case BAMD_OUT_F32: return gemm_tiles<T, BAMD_OUT_F32>(w, x, ldx, rows, out, ldo, limit, s);
        case BAMD_OUT_ACT: return gemm_tiles<T, BAMD_OUT_ACT>(w, x, ldx, rows, out, ldo, limit, s);
        case BAMD_OUT_ACT_T: return gemm_tiles<T, BAMD_OUT_ACT_T>(w, x, ldx, rows, out, ldo, limit, s);
        case BAMD_OUT_GLU: return (w.row_tiles & 1) || ldo < w.row_tiles * 8 ? 1 : gemm_tiles<T, BAMD_OUT_GLU>(w, x, ldx, rows, out, ldo, limit, s);
    }
    return 1;
}
int bamd_launch_dense_gemm(int act, const bamd_dense & w, const void * x, int ldx, int rows, void * out, int ldo, int kind, hipStream_t s, float limit) {
    if (rows < 1 || w.row_tiles < 1 || w.k_tiles < 1 || ldx < w.k_tiles * 32 || (ldx & 7) || (ldo & 3)) return 1;
    return act == BAMD_ACT_F32 ? gemm_out<float>(w, x, ldx, rows, out, ldo, kind, limit, s) : gemm_out<bamd_bf>(w, x, ldx, rows, out, ldo, kind, limit, s);
}

// ---- few rows ---------------------------------------------------------------------------------------------------------------------------------------
// NT: groups of 16 rows; NW: waves; U: 32-column blocks per request batch of a wave
template <typename T, int NT, int NW, int PRE>
__global__ void __launch_bounds__(64 * NW) dense_mv_kernel(bamd_dense w, bamd_batch_dev b, bamd_pre_args p, const T * x, int ldx, int rows, float * out, int ldo) {
    constexpr int U = sizeof(T) == 2 ? 8 : 4;
    extern __shared__ __align__(16) unsigned char lds[];
    __shared__ float red[NW * NT * 256];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int k0 = w.k_tiles * wave / NW, k1 = w.k_tiles * (wave + 1) / NW, kn = (w.k_tiles + NW - 1) / NW, nc = (kn + U - 1) / U;
    bamd_u4 cur[U], nxt[U] = {};
    auto request = [&](int tile, int c, bamd_u4 * d) {
        const uint16_t * base = w.w + ((size_t) tile * w.k_tiles * 64 + lane) * 8;
#pragma unroll
        for (int u = 0; u < U; ++u) { int kt = k0 + c * U + u; kt = kt < w.k_tiles ? kt : w.k_tiles - 1; d[u] = *(const bamd_u4 *) (base + (size_t) kt * 512); }
    };
    int tile = blockIdx.x;
    request(tile, 0, cur);                                        // on their way while the operand row is built
    if constexpr (PRE != BAMD_PRE_ROWS) {
        T * h = (T *) lds;
        if constexpr (PRE == BAMD_PRE_RESIDUAL) residual_row<T, true>(b, p.res, 0, h, blockIdx.x == 0, red);
        if constexpr (PRE == BAMD_PRE_POLY) poly_row<T>(p.poly, 0, h, red);
        if constexpr (PRE == BAMD_PRE_GROUP) group_norm_row<T>(p.grp, 0, h, red);
        if constexpr (PRE == BAMD_PRE_GLU) glu_row<T>(p.glu, 0, h, 0, p.glu.ldh);
        if constexpr (PRE == BAMD_PRE_LAYER) layer_row<T>(p.res, p.want ? p.want[0] : 0, p.want ? p.gf : p.res.gi, h, !p.want && blockIdx.x == 0, red);
        if constexpr (PRE == BAMD_PRE_FINAL) final_row<T>(p.res, p.want[0], p.gf, h, red);
        __syncthreads();
    }
    const int col = lane & 15, kq = (lane >> 4) * 8;
    for (; tile < w.row_tiles; tile += gridDim.x) {
        bamd_v4 acc[NT];
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[n] = bamd_v4{ 0, 0, 0, 0 };
        for (int c = 0; c < nc; ++c) {
            const bool more = c + 1 < nc;
            if (more) request(tile, c + 1, nxt);
            else if (tile + (int) gridDim.x < w.row_tiles) request(tile + gridDim.x, 0, nxt);
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int kt = k0 + c * U + u;
                if (kt < k1) {
                    Frag<T> wf; wf.weight(cur[u]);
#pragma unroll
                    for (int n = 0; n < NT; ++n) {
                        Frag<T> xf;
                        if constexpr (PRE != BAMD_PRE_ROWS) xf.load((const T *) lds + kt * 32 + kq);
                        else { int r = n * 16 + col; r = r < rows ? r : rows - 1; xf.load(x + (size_t) r * ldx + kt * 32 + kq); }
                        acc[n] = mma(wf, xf, acc[n]);
                    }
                }
            }
#pragma unroll
            for (int u = 0; u < U; ++u) cur[u] = nxt[u];
        }
        __syncthreads();                                          // (the sums of the tile before are read)
#pragma unroll
        for (int n = 0; n < NT; ++n) *(bamd_v4 *) (red + ((wave * NT + n) * 64 + lane) * 4) = acc[n];
        __syncthreads();
        for (int i = tid; i < NT * 256; i += 64 * NW) {
            const int n = i >> 8, l = (i >> 2) & 63, k = i & 3, r = n * 16 + (l & 15), o = tile * 16 + (l >> 4) * 4 + k;
            if (r < rows && o < w.rows) {
                float v = 0.f;
#pragma unroll
                for (int q = 0; q < NW; ++q) v += red[((q * NT + n) * 64 + l) * 4 + k];
                out[(size_t) r * ldo + o] = v;
            }
        }
    }
}
size_t bamd_dense_mv_lds(int act, int K) { return (size_t) (K + 31) / 32 * 32 * (act == BAMD_ACT_F32 ? 4 : 2); }
template <typename T, int NT, int NW, int PRE>
static void mv_go(const bamd_dense & w, const bamd_batch_dev & b, const bamd_pre_args & p, const void * x, int ldx, int rows, float * out, int ldo, hipStream_t s) {
    const int grid = w.row_tiles < 4096 / NW ? w.row_tiles : 4096 / NW;       // what is resident at once; blocks walk the tiles
    const size_t lds = PRE == BAMD_PRE_ROWS ? 0 : bamd_dense_mv_lds(sizeof(T) == 4 ? BAMD_ACT_F32 : BAMD_ACT_BF16, w.k_tiles * 32);
    hipLaunchKernelGGL((dense_mv_kernel<T, NT, NW, PRE>), dim3(grid), dim3(64 * NW), lds, s, w, b, p, (const T *) x, ldx, rows, out, ldo);
}
// sixteen waves where the tiles alone would leave the chip half empty
template <typename T, int PRE>
static void mv_one(const bamd_dense & w, const bamd_batch_dev & b, const bamd_pre_args & p, const void * x, int ldx, int rows, float * out, int ldo, hipStream_t s) {
    if (w.row_tiles <= 256) mv_go<T, 1, 16, PRE>(w, b, p, x, ldx, rows, out, ldo, s);
    else mv_go<T, 1, 8, PRE>(w, b, p, x, ldx, rows, out, ldo, s);
}
template <typename T>
static int mv_pick(const bamd_dense & w, int pre, const bamd_batch_dev & b, const bamd_pre_args & p, const void * x, int ldx, int rows, float * out, int ldo, hipStream_t s) {
    if (pre != BAMD_PRE_ROWS) {
        if (rows != 1 || bamd_dense_mv_lds(sizeof(T) == 4 ? BAMD_ACT_F32 : BAMD_ACT_BF16, w.k_tiles * 32) > BAMD_MV_LDS) return 1;
        const int ldh = pre == BAMD_PRE_POLY ? p.poly.ldh : pre == BAMD_PRE_GROUP ? p.grp.ldh : pre == BAMD_PRE_GLU ? p.glu.ldh : p.res.ldh;
        if (ldh != w.k_tiles * 32) return 1;
        if (pre == BAMD_PRE_RESIDUAL && p.res.norm != BAMD_NORM_LAYER) mv_one<T, BAMD_PRE_RESIDUAL>(w, b, p, x, ldx, rows, out, ldo, s);
        else if (pre == BAMD_PRE_POLY) mv_one<T, BAMD_PRE_POLY>(w, b, p, x, ldx, rows, out, ldo, s);
        else if (pre == BAMD_PRE_GROUP) mv_one<T, BAMD_PRE_GROUP>(w, b, p, x, ldx, rows, out, ldo, s);
        else if (pre == BAMD_PRE_GLU) mv_one<T, BAMD_PRE_GLU>(w, b, p, x, ldx, rows, out, ldo, s);
        else if (p.res.norm == BAMD_NORM_LAYER) mv_one<T, BAMD_PRE_LAYER>(w, b, p, x, ldx, rows, out, ldo, s);
        else mv_one<T, BAMD_PRE_FINAL>(w, b, p, x, ldx, rows, out, ldo, s);
        return 0;
    }
    if (rows < 1 || rows > BAMD_MV_ROWS || ldx < w.k_tiles * 32 || (ldx & 7)) return 1;
    if (rows <= 16) mv_one<T, BAMD_PRE_ROWS>(w, b, p, x, ldx, rows, out, ldo, s);
    else if (rows <= 32) mv_go<T, 2, 8, BAMD_PRE_ROWS>(w, b, p, x, ldx, rows, out, ldo, s);
    else mv_go<T, 4, 8, BAMD_PRE_ROWS>(w, b, p, x, ldx, rows, out, ldo, s);
    return 0;
}
int bamd_launch_dense_mv(int act, const bamd_dense & w, int pre, const bamd_batch_dev & b, const bamd_pre_args * p, const void * x, int ldx, int rows, float * out, int ldo, hipStream_t s) {
    static const bamd_pre_args none = {};
    return act == BAMD_ACT_F32 ? mv_pick<float>(w, pre, b, p ? *p : none, x, ldx, rows, out, ldo, s) : mv_pick<bamd_bf>(w, pre, b, p ? *p : none, x, ldx, rows, out, ldo, s);
}
