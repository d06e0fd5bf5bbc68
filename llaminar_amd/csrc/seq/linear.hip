// Linear layers with bf16 weights in matrix-unit tiles, for gfx950.
//
// Up to 16 rows (decoding): one workgroup per 16-row tile of W, its wavefronts dealing the
// k-steps among themselves and summing through LDS; each weight byte is read once, a contiguous
// kilobyte per load instruction, several in flight per wavefront.  The rows of A are the second
// matrix operand (16 columns, those past M ignored).  HBM-bound.
// More rows (prompts): 128x128 or 64x64 tiles, both operands staged through LDS, double buffered.
#include "linear.h"

namespace llamql
{
    // ---- up to 16 rows ------------------------------------------------------------------------
    // RT tiles of W per workgroup (2 for a gate tile beside its up tile, or to share the rows), NW wavefronts, U k-steps
    // in flight per wavefront.  NORM: A is fp32, normed by the workgroup into LDS (as T) while the
    // first weights are on their way.
    template <typename T, int NW, int RT, bool NORM>
    __device__ __forceinline__ void linear_small_tile(const LinearArgs &p, int block)
    {
        using O = Operand<T>;
        using V = typename O::V;
        constexpr int U = RT == 1 ? 8 : 4;
        constexpr int LPAD = 16 / sizeof(T); // between LDS rows: the rows start in different banks
        extern __shared__ __attribute__((aligned(16))) char smem[];
        __shared__ __attribute__((aligned(16))) float s_red[NW][RT][64][4];
        __shared__ float s_sum[NW];
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
        const int n = lane & 15, g = lane >> 4;
        const int z = blockIdx.y;
        const int ksteps = p.K >> 5;

        const u32x4 *w[RT];
#pragma unroll
        for (int t = 0; t < RT; ++t)
            w[t] = weight_tile(static_cast<const bf16 *>(p.w) + (size_t)z * p.w_stride - (t && (block * RT + t) * 16 >= p.N ? (size_t)ksteps * 512 : 0), (size_t)block * RT + t, ksteps, lane);
        u32x4 next[RT][U];
        auto fetch = [&](int s0) __attribute__((always_inline)) {
#pragma unroll
            for (int u = 0; u < U; ++u)
            {
                const int s = s0 + u * NW;
#pragma unroll
                for (int t = 0; t < RT; ++t)
                    next[t][u] = w[t][(size_t)(s < ksteps ? s : wave < ksteps ? wave : 0) * 64];
            }
        };
        fetch(wave);

        const T *arow;
        if (NORM)
        {
            T *h = reinterpret_cast<T *>(smem);
            const int ldh = p.K + LPAD;
            for (int m = 0; m < p.M; ++m)
            {
                const f32x4 *x = reinterpret_cast<const f32x4 *>(static_cast<const float *>(p.a) + (size_t)m * p.lda);
                float sum = 0.0f;
                for (int i = threadIdx.x; i < p.K / 4; i += NW * 64)
                {
                    const f32x4 v = x[i];
                    sum += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
                }
                sum = block_sum<NW * 64>(sum, s_sum);
                const float inv = 1.0f / sqrtf(sum / (float)p.k_real + p.eps);
                typedef T t4 __attribute__((ext_vector_type(4)));
                for (int i = threadIdx.x; i < p.K / 4; i += NW * 64)
                {
                    const f32x4 v = x[i] * inv * reinterpret_cast<const f32x4 *>(p.norm)[i];
                    const t4 o = __builtin_convertvector(v, t4);
                    *reinterpret_cast<t4 *>(h + (size_t)m * ldh + 4 * i) = o;
                    if (p.h_out && block == 0)
                        *reinterpret_cast<t4 *>(static_cast<T *>(p.h_out) + (size_t)m * p.K + 4 * i) = o;
                }
            }
            __syncthreads();
            arow = h + (size_t)(n < p.M ? n : 0) * ldh + 8 * g;
        }
        else
            arow = static_cast<const T *>(p.a) + (size_t)z * p.a_stride + (size_t)(n < p.M ? n : 0) * p.lda + 8 * g;

        f32x4 acc[RT];
#pragma unroll
        for (int t = 0; t < RT; ++t)
            acc[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        for (int s0 = wave; s0 < ksteps; s0 += NW * U)
        {
            u32x4 cur[RT][U];
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int t = 0; t < RT; ++t)
                    cur[t][u] = next[t][u];
            if (s0 + NW * U < ksteps)
                fetch(s0 + NW * U);
#pragma unroll
            for (int u = 0; u < U; ++u)
            {
                const int s = s0 + u * NW;
                if (s < ksteps)
                {
                    const V b = O::load(arow + s * 32);
#pragma unroll
                    for (int t = 0; t < RT; ++t)
                        acc[t] = O::mma(O::from_weights(cur[t][u]), b, acc[t]);
                }
            }
        }
#pragma unroll
        for (int t = 0; t < RT; ++t)
            *reinterpret_cast<f32x4 *>(s_red[wave][t][lane]) = acc[t];
        __syncthreads();
        if (threadIdx.x < 64 && n < p.M)
        {
            f32x4 sum[RT];
#pragma unroll
            for (int t = 0; t < RT; ++t)
            {
                sum[t] = *reinterpret_cast<const f32x4 *>(s_red[0][t][lane]);
#pragma unroll
                for (int v = 1; v < NW; ++v)
                    sum[t] = sum[t] + *reinterpret_cast<const f32x4 *>(s_red[v][t][lane]);
            }
            const size_t elem = p.out == LLAM_SEQ_OUT_F32 || p.out == LLAM_SEQ_OUT_ADD ? 4 : sizeof(T);
            char *y = static_cast<char *>(p.y) + (size_t)z * p.y_stride * elem;
            if (RT == 2 && is_gated(p.out))
                store4<T>(p, y, n, block * 16 + 4 * g, gated4(p, sum[0], sum[RT - 1]));
            else
            {
                // (the last tile of an odd number of them is a copy)
#pragma unroll
                for (int t = 0; t < RT; ++t)
                    if ((block * RT + t) * 16 < p.N)
                        store4<T>(p, y, n, (block * RT + t) * 16 + 4 * g, sum[t]);
            }
        }
    }

    template <typename T, int NW, int RT, bool NORM>
    __global__ void __launch_bounds__(NW * 64)
        linear_small_kernel(LinearArgs p)
    {
        linear_small_tile<T, NW, RT, NORM>(p, blockIdx.x);
    }

    // Two layers over the same rows: the first `blocks` workgroups belong to p.
    template <typename T, int NW, bool NORM>
    __global__ void __launch_bounds__(NW * 64)
        linear_small_pair_kernel(LinearArgs p, LinearArgs second, int blocks)
    {
        const bool other = (int)blockIdx.x >= blocks;
        linear_small_tile<T, NW, 2, NORM>(other ? second : p, other ? (int)blockIdx.x - blocks : (int)blockIdx.x);
    }

    namespace
    {
        template <typename T, int NW, int RT, bool NORM>
        bool small_launch(const char *fn, const LinearArgs &a, int batch, hipStream_t st)
        {
            static LdsGrant grant;
            const size_t lds = NORM ? (size_t)a.M * (a.K + 16 / sizeof(T)) * sizeof(T) : 0;
            if (lds > 32 * 1024 && allow_lds(grant, reinterpret_cast<const void *>(&linear_small_kernel<T, NW, RT, NORM>), 64 * 1024) != hipSuccess)
                return fail(fn, "cannot reserve %zu bytes of LDS", lds);
            hipLaunchKernelGGL((linear_small_kernel<T, NW, RT, NORM>), dim3(a.N / 16 / RT, batch), dim3(NW * 64), lds, st, a);
            return launched(fn);
        }
        template <typename T>
        bool small_dispatch(const char *fn, const LinearArgs &a, int batch, hipStream_t st)
        {
            const bool gated = is_gated(a.out);
            const bool wide = a.K >= 1024;
            if (a.norm)
                return gated ? small_launch<T, 8, 2, true>(fn, a, batch, st) : small_launch<T, 8, 1, true>(fn, a, batch, st);
            if (gated)
                return small_launch<T, 8, 2, false>(fn, a, batch, st);
            return wide ? small_launch<T, 8, 1, false>(fn, a, batch, st) : small_launch<T, 4, 1, false>(fn, a, batch, st);
        }
    } // namespace

    namespace
    {
        template <typename T, bool NORM>
        bool small_pair_launch(const char *fn, const LinearArgs &a, const LinearArgs &b, hipStream_t st)
        {
            static LdsGrant grant;
            const size_t lds = NORM ? (size_t)a.M * (a.K + 16 / sizeof(T)) * sizeof(T) : 0;
            if (lds > 32 * 1024 && allow_lds(grant, reinterpret_cast<const void *>(&linear_small_pair_kernel<T, 8, NORM>), 64 * 1024) != hipSuccess)
                return fail(fn, "cannot reserve %zu bytes of LDS", lds);
            const int blocks = ceil_div(a.N, 32);
            hipLaunchKernelGGL((linear_small_pair_kernel<T, 8, NORM>), dim3(blocks + ceil_div(b.N, 32)), dim3(512), lds, st, a, b, blocks);
            return launched(fn);
        }
        template <typename T>
        bool small_pair_dispatch(const char *fn, const LinearArgs &a, const LinearArgs &b, hipStream_t st)
        {
            return a.norm ? small_pair_launch<T, true>(fn, a, b, st) : small_pair_launch<T, false>(fn, a, b, st);
        }
    } // namespace

    bool linear_small(const char *fn, const LinearArgs &a, int batch, int dtype, hipStream_t st)
    {
        return dtype == LLAM_SEQ_F32 ? small_dispatch<float>(fn, a, batch, st) : small_dispatch<bf16>(fn, a, batch, st);
    }

    // ---- more rows ------------------------------------------------------------------------------
    // Workgroup tile BM rows of A x BN rows of W, four wavefronts in 2 x 2, 64 columns of K per turn.
    // W is the first operand, so a lane ends with four neighbouring output columns of one row.
    // LDS: W tiles as they lie in memory (a lane's piece at lane * 16: no bank conflicts), A rows
    // with their 16-byte pieces permuted by the row (xor), so that 16 rows read 16 bank groups.
    constexpr int GEMM_BK = 64;
    constexpr int GEMM_THREADS = 256;

    template <typename T, int BM, int BN>
    __global__ void __launch_bounds__(GEMM_THREADS)
        linear_tiled_kernel(LinearArgs p, int m_tiles, int n_tiles)
    {
        using O = Operand<T>;
        using V = typename O::V;
        constexpr int APIECES = GEMM_BK * sizeof(T) / 16; // 16-byte pieces of a row
        constexpr int ALOADS = BM * APIECES / GEMM_THREADS;
        constexpr int WLOADS = BN * (GEMM_BK * 2 / 16) / GEMM_THREADS;
        constexpr int ABYTES = BM * GEMM_BK * sizeof(T), WBYTES = BN * GEMM_BK * 2;
        constexpr int TM = BM / 32, TN = BN / 32; // 16-row tiles of a wavefront
        extern __shared__ __attribute__((aligned(16))) char smem[];
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
        const int c = lane & 15, g = lane >> 4;
        const int wm = wave & 1, wn = wave >> 1;

        // neighbouring tiles (all rows of A for one stretch of W) go to one die: blocks are dealt
        // round robin over the eight dies
        const int total = m_tiles * n_tiles;
        int id = blockIdx.x;
        const int per = total / 8;
        if (id < per * 8)
            id = (id & 7) * per + (id >> 3);
        const int nt = id / m_tiles, mt = id - nt * m_tiles;
        const int z = blockIdx.y;
        int row0 = 0, rows = p.M;
        if (p.group_offset)
        {
            row0 = p.group_offset[z];
            rows = p.group_offset[z + 1] - row0;
        }
        if (mt * BM >= rows)
            return;
        const T *abase = static_cast<const T *>(p.a) + (size_t)z * p.a_stride;
        const bf16 *wbase = static_cast<const bf16 *>(p.w) + (size_t)z * p.w_stride;
        const int ksteps = p.K >> 5, w_tiles = p.N >> 4;

        const u32x4 *asrc[ALOADS];
        int adst[ALOADS];
#pragma unroll
        for (int i = 0; i < ALOADS; ++i)
        {
            const int q = threadIdx.x + i * GEMM_THREADS, r = q / APIECES, piece = q % APIECES;
            int m = mt * BM + r;
            m = row0 + (m < rows ? m : rows - 1);
            if (p.row_source)
                m = p.row_source[m] / p.source_div;
            asrc[i] = reinterpret_cast<const u32x4 *>(abase + (size_t)m * p.lda) + piece;
            adst[i] = r * APIECES + (piece ^ (r & (APIECES - 1)));
        }
        const u32x4 *wsrc[WLOADS];
#pragma unroll
        for (int i = 0; i < WLOADS; ++i)
        {
            const int q = threadIdx.x + i * GEMM_THREADS, t = q >> 7; // a tile's two k-steps: 128 pieces
            int tile = nt * (BN / 16) + t;
            tile = tile < w_tiles ? tile : w_tiles - 1;
            wsrc[i] = reinterpret_cast<const u32x4 *>(wbase) + (size_t)tile * ksteps * 64 + (q & 127);
        }
        u32x4 areg[ALOADS], wreg[WLOADS];
        auto fetch = [&](int kt) __attribute__((always_inline)) {
#pragma unroll
            for (int i = 0; i < ALOADS; ++i)
                areg[i] = asrc[i][(size_t)kt * APIECES];
#pragma unroll
            for (int i = 0; i < WLOADS; ++i)
                wreg[i] = wsrc[i][(size_t)kt * 128];
        };
        auto put = [&](int buf) __attribute__((always_inline)) {
            u32x4 *sa = reinterpret_cast<u32x4 *>(smem + buf * (ABYTES + WBYTES));
            u32x4 *sw = reinterpret_cast<u32x4 *>(smem + buf * (ABYTES + WBYTES) + ABYTES);
#pragma unroll
            for (int i = 0; i < ALOADS; ++i)
                sa[adst[i]] = areg[i];
#pragma unroll
            for (int i = 0; i < WLOADS; ++i)
                sw[threadIdx.x + i * GEMM_THREADS] = wreg[i];
        };
        f32x4 acc[TN][TM];
#pragma unroll
        for (int j = 0; j < TN; ++j)
#pragma unroll
            for (int i = 0; i < TM; ++i)
                acc[j][i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};

        const int turns = p.K / GEMM_BK;
        fetch(0);
        put(0);
        __syncthreads();
        for (int kt = 0; kt < turns; ++kt)
        {
            if (kt + 1 < turns)
                fetch(kt + 1);
            const u32x4 *sa = reinterpret_cast<const u32x4 *>(smem + (kt & 1) * (ABYTES + WBYTES));
            const u32x4 *sw = reinterpret_cast<const u32x4 *>(smem + (kt & 1) * (ABYTES + WBYTES) + ABYTES);
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
            {
                V a[TM];
#pragma unroll
                for (int i = 0; i < TM; ++i)
                {
                    const int r = wm * (BM / 2) + i * 16 + c;
                    if constexpr (sizeof(T) == 2)
                        a[i] = __builtin_bit_cast(bf16x8, sa[r * APIECES + ((ks * 4 + g) ^ (r & (APIECES - 1)))]);
                    else
                    {
                        const f32x4 lo = __builtin_bit_cast(f32x4, sa[r * APIECES + ((ks * 8 + 2 * g) ^ (r & (APIECES - 1)))]);
                        const f32x4 hi = __builtin_bit_cast(f32x4, sa[r * APIECES + ((ks * 8 + 2 * g + 1) ^ (r & (APIECES - 1)))]);
                        a[i] = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
                    }
                }
#pragma unroll
                for (int j = 0; j < TN; ++j)
                {
                    const V w = O::from_weights(sw[(wn * TN + j) * 128 + ks * 64 + lane]);
#pragma unroll
                    for (int i = 0; i < TM; ++i)
                        acc[j][i] = O::mma(w, a[i], acc[j][i]);
                }
            }
            if (kt + 1 < turns)
                put((kt + 1) & 1);
            __syncthreads();
        }

        const size_t elem = p.out == LLAM_SEQ_OUT_F32 || p.out == LLAM_SEQ_OUT_ADD ? 4 : sizeof(T);
        char *y = static_cast<char *>(p.y) + (size_t)z * p.y_stride * elem;
#pragma unroll
        for (int i = 0; i < TM; ++i)
        {
            const int m = mt * BM + wm * (BM / 2) + i * 16 + c;
            if (m >= rows)
                continue;
            if (is_gated(p.out))
            {
#pragma unroll
                for (int j = 0; j < TN; j += 2)
                {
                    const int tile = nt * (BN / 16) + wn * TN + j;
                    if (tile < w_tiles)
                        store4<T>(p, y, row0 + m, tile * 8 + 4 * g, gated4(p, acc[j][i], acc[j + 1][i]));
                }
            }
            else
            {
#pragma unroll
                for (int j = 0; j < TN; ++j)
                {
                    const int tile = nt * (BN / 16) + wn * TN + j;
                    if (tile < w_tiles)
                        store4<T>(p, y, row0 + m, tile * 16 + 4 * g, acc[j][i]);
                }
            }
        }
    }

    namespace
    {
        template <typename T, int BM, int BN>
        bool tiled_launch(const char *fn, const LinearArgs &a, int batch, hipStream_t st)
        {
            static LdsGrant grant;
            constexpr size_t lds = 2 * (BM * GEMM_BK * sizeof(T) + BN * GEMM_BK * 2);
            if (lds > 64 * 1024 && allow_lds(grant, reinterpret_cast<const void *>(&linear_tiled_kernel<T, BM, BN>), lds) != hipSuccess)
                return fail(fn, "cannot reserve %zu bytes of LDS", lds);
            const int mt = ceil_div(a.M, BM), nt = ceil_div(a.N, BN);
            hipLaunchKernelGGL((linear_tiled_kernel<T, BM, BN>), dim3(mt * nt, batch), dim3(GEMM_THREADS), lds, st, a, mt, nt);
            return launched(fn);
        }
        template <typename T>
        bool tiled_dispatch(const char *fn, const LinearArgs &a, int batch, hipStream_t st)
        {
            // the wide tile wherever it still gives every compute unit a workgroup
            const long wide = (long)ceil_div(a.M, 128) * ceil_div(a.N, 128) * batch;
            return wide >= 256 ? tiled_launch<T, 128, 128>(fn, a, batch, st) : tiled_launch<T, 64, 64>(fn, a, batch, st);
        }
    } // namespace

    bool linear_tiled(const char *fn, const LinearArgs &a, int batch, int dtype, hipStream_t st)
    {
        return dtype == LLAM_SEQ_F32 ? tiled_dispatch<float>(fn, a, batch, st) : tiled_dispatch<bf16>(fn, a, batch, st);
    }
} // namespace llamql

using namespace llamql;

namespace
{
    bool linear_args(const char *fn, const llam_seq_linear_args *a, int dtype, LinearArgs &p)
    {
        if (!a || !a->d_a || !a->d_w || !a->d_y)
            return fail(fn, "null pointer");
        if (a->M < 0 || a->N < 1 || a->K < 1 || a->batch < 1 || a->batch > 65535)
            return fail(fn, "bad size (M=%d N=%d K=%d batch=%d)", a->M, a->N, a->K, a->batch);
        if (dtype != LLAM_SEQ_BF16 && dtype != LLAM_SEQ_F32)
            return fail(fn, "dtype %d", dtype);
        const int elem = dtype == LLAM_SEQ_F32 ? 4 : 2;
        const bool gated = is_gated(a->out);
        if ((a->N % (gated ? 32 : 16)) != 0 || (a->K % PAD) != 0)
            return fail(fn, "N=%d must be a multiple of %d and K=%d of %d", a->N, gated ? 32 : 16, a->K, PAD);
        if (a->out < LLAM_SEQ_OUT_F32 || a->out > LLAM_SEQ_OUT_GATED_CLAMP)
            return fail(fn, "output kind %d", a->out);
        if (a->lda < a->K || a->ldy < (gated ? a->N / 2 : a->N))
            return fail(fn, "row strides smaller than the rows");
        if (!aligned16(a->d_a) || !aligned16(a->d_w) || !aligned16(a->d_y) || ((a->lda * (a->d_norm ? 4 : elem)) % 16) != 0 ||
            (a->ldy % 4) != 0 || ((a->a_stride * elem) % 16) != 0 || ((a->w_stride * 2) % 16) != 0 || (a->y_stride % 4) != 0)
            return fail(fn, "misaligned rows");
        if (a->d_norm && (a->M > SMALL_M || a->batch != 1 || (long)a->M * a->K > NORM_FUSE_MAX || a->k_real < 1 || !aligned16(a->d_norm)))
            return fail(fn, "a fused norm takes up to %d rows and %d values, unbatched", SMALL_M, NORM_FUSE_MAX);
        p = LinearArgs{};
        p.a = a->d_a, p.w = a->d_w, p.y = a->d_y, p.bias = a->d_bias, p.norm = a->d_norm, p.h_out = a->d_h_out;
        p.eps = a->eps, p.k_real = a->k_real, p.M = a->M, p.N = a->N, p.K = a->K, p.lda = a->lda, p.ldy = a->ldy;
        p.out = a->out, p.limit = a->limit, p.a_stride = a->a_stride, p.w_stride = a->w_stride, p.y_stride = a->y_stride;
        p.source_div = 1;
        return true;
    }
} // namespace

extern "C" bool llam_seq_linear(const llam_seq_linear_args *a, int dtype, int device_id, void *stream)
{
    static const char *fn = "llam_seq_linear";
    LinearArgs p;
    if (!linear_args(fn, a, dtype, p))
        return false;
    if (a->M == 0)
        return true;
    if (!set_device(fn, device_id))
        return false;
    return a->M <= SMALL_M ? linear_small(fn, p, a->batch, dtype, as_stream(stream))
                           : linear_tiled(fn, p, a->batch, dtype, as_stream(stream));
}

extern "C" bool llam_seq_linear_pair(const llam_seq_linear_args *a, const llam_seq_linear_args *b, int dtype, int device_id, void *stream)
{
    static const char *fn = "llam_seq_linear_pair";
    LinearArgs p, q;
    if (!linear_args(fn, a, dtype, p) || !linear_args(fn, b, dtype, q))
        return false;
    if (p.M != q.M || p.K != q.K || a->batch != 1 || b->batch != 1 || !p.norm != !q.norm)
        return fail(fn, "the layers of a pair have the same rows and columns (M=%d, %d K=%d, %d)", p.M, q.M, p.K, q.K);
    if (p.M == 0)
        return true;
    if (!set_device(fn, device_id))
        return false;
    hipStream_t st = as_stream(stream);
    if (p.M <= SMALL_M)
        return dtype == LLAM_SEQ_F32 ? small_pair_dispatch<float>(fn, p, q, st) : small_pair_dispatch<bf16>(fn, p, q, st);
    return linear_tiled(fn, p, 1, dtype, st) && linear_tiled(fn, q, 1, dtype, st);
}
