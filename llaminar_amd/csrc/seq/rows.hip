// Row operators of sequence models: token embedding, RMS norm, and the routed expert
// feed-forward (choice of experts, grouping of tokens by expert, weighted sum).
#include "linear.h"

namespace llamql
{
    constexpr int ROW_THREADS = 256;

    constexpr int EMBED_WIDE_ROWS = 256; // rows from which a workgroup takes a whole row
    __global__ void __launch_bounds__(ROW_THREADS)
        seq_embed_kernel(llam_seq_embed_args p, const int32_t *__restrict__ ids, float *__restrict__ x, int ldx)
    {
        const int m = blockIdx.y, id = ids[m], last = m > 0 ? ids[m - 1] : 0;
        const bool ok = id >= 0 && id < p.vocab;
        const bf16 *table = static_cast<const bf16 *>(p.d_table), *pairs = static_cast<const bf16 *>(p.d_pairs);
        long pair = -1;
        if (pairs)
        {
            const int slot = p.d_row_slot[m], pos = p.d_row_pos[m];
            int32_t *history = p.d_history + (size_t)slot * p.cap;
            if (pos == 0)
                pair = p.buckets;
            else if (pos > 0 && pos < p.cap)
            {
                const int before = m > 0 && p.d_row_slot[m - 1] == slot ? last : history[pos - 1];
                const long sum = (long)before * p.mul_prev + (long)id * p.mul_cur;
                pair = (sum >> 32) == 0 ? (long)((uint32_t)sum % (uint32_t)p.buckets) : sum % p.buckets;
            }
            if (blockIdx.x == 0 && threadIdx.x == 0 && pos >= 0 && pos < p.cap)
                history[pos] = id;
        }
        if ((p.width & 3) == 0 && (ldx & 3) == 0)
        {
            // four columns at a time
#pragma unroll 2
            for (int c = (blockIdx.x * ROW_THREADS + threadIdx.x) * 4; c < ldx; c += gridDim.x * ROW_THREADS * 4)
            {
                f32x4 v = {0.0f, 0.0f, 0.0f, 0.0f};
                if (ok && c < p.width)
                {
                    v = __builtin_convertvector(*reinterpret_cast<const bf16x4 *>(table + (size_t)id * p.width + c), f32x4) * p.scale;
                    if (pair >= 0)
                        v = v + __builtin_convertvector(*reinterpret_cast<const bf16x4 *>(pairs + (size_t)pair * p.width + c), f32x4);
                }
                *reinterpret_cast<f32x4 *>(x + (size_t)m * ldx + c) = v;
            }
            return;
        }
        for (int c = blockIdx.x * ROW_THREADS + threadIdx.x; c < ldx; c += gridDim.x * ROW_THREADS)
        {
            float v = 0.0f;
            if (ok && c < p.width)
            {
                v = (float)table[(size_t)id * p.width + c] * p.scale;
                if (pair >= 0)
                    v += (float)pairs[(size_t)pair * p.width + c];
            }
            x[(size_t)m * ldx + c] = v;
        }
    }

    template <typename T>
    __global__ void __launch_bounds__(ROW_THREADS)
        seq_rmsnorm_kernel(const float *__restrict__ x, int ldx, const int32_t *__restrict__ rows,
                           const float *__restrict__ norm, float eps, int k_real, T *__restrict__ y, int K,
                           const float *__restrict__ norm2, T *__restrict__ y2)
    {
        typedef T t4 __attribute__((ext_vector_type(4)));
        __shared__ float s_sum[ROW_THREADS / 64];
        const int m = blockIdx.x;
        const f32x4 *row = reinterpret_cast<const f32x4 *>(x + (size_t)(rows ? rows[m] : m) * ldx);
        float sum = 0.0f;
        for (int i = threadIdx.x; i < K / 4; i += ROW_THREADS)
        {
            const f32x4 v = row[i];
            sum += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        }
        sum = block_sum<ROW_THREADS>(sum, s_sum);
        const float inv = 1.0f / sqrtf(sum / (float)k_real + eps);
        for (int i = threadIdx.x; i < K / 4; i += ROW_THREADS)
        {
            const f32x4 v = row[i] * inv;
            *reinterpret_cast<t4 *>(y + (size_t)m * K + 4 * i) =
                __builtin_convertvector(v * reinterpret_cast<const f32x4 *>(norm)[i], t4);
            if (norm2)
                *reinterpret_cast<t4 *>(y2 + (size_t)m * K + 4 * i) =
                    __builtin_convertvector(v * reinterpret_cast<const f32x4 *>(norm2)[i], t4);
        }
    }

    __global__ void __launch_bounds__(64)
        seq_record_kernel(const int32_t *__restrict__ ids, int n, int32_t *__restrict__ out, int32_t *__restrict__ count,
                          int max_count)
    {
        const int k = *count;
        if (k >= max_count)
            return;
        for (int b = threadIdx.x; b < n; b += 64)
            out[(size_t)k * n + b] = ids[b];
        if (threadIdx.x == 0)
            *count = k + 1;
    }

    // ---- routed experts -------------------------------------------------------------------------
    struct ExpertArgs
    {
        const float *logits;
        int ldz;
        const bf16 *up, *down, *shared_up, *shared_down;
        long up_stride, down_stride;
        int experts, top, ff, shared_ff, K, N;
        const void *h; // T [M][K]
        float *x;
        int ldx;
        int *ids;       // [M][top]
        float *weights; // [M][top + 1]: of the chosen experts, then of the shared one
        bool routed;    // few rows: ids and weights are there already
        void *act;      // T: few rows [M][top * ff + shared_ff], many rows [M * top][ff] then [M][shared_ff]
    };

    // A wavefront per token chooses its experts.
    __global__ void __launch_bounds__(ROW_THREADS)
        expert_route_kernel(ExpertArgs p, int M)
    {
        const int lane = threadIdx.x & 63, m = blockIdx.x * (ROW_THREADS / 64) + (threadIdx.x >> 6);
        if (m >= M)
            return;
        const float *z = p.logits + (size_t)m * p.ldz;
        int id;
        float weight;
        route_wave(z, p.experts, p.top, lane, id, weight);
        if (lane < p.top)
        {
            p.ids[m * p.top + lane] = id;
            p.weights[m * (p.top + 1) + lane] = weight;
        }
        if (lane == 0 && p.shared_ff)
            p.weights[m * (p.top + 1) + p.top] = sigmoidf(z[p.experts]);
    }

    // Few rows.  Workgroup = 16 outputs of one expert of one token.  With a single row all workgroups
    // choose the token's experts for themselves from the logits, and the first records the choice for
    // the down projections; with more, a launch before has chosen.
    constexpr int EXPERT_WAVES = 8;
    template <typename T>
    __global__ void __launch_bounds__(EXPERT_WAVES * 64)
        expert_up_small_kernel(ExpertArgs p)
    {
        using O = Operand<T>;
        typedef T t4 __attribute__((ext_vector_type(4)));
        __shared__ __attribute__((aligned(16))) float s_red[EXPERT_WAVES][64][4];
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4;
        const int job = blockIdx.y, m = blockIdx.z; // jobs 0 .. top - 1: chosen experts; top: the shared one
        const bool shared = job == p.top;
        const int tile = blockIdx.x;
        const float *z = p.logits + (size_t)m * p.ldz;
        int id = 0;
        float weight = 0.0f;
        if (!shared)
        {
            if (tile * 16 >= p.ff)
                return;
            if (p.routed)
                id = p.ids[m * p.top + job];
            else
                route_wave(z, p.experts, p.top, lane, id, weight);
            if (!p.routed && tile == 0 && job == 0 && wave == 0)
            {
                if (lane < p.top)
                {
                    p.ids[m * p.top + lane] = id;
                    p.weights[m * (p.top + 1) + lane] = weight;
                }
                if (lane == 0 && p.shared_ff)
                    p.weights[m * (p.top + 1) + p.top] = sigmoidf(z[p.experts]);
            }
        }
        else if (tile * 16 >= p.shared_ff)
            return;
        const int expert = __shfl(id, shared ? 0 : job, 64);
        const int ksteps = p.K >> 5;
        const u32x4 *w = weight_tile(shared ? p.shared_up : p.up + (size_t)expert * p.up_stride, tile, ksteps, lane);
        const T *h = static_cast<const T *>(p.h) + (size_t)m * p.K + 8 * g;
        f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        constexpr int U = 8;
        for (int s0 = wave; s0 < ksteps; s0 += EXPERT_WAVES * U)
        {
            u32x4 raw[U];
#pragma unroll
            for (int u = 0; u < U; ++u)
            {
                const int s = s0 + u * EXPERT_WAVES;
                raw[u] = w[(size_t)(s < ksteps ? s : s0) * 64];
            }
#pragma unroll
            for (int u = 0; u < U; ++u)
            {
                const int s = s0 + u * EXPERT_WAVES;
                if (s < ksteps)
                    acc = O::mma(O::from_weights(raw[u]), O::load(h + s * 32), acc);
            }
        }
        *reinterpret_cast<f32x4 *>(s_red[wave][lane]) = acc;
        __syncthreads();
        if (threadIdx.x < 64 && (lane & 15) == 0)
        {
            f32x4 v = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int i = 0; i < EXPERT_WAVES; ++i)
                v = v + *reinterpret_cast<const f32x4 *>(s_red[i][lane]);
#pragma unroll
            for (int r = 0; r < 4; ++r)
            {
                const float y = fmaxf(v[r], 0.0f);
                v[r] = y * y;
            }
            T *act = static_cast<T *>(p.act) + (size_t)m * (p.top * p.ff + p.shared_ff) + (size_t)job * p.ff;
            *reinterpret_cast<t4 *>(act + tile * 16 + 4 * g) = __builtin_convertvector(v, t4);
        }
    }

    // Workgroup = 16 columns of one token's output over all its experts: the k-steps of all of them
    // in one list, dealt to the wavefronts.
    template <typename T>
    __global__ void __launch_bounds__(EXPERT_WAVES * 64)
        expert_down_small_kernel(ExpertArgs p)
    {
        using O = Operand<T>;
        using V = typename O::V;
        __shared__ __attribute__((aligned(16))) float s_red[EXPERT_WAVES][64][4];
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4;
        __shared__ int s_ids[64];
        __shared__ float s_weights[65];
        const int tile = blockIdx.x, m = blockIdx.y;
        const int esteps = p.ff >> 5, ssteps = p.shared_ff >> 5;
        const int total = p.top * esteps + ssteps;
        if (threadIdx.x <= p.top)
        {
            if (threadIdx.x < p.top)
                s_ids[threadIdx.x] = p.ids[m * p.top + threadIdx.x];
            s_weights[threadIdx.x] = p.weights[m * (p.top + 1) + threadIdx.x];
        }
        const T *act = static_cast<const T *>(p.act) + (size_t)m * (p.top * p.ff + p.shared_ff) + 8 * g;
        __syncthreads();
        f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        constexpr int U = 8;
        // the wavefront's place in the list: step s is step `in` of expert `job`
        int job = 0, in = wave;
        for (int s0 = wave; s0 < total; s0 += EXPERT_WAVES * U)
        {
            u32x4 raw[U];
            V b[U];
            float scale[U];
#pragma unroll
            for (int u = 0; u < U; ++u)
            {
                const int s = s0 + u * EXPERT_WAVES;
                while (job < p.top && in >= esteps)
                {
                    in -= esteps;
                    ++job;
                }
                const bool live = s < total;
                const int id = __builtin_amdgcn_readfirstlane(s_ids[job < p.top ? job : 0]);
                // (past the end: any step of the first expert, with weight zero)
                const u32x4 *w = job < p.top || !live ? weight_tile(p.down + (size_t)id * p.down_stride, tile, esteps, lane)
                                             : weight_tile(p.shared_down, tile, ssteps, lane);
                raw[u] = w[(size_t)(live ? in : 0) * 64];
                b[u] = O::load(act + (size_t)(live ? s : 0) * 32);
                scale[u] = live ? s_weights[job < p.top ? job : p.top] : 0.0f;
                in += EXPERT_WAVES;
            }
#pragma unroll
            for (int u = 0; u < U; ++u)
            {
                const f32x4 zero = {0.0f, 0.0f, 0.0f, 0.0f};
                acc = acc + O::mma(O::from_weights(raw[u]), b[u], zero) * scale[u];
            }
        }
        *reinterpret_cast<f32x4 *>(s_red[wave][lane]) = acc;
        __syncthreads();
        if (threadIdx.x < 64 && (lane & 15) == 0)
        {
            f32x4 *x = reinterpret_cast<f32x4 *>(p.x + (size_t)m * p.ldx + tile * 16 + 4 * g);
            f32x4 v = *x;
#pragma unroll
            for (int i = 0; i < EXPERT_WAVES; ++i)
                v = v + *reinterpret_cast<const f32x4 *>(s_red[i][lane]);
            *x = v;
        }
    }

    // Many rows: after the choice of experts
    // the (token, choice) pairs are put in order of their expert, each expert's in the order of
    // the tokens: one workgroup per expert counts the pairs of lower experts and places its own
    constexpr int GROUP_THREADS = 1024;
    __global__ void __launch_bounds__(GROUP_THREADS)
        expert_group_kernel(const int *__restrict__ ids, int pairs, int experts, int *__restrict__ offset,
                            int *__restrict__ order, int *__restrict__ place)
    {
        __shared__ int s_low[GROUP_THREADS / 64], s_own[GROUP_THREADS / 64];
        const int e = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
        int low = 0;
        for (int i = threadIdx.x; i < pairs; i += GROUP_THREADS)
            low += ids[i] < e;
#pragma unroll
        for (int off = 32; off > 0; off >>= 1)
            low += __shfl_xor(low, off, 64);
        if (lane == 0)
            s_low[wave] = low;
        __syncthreads();
        int base = 0;
        for (int w = 0; w < GROUP_THREADS / 64; ++w)
            base += s_low[w];
        if (threadIdx.x == 0)
        {
            offset[e] = base;
            if (e == experts - 1)
                offset[experts] = pairs;
        }
        for (int i0 = 0; i0 < pairs; i0 += GROUP_THREADS)
        {
            const int i = i0 + threadIdx.x;
            const bool own = i < pairs && ids[i] == e;
            const unsigned long long mask = __ballot(own);
            if (lane == 0)
                s_own[wave] = __popcll(mask);
            __syncthreads();
            int at = base;
            for (int w = 0; w < GROUP_THREADS / 64; ++w)
            {
                if (w < wave)
                    at += s_own[w];
                base += s_own[w];
            }
            if (own)
            {
                at += __popcll(mask & ((1ull << lane) - 1));
                order[at] = i;
                place[i] = at;
            }
            __syncthreads();
        }
    }

    // and the experts' outputs are summed in the order of the choice
    __global__ void __launch_bounds__(ROW_THREADS)
        expert_combine_kernel(ExpertArgs p, const float *__restrict__ pair_out, const float *__restrict__ shared_out,
                              const int *__restrict__ place)
    {
        const int m = blockIdx.x;
        const float *weights = p.weights + m * (p.top + 1);
        for (int i = threadIdx.x; i < p.N / 4; i += ROW_THREADS)
        {
            f32x4 *x = reinterpret_cast<f32x4 *>(p.x + (size_t)m * p.ldx) + i;
            f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
            for (int t = 0; t < p.top; ++t)
                y = y + reinterpret_cast<const f32x4 *>(pair_out + (size_t)place[m * p.top + t] * p.N)[i] * weights[t];
            if (p.shared_ff)
                y = y + reinterpret_cast<const f32x4 *>(shared_out + (size_t)m * p.N)[i] * weights[p.top];
            *x = *x + y;
        }
    }

    namespace
    {
        // scratch of the experts, from one buffer
        struct ExpertScratch
        {
            size_t ids, weights, act, offset, order, place, pair_out, shared_out, total;
        };
        ExpertScratch expert_scratch(int M, int experts, int top, int ff, int shared_ff, int N)
        {
            ExpertScratch s{};
            size_t at = 0;
            auto take = [&at](size_t bytes) {
                const size_t here = at;
                at += (bytes + 255) & ~(size_t)255;
                return here;
            };
            const size_t pairs = (size_t)M * top;
            s.ids = take(pairs * 4);
            s.weights = take((size_t)M * (top + 1) * 4);
            s.act = take((pairs * ff + (size_t)M * shared_ff) * 4);
            s.offset = take((size_t)(experts + 1) * 4);
            s.order = take(pairs * 4);
            s.place = take(pairs * 4);
            s.pair_out = take(pairs * N * 4);
            s.shared_out = take(shared_ff ? (size_t)M * N * 4 : 0);
            s.total = at;
            return s;
        }

        template <typename T>
        bool experts_run(const char *fn, ExpertArgs p, int M, char *scratch, int dtype, hipStream_t st)
        {
            const ExpertScratch at = expert_scratch(M, p.experts, p.top, p.ff, p.shared_ff, p.N);
            p.ids = reinterpret_cast<int *>(scratch + at.ids);
            p.weights = reinterpret_cast<float *>(scratch + at.weights);
            p.act = scratch + at.act;
            if (M > 1)
            {
                hipLaunchKernelGGL(expert_route_kernel, dim3(ceil_div(M, ROW_THREADS / 64)), dim3(ROW_THREADS), 0, st, p, M);
                if (!launched(fn))
                    return false;
                p.routed = true;
            }
            if (M <= SMALL_M)
            {
                const int widest = p.shared_ff > p.ff ? p.shared_ff : p.ff;
                hipLaunchKernelGGL(expert_up_small_kernel<T>, dim3(widest / 16, p.top + (p.shared_ff ? 1 : 0), M),
                                   dim3(EXPERT_WAVES * 64), 0, st, p);
                if (!launched(fn))
                    return false;
                hipLaunchKernelGGL(expert_down_small_kernel<T>, dim3(p.N / 16, M), dim3(EXPERT_WAVES * 64), 0, st, p);
                return launched(fn);
            }
            int *offset = reinterpret_cast<int *>(scratch + at.offset), *order = reinterpret_cast<int *>(scratch + at.order);
            int *place = reinterpret_cast<int *>(scratch + at.place);
            float *pair_out = reinterpret_cast<float *>(scratch + at.pair_out);
            float *shared_out = reinterpret_cast<float *>(scratch + at.shared_out);
            hipLaunchKernelGGL(expert_group_kernel, dim3(p.experts), dim3(GROUP_THREADS), 0, st, p.ids, M * p.top, p.experts,
                               offset, order, place);
            if (!launched(fn))
                return false;
            LinearArgs l{};
            l.source_div = 1;
            T *act = static_cast<T *>(p.act), *shared_act = act + (size_t)M * p.top * p.ff;
            // the gated tokens of each expert: every expert may get all M
            l.a = p.h, l.lda = p.K, l.w = p.up, l.w_stride = p.up_stride, l.y = act, l.ldy = p.ff;
            l.M = M, l.N = p.ff, l.K = p.K, l.out = LLAM_SEQ_OUT_RELU2;
            l.group_offset = offset, l.row_source = order, l.source_div = p.top;
            if (!linear_tiled(fn, l, p.experts, dtype, st))
                return false;
            l.a = act, l.lda = p.ff, l.w = p.down, l.w_stride = p.down_stride, l.y = pair_out, l.ldy = p.N;
            l.N = p.N, l.K = p.ff, l.out = LLAM_SEQ_OUT_F32, l.row_source = nullptr, l.source_div = 1;
            if (!linear_tiled(fn, l, p.experts, dtype, st))
                return false;
            if (p.shared_ff)
            {
                LinearArgs s{};
                s.source_div = 1;
                s.a = p.h, s.lda = p.K, s.w = p.shared_up, s.y = shared_act, s.ldy = p.shared_ff;
                s.M = M, s.N = p.shared_ff, s.K = p.K, s.out = LLAM_SEQ_OUT_RELU2;
                if (!linear_tiled(fn, s, 1, dtype, st))
                    return false;
                s.a = shared_act, s.lda = p.shared_ff, s.w = p.shared_down, s.y = shared_out, s.ldy = p.N;
                s.N = p.N, s.K = p.shared_ff, s.out = LLAM_SEQ_OUT_F32;
                if (!linear_tiled(fn, s, 1, dtype, st))
                    return false;
            }
            hipLaunchKernelGGL(expert_combine_kernel, dim3(M), dim3(ROW_THREADS), 0, st, p, pair_out, shared_out, place);
            return launched(fn);
        }
    } // namespace
} // namespace llamql

using namespace llamql;

extern "C" bool llam_seq_embed(const llam_seq_embed_args *a, const int32_t *d_ids, float *d_x, int M, int ldx, int device_id,
                               void *stream)
{
    static const char *fn = "llam_seq_embed";
    if (!a || !a->d_table || !d_ids || !d_x)
        return fail(fn, "null pointer");
    if (M < 0 || M > 65535 || a->vocab < 1 || a->width < 1 || ldx < a->width)
        return fail(fn, "bad size (M=%d vocab=%d width=%d ldx=%d)", M, a->vocab, a->width, ldx);
    if (a->d_pairs && (!a->d_row_slot || !a->d_row_pos || !a->d_history || a->buckets < 1 || a->cap < 1))
        return fail(fn, "pairs of tokens need rows, a history and buckets=%d cap=%d of at least 1", a->buckets, a->cap);
    if (!aligned16(a->d_table) || !aligned16(a->d_pairs) || !aligned16(d_x))
        return fail(fn, "misaligned rows");
    if (M == 0)
        return true;
    if (!set_device(fn, device_id))
        return false;
    hipLaunchKernelGGL(seq_embed_kernel, dim3(M >= EMBED_WIDE_ROWS ? 1 : ceil_div(ldx, 4 * ROW_THREADS), M), dim3(ROW_THREADS), 0, as_stream(stream), *a, d_ids, d_x, ldx);
    return launched(fn);
}

namespace
{
    bool rmsnorm(const char *fn, const float *d_x, int ldx, const int32_t *d_rows, const float *d_norm, const float *d_norm2, float eps,
                 int k_real, void *d_y, void *d_y2, int M, int K, int dtype, int device_id, void *stream)
    {
        if (M < 0 || K < 1 || k_real < 1 || k_real > K || ldx < K)
            return fail(fn, "bad size (M=%d K=%d k_real=%d ldx=%d)", M, K, k_real, ldx);
        if (M == 0)
            return true;
        if (!d_x || !d_norm || !d_y)
            return fail(fn, "null pointer");
        if ((K % 8) != 0 || (ldx % 4) != 0 || !aligned16(d_x) || !aligned16(d_norm) || !aligned16(d_y) || !aligned16(d_norm2) || !aligned16(d_y2))
            return fail(fn, "misaligned rows");
        if (!set_device(fn, device_id))
            return false;
        if (dtype == LLAM_SEQ_F32)
            hipLaunchKernelGGL(seq_rmsnorm_kernel<float>, dim3(M), dim3(ROW_THREADS), 0, as_stream(stream), d_x, ldx, d_rows,
                               d_norm, eps, k_real, static_cast<float *>(d_y), K, d_norm2, static_cast<float *>(d_y2));
        else
            hipLaunchKernelGGL(seq_rmsnorm_kernel<bf16>, dim3(M), dim3(ROW_THREADS), 0, as_stream(stream), d_x, ldx, d_rows,
                               d_norm, eps, k_real, static_cast<bf16 *>(d_y), K, d_norm2, static_cast<bf16 *>(d_y2));
        return launched(fn);
    }
} // namespace

extern "C" bool llam_seq_rmsnorm(const float *d_x, int ldx, const int32_t *d_rows, const float *d_norm, float eps,
                                 int k_real, void *d_y, int M, int K, int dtype, int device_id, void *stream)
{
    return rmsnorm("llam_seq_rmsnorm", d_x, ldx, d_rows, d_norm, nullptr, eps, k_real, d_y, nullptr, M, K, dtype, device_id, stream);
}

extern "C" bool llam_seq_rmsnorm_pair(const float *d_x, int ldx, const float *d_norm_a, const float *d_norm_b, float eps, int k_real,
                                      void *d_ya, void *d_yb, int M, int K, int dtype, int device_id, void *stream)
{
    static const char *fn = "llam_seq_rmsnorm_pair";
    if (!d_norm_b || !d_yb)
        return fail(fn, "null pointer");
    return rmsnorm(fn, d_x, ldx, nullptr, d_norm_a, d_norm_b, eps, k_real, d_ya, d_yb, M, K, dtype, device_id, stream);
}

extern "C" size_t llam_seq_experts_scratch_bytes(int max_rows, int experts, int top, int ff, int shared_ff, int N)
{
    if (max_rows < 1 || experts < 1 || top < 1 || ff < 1 || shared_ff < 0 || N < 1)
        return 0;
    return expert_scratch(max_rows, experts, top, ff, shared_ff, N).total;
}

extern "C" bool llam_seq_experts(const llam_seq_experts_args *a, int M, void *d_scratch, size_t scratch_bytes, int dtype,
                                 int device_id, void *stream)
{
    static const char *fn = "llam_seq_experts";
    if (!a || !a->d_logits || !a->d_up || !a->d_down || !a->d_h || !a->d_x || !d_scratch)
        return fail(fn, "null pointer");
    if (M < 0 || a->experts < 1 || a->top < 1 || a->top > a->experts || a->top > 64 || a->experts > 64 * ROUTE_MAX)
        return fail(fn, "bad size (M=%d experts=%d top=%d)", M, a->experts, a->top);
    if (M == 0)
        return true;
    if ((a->ff % PAD) != 0 || a->ff < PAD || (a->shared_ff % PAD) != 0 || (a->K % PAD) != 0 || (a->N % 16) != 0 || (a->ldx % 4) != 0 || a->ldx < a->N)
        return fail(fn, "ff=%d, shared_ff=%d and K=%d must be multiples of %d, N=%d of 16", a->ff, a->shared_ff, a->K, PAD, a->N);
    if (a->shared_ff && (!a->d_shared_up || !a->d_shared_down))
        return fail(fn, "null pointer (shared expert)");
    if (a->ldz < a->experts + (a->shared_ff ? 1 : 0))
        return fail(fn, "ldz=%d too small", a->ldz);
    if (llam_seq_experts_scratch_bytes(M, a->experts, a->top, a->ff, a->shared_ff, a->N) > scratch_bytes)
        return fail(fn, "scratch too small");
    if (M > 65535)
        return fail(fn, "M=%d rows", M);
    if (!set_device(fn, device_id))
        return false;
    ExpertArgs p{};
    p.logits = a->d_logits, p.ldz = a->ldz;
    p.up = static_cast<const bf16 *>(a->d_up), p.down = static_cast<const bf16 *>(a->d_down);
    p.shared_up = static_cast<const bf16 *>(a->d_shared_up), p.shared_down = static_cast<const bf16 *>(a->d_shared_down);
    p.up_stride = a->up_stride, p.down_stride = a->down_stride;
    p.experts = a->experts, p.top = a->top, p.ff = a->ff, p.shared_ff = a->shared_ff, p.K = a->K, p.N = a->N;
    p.h = a->d_h, p.x = a->d_x, p.ldx = a->ldx;
    return dtype == LLAM_SEQ_F32 ? experts_run<float>(fn, p, M, static_cast<char *>(d_scratch), dtype, as_stream(stream))
                                 : experts_run<bf16>(fn, p, M, static_cast<char *>(d_scratch), dtype, as_stream(stream));
}

extern "C" bool llam_seq_record(const int32_t *d_ids, int n, int32_t *d_out, int32_t *d_count, int max_count,
                                int device_id, void *stream)
{
    static const char *fn = "llam_seq_record";
    if (n < 1 || max_count < 0 || !d_ids || !d_out || !d_count)
        return fail(fn, "bad arguments");
    if (!set_device(fn, device_id))
        return false;
    hipLaunchKernelGGL(seq_record_kernel, dim3(1), dim3(64), 0, as_stream(stream), d_ids, n, d_out, d_count, max_count);
    return launched(fn);
}
