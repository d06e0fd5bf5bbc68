// Greedy sampling, for gfx950: the index of the largest logit of every row, in two passes.
#include "ql_device.h"
#include "ql_host.h"

#include <cfloat>
#include <climits>

#include "llaminar_amd/decode_api.h"

namespace llamql
{
    // ---- greedy sampling -----------------------------------------------------------------------
    constexpr int ARGMAX_THREADS = 256;
    constexpr int ARGMAX_PER_THREAD = 8;

    __device__ __forceinline__ bool argmax_better(float cv, int ci, float v, int i)
    {
        return cv > v || (cv == v && ci < i);
    }

    __device__ __forceinline__ void argmax_block_reduce(float &v, int &idx, float *s_v, int *s_i)
    {
#pragma unroll
        for (int off = WAVE / 2; off > 0; off >>= 1)
        {
            const float ov = __shfl_xor(v, off, WAVE);
            const int oi = __shfl_xor(idx, off, WAVE);
            if (argmax_better(ov, oi, v, idx))
            {
                v = ov;
                idx = oi;
            }
        }
        if ((threadIdx.x & (WAVE - 1)) == 0)
        {
            s_v[threadIdx.x >> 6] = v;
            s_i[threadIdx.x >> 6] = idx;
        }
        __syncthreads();
        if (threadIdx.x == 0)
        {
            for (int w = 1; w < ARGMAX_THREADS / WAVE; ++w)
                if (argmax_better(s_v[w], s_i[w], v, idx))
                {
                    v = s_v[w];
                    idx = s_i[w];
                }
        }
    }

    __global__ void __launch_bounds__(ARGMAX_THREADS)
        argmax_partial_kernel(const float *__restrict__ logits, int ld, int n, float *__restrict__ pv,
                              int *__restrict__ pi)
    {
        __shared__ float s_v[ARGMAX_THREADS / WAVE];
        __shared__ int s_i[ARGMAX_THREADS / WAVE];
        const int b = blockIdx.y;
        const float *row = logits + (size_t)b * ld;
        float v = -FLT_MAX;
        int idx = INT_MAX;
        const int stride = ARGMAX_THREADS * gridDim.x;
        for (int i = blockIdx.x * ARGMAX_THREADS + threadIdx.x; i < n; i += stride)
        {
            const float x = row[i];
            if (argmax_better(x, i, v, idx))
            {
                v = x;
                idx = i;
            }
        }
        argmax_block_reduce(v, idx, s_v, s_i);
        if (threadIdx.x == 0)
        {
            pv[(size_t)b * gridDim.x + blockIdx.x] = v;
            pi[(size_t)b * gridDim.x + blockIdx.x] = idx;
        }
    }

    __global__ void __launch_bounds__(ARGMAX_THREADS)
        argmax_final_kernel(const float *__restrict__ pv, const int *__restrict__ pi, int n_part,
                            int32_t *__restrict__ ids, int32_t *__restrict__ pos)
    {
        __shared__ float s_v[ARGMAX_THREADS / WAVE];
        __shared__ int s_i[ARGMAX_THREADS / WAVE];
        const int b = blockIdx.x;
        float v = -FLT_MAX;
        int idx = INT_MAX;
        for (int i = threadIdx.x; i < n_part; i += ARGMAX_THREADS)
        {
            const float x = pv[(size_t)b * n_part + i];
            const int xi = pi[(size_t)b * n_part + i];
            if (argmax_better(x, xi, v, idx))
            {
                v = x;
                idx = xi;
            }
        }
        argmax_block_reduce(v, idx, s_v, s_i);
        if (threadIdx.x == 0)
        {
            ids[b] = idx;
            if (pos)
                pos[b] += 1;
        }
    }

    inline int argmax_blocks(int n)
    {
        const int per_block = ARGMAX_THREADS * ARGMAX_PER_THREAD;
        return (n + per_block - 1) / per_block;
    }
} // namespace llamql

using namespace llamql;

extern "C" size_t llam_dec_argmax_scratch_bytes(int B, int n)
{
    if (B < 1 || n < 1)
        return 0;
    return (size_t)B * argmax_blocks(n) * (sizeof(float) + sizeof(int));
}

extern "C" bool llam_dec_argmax(const float *d_logits, int ld, int n, int B, int32_t *d_ids, int32_t *d_pos,
                                void *d_scratch, int device_id, void *stream)
{
    static const char *fn = "llam_dec_argmax";
    if (B < 0 || n < 1 || ld < n)
        return fail(fn, "bad size (B=%d n=%d ld=%d)", B, n, ld);
    if (B == 0)
        return true;
    if (!d_logits || !d_ids || !d_scratch)
        return fail(fn, "null pointer");
    if (!aligned4(d_logits) || !aligned4(d_ids) || !aligned4(d_scratch) || (d_pos && !aligned4(d_pos)))
        return fail(fn, "misaligned pointer");
    if (B > 65535)
        return fail(fn, "too many rows");
    if (!set_device(fn, device_id))
        return false;
    const int blocks = argmax_blocks(n);
    float *pv = static_cast<float *>(d_scratch);
    int *pi = reinterpret_cast<int *>(pv + (size_t)B * blocks);
    hipLaunchKernelGGL(argmax_partial_kernel, dim3(blocks, B), dim3(ARGMAX_THREADS), 0, as_stream(stream), d_logits,
                       ld, n, pv, pi);
    if (!launched(fn))
        return false;
    hipLaunchKernelGGL(argmax_final_kernel, dim3(B), dim3(ARGMAX_THREADS), 0, as_stream(stream), pv, pi, blocks,
                       d_ids, d_pos);
    return launched(fn);
}
