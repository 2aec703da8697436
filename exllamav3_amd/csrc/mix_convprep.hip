// What attention reads when its projected rows are filtered along the tokens first: every channel of q | k | v becomes the weighted sum of its last `taps` values,
// sum_i w[taps - 1 - i] x_(t - i) (nothing ahead of the first token), then per query / key head the RMS norm and the rotation of qk_prep (mix_diffattn.hip), and the rows that the sequence keeps go
// into its rings of keys and values.  One launch for prompt steps and for steps of one row per sequence: a row's predecessors are the step's own rows where the
// sequence has them in the step and the slot's ring of the last taps - 1 projected rows otherwise.  Sums, norms, angles are float32; the result is rounded once.
//
// One workgroup = R consecutive rows x one group of heads (about CP_CHANNELS channels of one of the three parts): the convolution's weights of a channel are
// loaded once for the R rows, the convolved rows of the group wait in LDS as float32 for the wave that norms and rotates a head.
#include "mix_common.cuh"

#define CP_THREADS 256
#define CP_WAVES 4
#define CP_CHANNELS 1024
#define CP_MAX_TAPS 16

// V neighbouring floats in pieces of four (16-byte aligned where V is a multiple of four)
template <int V> __device__ __forceinline__ void load_f(const float* p, float (&o)[V])
{
    if constexpr (V % 4 == 0)
    {
        #pragma unroll
        for (int a = 0; a < V; a += 4) { const float4 t = *(const float4*) (p + a); o[a] = t.x; o[a + 1] = t.y; o[a + 2] = t.z; o[a + 3] = t.w; }
    }
    else
    {
        #pragma unroll
        for (int e = 0; e < V; ++e) o[e] = p[e];
    }
}
template <int V> __device__ __forceinline__ void store_f(float* p, const float (&o)[V])
{
    if constexpr (V % 4 == 0)
    {
        #pragma unroll
        for (int a = 0; a < V; a += 4) *(float4*) (p + a) = make_float4(o[a], o[a + 1], o[a + 2], o[a + 3]);
    }
    else
    {
        #pragma unroll
        for (int e = 0; e < V; ++e) p[e] = o[e];
    }
}

// V: channels per thread and access; R: rows per workgroup; TAPS: number of taps, 0: read from `taps` (weights are then read per row)
template <typename T, int V, int R, int TAPS>
__global__ __launch_bounds__(CP_THREADS) void conv_prep_kernel(T* __restrict__ out, const T* __restrict__ x, int64_t x_ld, const float* __restrict__ conv_w, int taps_rt,
                                                               T* __restrict__ conv_ring, const float* __restrict__ q_norm, const float* __restrict__ k_norm,
                                                               const float* __restrict__ freq, int rot_dims, float mag, int interleaved, float eps, T* __restrict__ ring_k,
                                                               T* __restrict__ ring_v, const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ tok_pos,
                                                               const int32_t* __restrict__ slots, const int32_t* __restrict__ pos0, const int32_t* __restrict__ len_after,
                                                               int n, int q_heads, int kv_heads, int dim, int vdim, int rows, int keep_first, int q_per, int v_per, int q_groups, int k_groups)
{
    extern __shared__ __attribute__((aligned(16))) float smem[];                           // [R][channels of the group] | cos, sin [R][rot_dims / 2] each
    const int taps = TAPS ? TAPS : taps_rt, keep = taps - 1;
    const int n0 = blockIdx.x * R, lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
    const int nq = q_heads * dim, nk = kv_heads * dim, nv = kv_heads * vdim, C = nq + nk + nv;
    // this group: `cols` channels from column c0 of the projection
    int gr = blockIdx.y, part = 0;
    if (gr >= q_groups) { gr -= q_groups; part = 1; if (gr >= k_groups) { gr -= k_groups; part = 2; } }
    const int per = part == 2 ? v_per : q_per, hd = part == 2 ? vdim : dim, h0 = gr * per, hn = min(per, (part == 0 ? q_heads : kv_heads) - h0);
    const int cols = hn * hd, at0 = h0 * hd, c0 = at0 + (part == 0 ? 0 : (part == 1 ? nq : nq + nk));
    const int half = (freq && part < 2) ? rot_dims >> 1 : 0;
    float* cs = smem + R * q_per * dim;
    float* sn = cs + R * half;
    for (int t = threadIdx.x; t < R * half; t += CP_THREADS)
    {
        const int r = t / half, p = t - r * half;
        float sv = 0.f, cv = 0.f;
        if (n0 + r < n) sincosf((float) tok_pos[n0 + r] * freq[p], &sv, &cv);
        cs[t] = cv * mag; sn[t] = sv * mag;
    }
    for (int i = threadIdx.x * V; i < cols; i += CP_THREADS * V)
    {
        const int ch = c0 + i;
        float wt[TAPS ? TAPS : 1][V];
        if (TAPS)
        {
            #pragma unroll
            for (int j = 0; j < (TAPS ? TAPS : 1); ++j)
            {
                load_f<V>(conv_w + (int64_t) j * C + ch, wt[j]);
            }
        }
        #pragma unroll
        for (int r = 0; r < R; ++r)
        {
            const int row = n0 + r;
            if (row >= n) break;
            const int b = tok_seq[row], pos = tok_pos[row], start = pos0[b];
            const int64_t slot = slots[b];
            T* rg = conv_ring + slot * (keep > 0 ? keep : 1) * C + ch;
            float acc[V], own[V];
            load_n<T, V>(x + (int64_t) row * x_ld + ch, own);
            #pragma unroll
            for (int e = 0; e < V; ++e) acc[e] = 0.f;
            #pragma unroll
            for (int j = 0; j < (TAPS ? TAPS : CP_MAX_TAPS); ++j)
            {
                if (j >= keep) break;
                const int back = keep - j, p = pos - back;
                if (p < 0) continue;
                float u[V];
                load_n<T, V>(p >= start ? x + (int64_t) (row - back) * x_ld + ch : rg + (int64_t) (p % keep) * C, u);
                #pragma unroll
                for (int e = 0; e < V; ++e) acc[e] = __builtin_fmaf(TAPS ? wt[TAPS ? j : 0][e] : conv_w[(int64_t) j * C + ch + e], u[e], acc[e]);
            }
            #pragma unroll
            for (int e = 0; e < V; ++e) acc[e] = __builtin_fmaf(TAPS ? wt[TAPS ? TAPS - 1 : 0][e] : conv_w[(int64_t) keep * C + ch + e], own[e], acc[e]);
            if (keep > 0 && pos >= len_after[b] - keep) store_n<T, V>(rg + (int64_t) (pos % keep) * C, own);      // after this thread's own reads of the channel
            if (part < 2)
            {
                store_f<V>(smem + r * cols + i, acc);
                continue;
            }
            store_n<T, V>(out + (int64_t) row * C + ch, acc);
            if (ring_holds(pos, len_after[b], rows, keep_first)) store_n<T, V>(ring_v + (slot * rows + ring_entry(pos, rows, keep_first)) * nv + at0 + i, acc);
        }
    }
    if (part == 2) return;
    __syncthreads();
    const float* nw = part == 0 ? q_norm : k_norm;
    const int live = min(R, n - n0);
    for (int item = wv; item < live * hn; item += CP_WAVES)
    {
        const int r = item / hn;
        float* buf = smem + r * cols + (item - r * hn) * dim;
        if (nw)
        {
            float ss = 0.f;
            for (int i = lane; i < dim; i += 64) { const float y = buf[i]; ss += y * y; }
            ss = wave_sum(ss);
            const float inv = 1.0f / sqrtf(ss / (float) dim + eps);
            for (int i = lane; i < dim; i += 64) buf[i] = buf[i] * inv * nw[i];
            __builtin_amdgcn_wave_barrier();                  // LDS serves a wave's accesses in order: the stores above are visible to the reads below
        }
        for (int p = lane; p < half; p += 64)
        {
            const int i0 = interleaved ? 2 * p : p, i1 = interleaved ? 2 * p + 1 : p + half;
            const float u = buf[i0], w = buf[i1], cv = cs[r * half + p], sv = sn[r * half + p];
            buf[i0] = u * cv - w * sv;
            buf[i1] = w * cv + u * sv;
        }
    }
    __syncthreads();
    for (int i = threadIdx.x * V; i < cols; i += CP_THREADS * V)
    {
        for (int r = 0; r < live; ++r)
        {
            const int row = n0 + r;
            float y[V];
            load_f<V>(smem + r * cols + i, y);
            store_n<T, V>(out + (int64_t) row * C + c0 + i, y);
            if (part == 1)
            {
                const int b = tok_seq[row], pos = tok_pos[row];
                if (ring_holds(pos, len_after[b], rows, keep_first)) store_n<T, V>(ring_k + ((int64_t) slots[b] * rows + ring_entry(pos, rows, keep_first)) * nk + at0 + i, y);
            }
        }
    }
}

extern "C" int exl3_mix_conv_prep(void* out, const void* x, int64_t x_ld, const float* conv_w, int taps, void* conv_ring, const float* q_norm, const float* k_norm, const float* freq,
                                  int rot_dims, float mag, int interleaved, float eps, void* ring_k, void* ring_v, const int32_t* tok_seq, const int32_t* tok_pos, const int32_t* slots,
                                  const int32_t* pos0, const int32_t* len_after, int n, int q_heads, int kv_heads, int dim, int vdim, int rows, int keep_first, int dtype, void* stream)
{
    MIX_CHECK(out && x && conv_w && conv_ring && ring_k && ring_v && tok_seq && tok_pos && slots && pos0 && len_after, "mix_conv_prep: null pointer");
    MIX_CHECK(n >= 0 && q_heads > 0 && kv_heads > 0 && dim > 0 && dim <= 1024 && vdim > 0 && vdim <= 1024 && taps >= 1 && taps <= CP_MAX_TAPS,
              "mix_conv_prep: head sizes %d / %d (<= 1024) or %d taps (1..%d) out of range", dim, vdim, taps, CP_MAX_TAPS);
    const int64_t C = (int64_t) q_heads * dim + (int64_t) kv_heads * (dim + vdim);
    MIX_CHECK(x_ld >= C && out != x, "mix_conv_prep: bad row stride");
    MIX_CHECK(rows > 0 && keep_first >= 0 && keep_first < rows, "mix_conv_prep: a ring of %d entries cannot keep %d first positions", rows, keep_first);
    MIX_CHECK(!freq || (rot_dims >= 2 && rot_dims % 2 == 0 && rot_dims <= dim), "mix_conv_prep: %d rotated entries of %d", rot_dims, dim);
    if (n == 0) return EXL3_MIX_OK;
    const int vn = dtype == EXL3_MIX_BF16 ? 8 : 4;
    const bool vec = dim % vn == 0 && vdim % vn == 0 && x_ld % vn == 0 && (uintptr_t) x % 16 == 0 && (uintptr_t) out % 16 == 0 && (uintptr_t) conv_ring % 16 == 0 && (uintptr_t) ring_k % 16 == 0 &&
                     (uintptr_t) ring_v % 16 == 0 && (uintptr_t) conv_w % 16 == 0;
    const bool many = vec && n >= 512;
    const int q_per = CP_CHANNELS / dim, v_per = CP_CHANNELS / vdim;
    const int q_groups = (q_heads + q_per - 1) / q_per, k_groups = (kv_heads + q_per - 1) / q_per, v_groups = (kv_heads + v_per - 1) / v_per;
    MIX_CHECK(q_groups + k_groups + v_groups <= 65535, "mix_conv_prep: too many heads");
    const int R = many ? 4 : 1;
    const size_t sm = (size_t) R * (q_per * dim + (freq ? rot_dims : 0)) * sizeof(float);
    #define CP_LAUNCH(VV, RR, TT) hipLaunchKernelGGL((conv_prep_kernel<T, VV, RR, TT>), dim3((n + RR - 1) / RR, q_groups + k_groups + v_groups), dim3(CP_THREADS), sm, (hipStream_t) stream, \
                                                     (T*) out, (const T*) x, x_ld, conv_w, taps, (T*) conv_ring, q_norm, k_norm, freq, rot_dims, mag, interleaved, eps, (T*) ring_k, (T*) ring_v, \
                                                     tok_seq, tok_pos, slots, pos0, len_after, n, q_heads, kv_heads, dim, vdim, rows, keep_first, q_per, v_per, q_groups, k_groups)
    #define CP_TAPS(VV, RR) do { if (taps == 4) CP_LAUNCH(VV, RR, 4); else if (taps == 3) CP_LAUNCH(VV, RR, 3); else if (taps == 2) CP_LAUNCH(VV, RR, 2); else CP_LAUNCH(VV, RR, 0); } while (0)
    if (dtype == EXL3_MIX_BF16)
    {
        using T = bf16_t;
        if (many) CP_TAPS(8, 4); else if (vec) CP_TAPS(8, 1); else CP_LAUNCH(1, 1, 0);
    }
    else
    {
        using T = float;
        if (many) CP_TAPS(4, 4); else if (vec) CP_TAPS(4, 1); else CP_LAUNCH(1, 1, 0);
    }
    #undef CP_LAUNCH
    #undef CP_TAPS
    return mix_check_launch("mix_conv_prep");
}
