// Time mixing with a decay per key channel and token and a bonus for the current token (RWKV-style).  Per head, with decays w_t in (0, 1] given by their logarithms:
//   o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,   S_t = diag(w_t) S_(t-1) + k_t v_t^T
// Everything that enters the recurrence besides the projections is float32; the state [slot][head][dim][vdim] is float32.
//
//   token_shift    what the projections read: h + (h' - h) mu_m for every mix m, h' the previous token's row (of the step, or from the slot)
//   decay_log      log w = -exp(w0 + W2 tanh(t)) from the low-rank input t, on the float32 matrix instruction
//   timemix        prompt steps in tiles of 16 tokens, whole sequences or parallel segments; optionally with the head norm and gate that follow
//   timemix_step   one row per sequence: decays, read-out, state update, head norm and gate in one launch
//
// A tile of 16 tokens is four products on the float32 matrix instruction.  With L_t the sum of the tile's log decays up to and including token t, L'_t the sum
// before it and M = L_7 (the middle of the tile), q_t = r_t e^(L'_t - M) and p_t = k_t e^(M - L_t):
//   S' = diag(e^M) S;   O = Q S' + A V,  A[t][j] = q_t . p_j for j < t, A[t][t] = sum_c r_t u k_t;   S <- diag(e^(L_15 - M)) (S' + P^T V)
// Taking the exponents from the middle keeps both factors in range while every channel decays by less than e^-60 over each half of the tile; a tile with a
// stronger decay (uniform over the workgroup) runs token by token on the same registers instead, in which every exponent is a decay's own.
//
// v_mfma_f32_16x16x4_f32: operand lane (g = lane / 16, c = lane % 16) holds row / column c and contraction slot g; result lane (g, c) holds rows 4g .. 4g+3 of column
// c.  Contraction slot g of step i is index 4g + i of a block of 16, so four steps of an operand are one 16-byte LDS read and the registers of the state (rows
// 4g + i of a 16 x 16 block) are the B operand of Q S' as they stand.  One workgroup = one head, 64 value columns, 4 waves of 16 columns.
#include "mix_common.cuh"

typedef float f32x4 __attribute__((ext_vector_type(4)));

#define TM_THREADS 256
#define TM_WAVES 4
#define TM_TILE 16
#define TM_COLS 64
#define TM_WHOLE 0
#define TM_SEG_LOCAL 1
#define TM_SEG_FINAL 2
#define TM_MAX_EXP 60.0f

// out[m][n] = h[n] + (h'[n] - h[n]) mu[m]; h' = the row before n in its sequence: the step's own where the sequence has it in the step, the slot's otherwise, zeros
// ahead of the first token.  The last row of a sequence goes into its slot.  A thread holds V channels of R consecutive rows and of the row before them.
template <typename T, int V, int R>
__global__ __launch_bounds__(256) void token_shift_kernel(T* __restrict__ out, const T* __restrict__ h, int64_t h_ld, T* __restrict__ last, const float* __restrict__ mu, int mixes,
                                                          const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ slots,
                                                          const int32_t* __restrict__ pos0, const int32_t* __restrict__ len_after, int n, int width)
{
    const int n0 = blockIdx.x * R;
    const int i = (blockIdx.y * 256 + threadIdx.x) * V;
    if (i >= width) return;
    float cur[R][V], diff[R][V];
    float prev[V];
    #pragma unroll
    for (int e = 0; e < V; ++e) prev[e] = 0.f;
    {
        const int b = tok_seq[n0], pos = tok_pos[n0];
        if (pos > pos0[b]) load_n<T, V>(h + (int64_t) (n0 - 1) * h_ld + i, prev);
        else if (pos > 0)  load_n<T, V>(last + (int64_t) slots[b] * width + i, prev);
    }
    #pragma unroll
    for (int r = 0; r < R; ++r)
    {
        const int row = n0 + r;
        if (row >= n)
        {
            #pragma unroll
            for (int e = 0; e < V; ++e) { cur[r][e] = 0.f; diff[r][e] = 0.f; }
            continue;
        }
        const int b = tok_seq[row], pos = tok_pos[row];
        load_n<T, V>(h + (int64_t) row * h_ld + i, cur[r]);
        if (r > 0 && pos == pos0[b])                              // another sequence begins at this row
        {
            if (pos > 0) load_n<T, V>(last + (int64_t) slots[b] * width + i, prev);
            else
            {
                #pragma unroll
                for (int e = 0; e < V; ++e) prev[e] = 0.f;
            }
        }
        if (pos == len_after[b] - 1) store_n<T, V>(last + (int64_t) slots[b] * width + i, cur[r]);      // after this thread's own read of the slot
        #pragma unroll
        for (int e = 0; e < V; ++e) { diff[r][e] = prev[e] - cur[r][e]; prev[e] = cur[r][e]; }
    }
    for (int m = 0; m < mixes; ++m)
    {
        float w[V];
        #pragma unroll
        for (int e = 0; e < V; ++e) w[e] = mu[(int64_t) m * width + i + e];
        #pragma unroll
        for (int r = 0; r < R; ++r)
        {
            if (n0 + r >= n) break;
            float y[V];
            #pragma unroll
            for (int e = 0; e < V; ++e) y[e] = __builtin_fmaf(diff[r][e], w[e], cur[r][e]);
            store_n<T, V>(out + ((int64_t) m * n + n0 + r) * width + i, y);
        }
    }
}

// out[n][c] = -exp(w0[c] + sum_r tanh(t[n][r]) w2[c][r]): 32 rows x 256 channels per workgroup, a wave takes 64 of the channels; tanh and the products are float32
#define DL_ROWS 32
#define DL_COLS 256
#define DL_K 32
template <typename T>
__global__ __launch_bounds__(256) void decay_log_kernel(float* __restrict__ out, const T* __restrict__ t, int64_t t_ld, const T* __restrict__ w2, const float* __restrict__ w0, int n,
                                                        int channels, int rank)
{
    __shared__ __attribute__((aligned(16))) float ts[DL_ROWS * (DL_K + 4)];
    __shared__ __attribute__((aligned(16))) float wsm[DL_COLS * (DL_K + 4)];
    const int n0 = blockIdx.x * DL_ROWS, c0 = blockIdx.y * DL_COLS;
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
    f32x4 acc[2][4];
    #pragma unroll
    for (int a = 0; a < 2; ++a)
    {
        #pragma unroll
        for (int b = 0; b < 4; ++b) acc[a][b] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    for (int k0 = 0; k0 < rank; k0 += DL_K)
    {
        __syncthreads();
        for (int idx = threadIdx.x; idx < DL_ROWS * DL_K; idx += 256)
        {
            const int r = idx / DL_K, k = idx - r * DL_K;
            ts[r * (DL_K + 4) + k] = (n0 + r < n && k0 + k < rank) ? tanhf(to_f(t[(int64_t) (n0 + r) * t_ld + k0 + k])) : 0.f;
        }
        #pragma unroll 8
        for (int idx = threadIdx.x; idx < DL_COLS * DL_K; idx += 256)
        {
            const int r = idx / DL_K, k = idx - r * DL_K;
            wsm[r * (DL_K + 4) + k] = (c0 + r < channels && k0 + k < rank) ? to_f(w2[(int64_t) (c0 + r) * rank + k0 + k]) : 0.f;
        }
        __syncthreads();
        #pragma unroll
        for (int kt = 0; kt < DL_K / 16; ++kt)
        {
            f32x4 av[2], bv[4];
            #pragma unroll
            for (int a = 0; a < 2; ++a) av[a] = *(const f32x4*) (ts + (a * 16 + c) * (DL_K + 4) + kt * 16 + 4 * g);
            #pragma unroll
            for (int b = 0; b < 4; ++b) bv[b] = *(const f32x4*) (wsm + (w * 64 + b * 16 + c) * (DL_K + 4) + kt * 16 + 4 * g);
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                #pragma unroll
                for (int a = 0; a < 2; ++a)
                {
                    #pragma unroll
                    for (int b = 0; b < 4; ++b) acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[a][i], bv[b][i], acc[a][b], 0, 0, 0);
                }
            }
        }
    }
    #pragma unroll
    for (int b = 0; b < 4; ++b)
    {
        const int col = c0 + w * 64 + b * 16 + c;
        if (col >= channels) continue;
        const float z0 = w0[col];
        #pragma unroll
        for (int a = 0; a < 2; ++a)
        {
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const int row = n0 + a * 16 + 4 * g + i;
                if (row < n) out[(int64_t) row * channels + col] = -expf(acc[a][b][i] + z0);
            }
        }
    }
}

// DT: 16-row blocks of the (zero-padded) key dim.  Preparation: wave w owns the tile's tokens 4w .. 4w + 3, lane l the channels l, l + 64, ...
// out (optional, vdim <= 64): the heads after norm and gate, o / rms(o) * norm_w * silu(gate), instead of o.
template <typename T, int DT, int MODE>
__global__ __launch_bounds__(TM_THREADS) void timemix_chunk_kernel(float* __restrict__ o, T* __restrict__ out, int64_t out_ld, const T* __restrict__ gate, int64_t gate_ld,
                                                                   const float* __restrict__ norm_w, float eps, float* __restrict__ state,
                                                                   const T* __restrict__ r, int64_t r_ld, const T* __restrict__ k, int64_t k_ld, const T* __restrict__ v, int64_t v_ld,
                                                                   const float* __restrict__ logw, const float* __restrict__ u, const int32_t* __restrict__ cu,
                                                                   const int32_t* __restrict__ slots, const int32_t* __restrict__ pos0, int heads, int dim, int vdim,
                                                                   int segs, int seg_len, float* __restrict__ seg_state, float* __restrict__ seg_decay)
{
    constexpr int DP = DT * 16, LS = DP + 4, CI = (DP + 63) / 64, PS = TM_TILE + 4, TW = TM_TILE / TM_WAVES;
    constexpr bool READ = MODE != TM_SEG_LOCAL;
    __shared__ __attribute__((aligned(16))) float ks[TM_TILE * LS], ws[TM_TILE * LS];
    __shared__ __attribute__((aligned(16))) float rs[READ ? TM_TILE * LS : 4];
    __shared__ __attribute__((aligned(16))) float ps[READ ? TM_WAVES * TM_TILE * PS : 4];
    __shared__ __attribute__((aligned(16))) float em[DP], et[DP];
    __shared__ float tot[2][TM_WAVES][CI * 64], dg[2][TM_TILE], red[TM_WAVES][TM_TILE];
    const int b = (MODE == TM_WHOLE) ? blockIdx.x : blockIdx.x / segs, h = blockIdx.y;
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
    const int col = blockIdx.z * TM_COLS + w * 16 + c;
    const bool col_ok = col < vdim;
    int first = cu[b], last = cu[b + 1];
    float* st = state + ((int64_t) slots[b] * heads + h) * dim * vdim;
    bool resume = pos0[b] > 0;
    if (MODE != TM_WHOLE)
    {
        first += (blockIdx.x - b * segs) * seg_len;
        last = min(last, first + seg_len);
        if (first >= last) return;                                    // uniform: a shorter sequence has fewer segments
        st = seg_state + ((int64_t) blockIdx.x * heads + h) * dim * vdim;
        resume = (MODE == TM_SEG_FINAL);
    }
    f32x4 S[DT];
    #pragma unroll
    for (int kt = 0; kt < DT; ++kt)
    {
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int row = kt * 16 + 4 * g + i;
            S[kt][i] = (resume && col_ok && row < dim) ? st[(int64_t) row * vdim + col] : 0.f;
        }
    }
    float uc[CI], seg_sum[CI];
    #pragma unroll
    for (int ci = 0; ci < CI; ++ci)
    {
        uc[ci] = (READ && lane + 64 * ci < dim) ? u[h * dim + lane + 64 * ci] : 0.f;
        seg_sum[ci] = 0.f;
    }
    // the rows of the next tile wait in registers, as loaded, while the current one is computed
    T tr[CI][TW], tk[CI][TW], tv[4];
    float tw[CI][TW];
    const T zero = from_f<T>(0.f);
    auto fetch = [&](int n0) __attribute__((always_inline))
    {
        #pragma unroll
        for (int j = 0; j < TW; ++j)
        {
            const int t = n0 + w * TW + j;
            #pragma unroll
            for (int ci = 0; ci < CI; ++ci)
            {
                const int ch = lane + 64 * ci;
                const bool ok = t < last && ch < dim;
                const int64_t at = (int64_t) h * dim + ch;
                tk[ci][j] = ok ? k[(int64_t) t * k_ld + at] : zero;
                tr[ci][j] = (READ && ok) ? r[(int64_t) t * r_ld + at] : zero;
                tw[ci][j] = ok ? logw[(int64_t) t * heads * dim + at] : 0.f;
            }
        }
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int t = n0 + 4 * g + i;
            tv[i] = (t < last && col_ok) ? v[(int64_t) t * v_ld + (int64_t) h * vdim + col] : zero;
        }
    };
    fetch(first);
    int par = 0;
    for (int n0 = first; n0 < last; n0 += TM_TILE, par ^= 1)
    {
        const int tc = min(TM_TILE, last - n0);
        float kf[CI][TW], rf[CI][TW], lw[CI][TW], vr[4];
        float bonus[TW];
        #pragma unroll
        for (int j = 0; j < TW; ++j) bonus[j] = 0.f;
        #pragma unroll
        for (int ci = 0; ci < CI; ++ci)
        {
            float sum = 0.f;
            #pragma unroll
            for (int j = 0; j < TW; ++j)
            {
                kf[ci][j] = to_f(tk[ci][j]); rf[ci][j] = to_f(tr[ci][j]); lw[ci][j] = tw[ci][j];
                sum += lw[ci][j];
                bonus[j] += rf[ci][j] * uc[ci] * kf[ci][j];
            }
            tot[par][w][lane + 64 * ci] = sum;
        }
        #pragma unroll
        for (int i = 0; i < 4; ++i) vr[i] = to_f(tv[i]);
        if (READ)
        {
            #pragma unroll
            for (int j = 0; j < TW; ++j)
            {
                const float s = wave_sum(bonus[j]);
                if (lane == 0) dg[par][w * TW + j] = s;
            }
        }
        __syncthreads();                                              // tot and dg are there; the previous tile's reads of everything else are over
        if (n0 + TM_TILE < last) fetch(n0 + TM_TILE);
        bool strong = false;
        float half0[CI], half1[CI], base[CI];
        #pragma unroll
        for (int ci = 0; ci < CI; ++ci)
        {
            const int ch = lane + 64 * ci;
            const float a0 = tot[par][0][ch], a1 = tot[par][1][ch], a2 = tot[par][2][ch], a3 = tot[par][3][ch];
            half0[ci] = a0 + a1; half1[ci] = a2 + a3;
            base[ci] = w == 0 ? -half0[ci] : (w == 1 ? -a1 : (w == 2 ? 0.f : a2));      // the exponent ahead of this wave's first token, counted from the middle
            strong = strong || half0[ci] < -TM_MAX_EXP || half1[ci] < -TM_MAX_EXP;
            seg_sum[ci] += half0[ci] + half1[ci];
        }
        const bool slow = __any(strong);                              // every wave looks at every channel: the same answer in all of them
        #pragma unroll
        for (int ci = 0; ci < CI; ++ci)
        {
            const int ch = lane + 64 * ci;
            if (ch < DP)
            {
                float e = base[ci];
                #pragma unroll
                for (int j = 0; j < TW; ++j)
                {
                    const int at = (w * TW + j) * LS + ch;
                    if (slow)
                    {
                        if (READ) rs[at] = rf[ci][j];
                        ks[at] = kf[ci][j];
                        ws[at] = expf(lw[ci][j]);
                    }
                    else
                    {
                        if (READ) rs[at] = rf[ci][j] * expf(e);
                        e += lw[ci][j];
                        ks[at] = kf[ci][j] * expf(-e);
                    }
                }
                if (w == 0) em[ch] = expf(half0[ci]);
                if (w == 3) et[ch] = expf(half1[ci]);
            }
        }
        __syncthreads();
        f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
        if (slow)
        {
            #pragma unroll
            for (int t = 0; t < TM_TILE; ++t)
            {
                if (t >= tc) break;
                const float vv = __shfl(vr[t & 3], (t >> 2) * 16 + c, 64);
                float po = 0.f;
                #pragma unroll
                for (int kt = 0; kt < DT; ++kt)
                {
                    const int at = t * LS + kt * 16 + 4 * g;
                    const f32x4 kk = *(const f32x4*) (ks + at), dd = *(const f32x4*) (ws + at);
                    if (READ)
                    {
                        const f32x4 rr = *(const f32x4*) (rs + at);
                        #pragma unroll
                        for (int i = 0; i < 4; ++i) po = __builtin_fmaf(rr[i], S[kt][i], po);
                    }
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) S[kt][i] = __builtin_fmaf(dd[i], S[kt][i], kk[i] * vv);
                }
                if (READ)
                {
                    po += __shfl_xor(po, 16, 64);
                    po += __shfl_xor(po, 32, 64);
                    if (g == (t >> 2)) acc[t & 3] = __builtin_fmaf(dg[par][t], vv, po);
                }
            }
        }
        else
        {
            #pragma unroll
            for (int kt = 0; kt < DT; ++kt) S[kt] *= *(const f32x4*) (em + kt * 16 + 4 * g);
            if (READ)
            {
                // the scores' contraction is shared out over the waves; partial tiles meet in LDS
                f32x4 sc = f32x4{0.f, 0.f, 0.f, 0.f};
                #pragma unroll
                for (int kt = 0; kt < DT; ++kt)
                {
                    const f32x4 a = *(const f32x4*) (rs + c * LS + kt * 16 + 4 * g);
                    if ((kt & (TM_WAVES - 1)) == w)
                    {
                        const f32x4 bk = *(const f32x4*) (ks + c * LS + kt * 16 + 4 * g);
                        #pragma unroll
                        for (int i = 0; i < 4; ++i) sc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], bk[i], sc, 0, 0, 0);
                    }
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], S[kt][i], acc, 0, 0, 0);
                }
                #pragma unroll
                for (int i = 0; i < 4; ++i) ps[(w * TM_TILE + 4 * g + i) * PS + c] = 4 * g + i > c ? sc[i] : 0.f;
                __syncthreads();
                f32x4 a = *(const f32x4*) (ps + c * PS + 4 * g);
                #pragma unroll
                for (int ww = 1; ww < TM_WAVES; ++ww) a += *(const f32x4*) (ps + (ww * TM_TILE + c) * PS + 4 * g);
                const float own = dg[par][c];
                #pragma unroll
                for (int i = 0; i < 4; ++i)
                {
                    if (4 * g + i == c) a[i] = own;
                    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], vr[i], acc, 0, 0, 0);
                }
            }
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                #pragma unroll
                for (int kt = 0; kt < DT; ++kt) S[kt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(4 * g + i) * LS + kt * 16 + c], vr[i], S[kt], 0, 0, 0);
            }
            #pragma unroll
            for (int kt = 0; kt < DT; ++kt) S[kt] *= *(const f32x4*) (et + kt * 16 + 4 * g);
        }
        if (!READ) continue;
        if (out)
        {
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const float s = row16_sum(col_ok ? acc[i] * acc[i] : 0.f);
                if (c == 0) red[w][4 * g + i] = s;
            }
            __syncthreads();
        }
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int t = 4 * g + i;
            if (t >= tc || !col_ok) continue;
            if (out)
            {
                const float ss = (red[0][t] + red[1][t]) + (red[2][t] + red[3][t]);
                const float inv = 1.0f / sqrtf(ss / (float) vdim + eps);
                const int64_t at = (int64_t) h * vdim + col;
                out[(int64_t) (n0 + t) * out_ld + at] = from_f<T>(acc[i] * inv * norm_w[at] * silu_f(to_f(gate[(int64_t) (n0 + t) * gate_ld + at])));
            }
            else o[((int64_t) (n0 + t) * heads + h) * vdim + col] = acc[i];
        }
    }
    if (MODE == TM_SEG_FINAL) return;
    #pragma unroll
    for (int kt = 0; kt < DT; ++kt)
    {
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int row = kt * 16 + 4 * g + i;
            if (col_ok && row < dim) st[(int64_t) row * vdim + col] = S[kt][i];
        }
    }
    if (MODE == TM_SEG_LOCAL && blockIdx.z == 0 && w == 0)
    {
        #pragma unroll
        for (int ci = 0; ci < CI; ++ci)
        {
            const int ch = lane + 64 * ci;
            if (ch < dim) seg_decay[((int64_t) blockIdx.x * heads + h) * dim + ch] = expf(seg_sum[ci]);
        }
    }
}

// Between the two segment passes: every segment's own contribution in seg_state becomes the state it starts from; the state after the last one goes to the slot.
#define TM_AHEAD 8
__global__ __launch_bounds__(256) void timemix_combine_kernel(float* __restrict__ state, float* seg_state, const float* __restrict__ seg_decay, const int32_t* __restrict__ cu,
                                                              const int32_t* __restrict__ slots, const int32_t* __restrict__ pos0, int heads, int dim, int vdim, int segs, int seg_len)
{
    const int b = blockIdx.x, h = blockIdx.y;
    const int64_t per = (int64_t) dim * vdim;
    const int used = min(segs, (cu[b + 1] - cu[b] + seg_len - 1) / seg_len);
    float* st = state + ((int64_t) slots[b] * heads + h) * per;
    const int64_t e = (int64_t) blockIdx.z * 256 + threadIdx.x;
    if (e >= per) return;
    const int row = (int) (e / vdim);
    float S = pos0[b] > 0 ? st[e] : 0.f;
    for (int s0 = 0; s0 < used; s0 += TM_AHEAD)                       // several segments' loads in flight, then their sums in order
    {
        float local[TM_AHEAD], dec[TM_AHEAD];
        #pragma unroll
        for (int x = 0; x < TM_AHEAD; ++x)
        {
            const int64_t blk = ((int64_t) b * segs + s0 + x) * heads + h;
            const bool ok = s0 + x < used;
            local[x] = ok ? seg_state[blk * per + e] : 0.f;
            dec[x] = ok ? seg_decay[blk * dim + row] : 1.f;
        }
        #pragma unroll
        for (int x = 0; x < TM_AHEAD; ++x)
        {
            if (s0 + x >= used) break;
            seg_state[(((int64_t) b * segs + s0 + x) * heads + h) * per + e] = S;
            S = __builtin_fmaf(dec[x], S, local[x]);
        }
    }
    st[e] = S;
}

// Steps of one row per sequence, one workgroup per (sequence, head).  Eight lanes share a channel's low-rank product; then a thread owns V neighbouring value columns of
// every (threads / column groups)-th row of the state; partial read-outs meet in LDS.  out = o / rms(o) * norm_w * silu(gate).
#define TS_THREADS 512
template <typename T, int V>
__global__ __launch_bounds__(TS_THREADS) void timemix_step_kernel(T* __restrict__ out, int64_t out_ld, float* __restrict__ state, const T* __restrict__ r, int64_t r_ld,
                                                                  const T* __restrict__ k, int64_t k_ld, const T* __restrict__ v, int64_t v_ld, const T* __restrict__ gate, int64_t gate_ld,
                                                                  const T* __restrict__ t, int64_t t_ld, const T* __restrict__ w2, const float* __restrict__ w0,
                                                                  const float* __restrict__ u, const float* __restrict__ norm_w, const int32_t* __restrict__ tok_pos,
                                                                  const int32_t* __restrict__ slots, int heads, int dim, int vdim, int rank, float eps)
{
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ float red[TS_THREADS / 64];
    const int cg = (vdim + V - 1) / V;                                // column groups (vdim is a multiple of V)
    const int rp = TS_THREADS / cg;                                   // rows of the state in flight
    float* part = smem;                                               // [rp][vdim]
    float* rk = part + rp * vdim;                                     // [dim] r
    float* kk = rk + dim;                                             // [dim] k
    float* dc = kk + dim;                                             // [dim] decay
    float* ub = dc + dim;                                             // [dim] r u k
    float* th = ub + dim;                                             // [rank] tanh of the low-rank input
    const int n = blockIdx.x, h = blockIdx.y;
    for (int i = threadIdx.x; i < dim; i += TS_THREADS)
    {
        const int64_t at = (int64_t) h * dim + i;
        const float a = to_f(r[(int64_t) n * r_ld + at]), b = to_f(k[(int64_t) n * k_ld + at]);
        rk[i] = a; kk[i] = b; ub[i] = a * u[at] * b;
    }
    for (int i = threadIdx.x; i < rank; i += TS_THREADS) th[i] = tanhf(to_f(t[(int64_t) n * t_ld + i]));
    const int r0 = threadIdx.x / cg, c0 = (threadIdx.x - r0 * cg) * V;
    const bool live = r0 < rp, resume = tok_pos[n] > 0;
    float* st = state + ((int64_t) slots[n] * heads + h) * dim * vdim;
    __syncthreads();
    {
        const int sub = threadIdx.x & 7;
        for (int i0 = 0; i0 < dim; i0 += TS_THREADS / 8)              // uniform trip count: the shuffles see whole groups of eight
        {
            const int i = i0 + (threadIdx.x >> 3);
            float z = 0.f;
            if (i < dim)
            {
                const T* wr = w2 + ((int64_t) h * dim + i) * rank;
                for (int x = sub; x < rank; x += 8) z = __builtin_fmaf(th[x], to_f(wr[x]), z);
            }
            z += __shfl_xor(z, 1, 64); z += __shfl_xor(z, 2, 64); z += __shfl_xor(z, 4, 64);
            if (i < dim && sub == 0) dc[i] = expf(-expf(z + w0[(int64_t) h * dim + i]));
        }
    }
    __syncthreads();
    if (live)
    {
        const T* vp = v + (int64_t) n * v_ld + (int64_t) h * vdim + c0;
        float vv[V], acc[V];
        #pragma unroll
        for (int e = 0; e < V; ++e) { vv[e] = to_f(vp[e]); acc[e] = 0.f; }
        #pragma unroll 4
        for (int row = r0; row < dim; row += rp)
        {
            float* sp = st + (int64_t) row * vdim + c0;
            float s[V];
            if constexpr (V == 4) { const float4 q = resume ? *(const float4*) sp : make_float4(0.f, 0.f, 0.f, 0.f); s[0] = q.x; s[1] = q.y; s[2] = q.z; s[V - 1] = q.w; }
            else s[0] = resume ? sp[0] : 0.f;
            const float kx = kk[row], rx = rk[row], dx = dc[row], ux = ub[row];
            #pragma unroll
            for (int e = 0; e < V; ++e)
            {
                acc[e] = __builtin_fmaf(rx, s[e], __builtin_fmaf(ux, vv[e], acc[e]));
                s[e] = __builtin_fmaf(dx, s[e], kx * vv[e]);
            }
            if constexpr (V == 4) *(float4*) sp = make_float4(s[0], s[1], s[2], s[V - 1]); else sp[0] = s[0];
        }
        #pragma unroll
        for (int e = 0; e < V; ++e) part[r0 * vdim + c0 + e] = acc[e];
    }
    __syncthreads();
    float ss = 0.f;
    for (int c = threadIdx.x; c < vdim; c += TS_THREADS)
    {
        float s = 0.f;
        for (int x = 0; x < rp; ++x) s += part[x * vdim + c];
        part[c] = s;                                                  // the column's own first row: read by this thread only
        ss += s * s;
    }
    ss = block_sum<TS_THREADS / 64>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float) vdim + eps);
    for (int c = threadIdx.x; c < vdim; c += TS_THREADS)
    {
        const int64_t at = (int64_t) h * vdim + c;
        out[(int64_t) n * out_ld + at] = from_f<T>(part[c] * inv * norm_w[at] * silu_f(to_f(gate[(int64_t) n * gate_ld + at])));
    }
}

extern "C" int exl3_mix_token_shift(void* out, const void* h, int64_t h_ld, void* last, const float* mu, int mixes, const int32_t* tok_seq, const int32_t* tok_pos, const int32_t* slots,
                                    const int32_t* pos0, const int32_t* len_after, int n, int width, int dtype, void* stream)
{
    MIX_CHECK(out && h && last && mu && tok_seq && tok_pos && slots && pos0 && len_after, "mix_token_shift: null pointer");
    MIX_CHECK(n >= 0 && width > 0 && mixes >= 1 && h_ld >= width && out != h, "mix_token_shift: bad sizes");
    if (n == 0) return EXL3_MIX_OK;
    const int vn = dtype == EXL3_MIX_BF16 ? 8 : 4;
    const bool vec = width % vn == 0 && h_ld % vn == 0 && (uintptr_t) out % 16 == 0 && (uintptr_t) h % 16 == 0 && (uintptr_t) last % 16 == 0;
    #define SH_LAUNCH(VV, RR) hipLaunchKernelGGL((token_shift_kernel<T, VV, RR>), dim3((n + RR - 1) / RR, (width + 256 * VV - 1) / (256 * VV)), dim3(256), 0, (hipStream_t) stream, \
                                                 (T*) out, (const T*) h, h_ld, (T*) last, mu, mixes, tok_seq, tok_pos, slots, pos0, len_after, n, width)
    MIX_CHECK((width + 255) / 256 <= 65535, "mix_token_shift: width %d", width);
    if (dtype == EXL3_MIX_BF16)
    {
        using T = bf16_t;
        if (vec) { if (n >= 1024) SH_LAUNCH(8, 4); else SH_LAUNCH(8, 1); } else SH_LAUNCH(1, 1);
    }
    else
    {
        using T = float;
        if (vec) { if (n >= 1024) SH_LAUNCH(4, 4); else SH_LAUNCH(4, 1); } else SH_LAUNCH(1, 1);
    }
    #undef SH_LAUNCH
    return mix_check_launch("mix_token_shift");
}

extern "C" int exl3_mix_decay_log(float* out, const void* t, int64_t t_ld, const void* w2, const float* w0, int n, int channels, int rank, int dtype, void* stream)
{
    MIX_CHECK(out && t && w2 && w0 && n >= 0 && channels > 0 && rank > 0 && t_ld >= rank && (channels + DL_COLS - 1) / DL_COLS <= 65535, "mix_decay_log: bad arguments");
    if (n == 0) return EXL3_MIX_OK;
    MIX_DISPATCH_T(dtype, hipLaunchKernelGGL(decay_log_kernel<T>, dim3((n + DL_ROWS - 1) / DL_ROWS, (channels + DL_COLS - 1) / DL_COLS), dim3(256), 0, (hipStream_t) stream, out, (const T*) t,
                                             t_ld, (const T*) w2, w0, n, channels, rank));
    return mix_check_launch("mix_decay_log");
}

static int timemix_check(const char* what, int heads, int dim, int vdim)
{
    MIX_CHECK(heads > 0 && heads <= 65535 && dim > 0 && dim <= 256 && vdim > 0 && vdim <= 1024, "%s: dim %d (<= 256) / vdim %d (<= 1024) out of range", what, dim, vdim);
    return EXL3_MIX_OK;
}

template <int MODEV>
static int timemix_launch(float* o, void* out, int64_t out_ld, const void* gate, int64_t gate_ld, const float* norm_w, float eps, float* state, const void* r, int64_t r_ld, const void* k,
                          int64_t k_ld, const void* v, int64_t v_ld, const float* logw, const float* u, const int32_t* cu, const int32_t* slots, const int32_t* pos0, int batch, int heads,
                          int dim, int vdim, int segs, int seg_len, float* seg_state, float* seg_decay, int dtype, void* stream)
{
    const dim3 grid(batch * segs, heads, (vdim + TM_COLS - 1) / TM_COLS);
    #define TM_LAUNCH(DTV) hipLaunchKernelGGL((timemix_chunk_kernel<T, DTV, MODEV>), grid, dim3(TM_THREADS), 0, (hipStream_t) stream, o, (T*) out, out_ld, (const T*) gate, gate_ld, norm_w, \
                                              eps, state, (const T*) r, r_ld, (const T*) k, k_ld, (const T*) v, v_ld, logw, u, cu, slots, pos0, heads, dim, vdim, segs, seg_len, seg_state, \
                                              seg_decay)
    MIX_DISPATCH_T(dtype, if (dim <= 32) TM_LAUNCH(2); else if (dim <= 48) TM_LAUNCH(3); else if (dim <= 64) TM_LAUNCH(4); else if (dim <= 128) TM_LAUNCH(8); else TM_LAUNCH(16));
    #undef TM_LAUNCH
    return mix_check_launch("mix_timemix");
}

extern "C" int exl3_mix_timemix(float* o, void* out, int64_t out_ld, const void* gate, int64_t gate_ld, const float* norm_w, float eps, float* state, const void* r, int64_t r_ld,
                                const void* k, int64_t k_ld, const void* v, int64_t v_ld, const float* logw, const float* u, const int32_t* cu, const int32_t* slots,
                                const int32_t* pos0, int batch, int heads, int dim, int vdim, int segs, int seg_len, float* seg_state, float* seg_decay, int dtype, void* stream)
{
    MIX_CHECK((o || out) && state && r && k && v && logw && u && cu && slots && pos0 && batch >= 0, "mix_timemix: null pointer");
    if (int rc = timemix_check("mix_timemix", heads, dim, vdim)) return rc;
    MIX_CHECK(r_ld >= (int64_t) heads * dim && k_ld >= (int64_t) heads * dim && v_ld >= (int64_t) heads * vdim, "mix_timemix: bad row strides");
    MIX_CHECK(!out || (gate && norm_w && vdim <= TM_COLS && out_ld >= (int64_t) heads * vdim && gate_ld >= (int64_t) heads * vdim),
              "mix_timemix: norm and gate in the same launch need vdim <= %d, the gate and the weight", TM_COLS);
    MIX_CHECK(segs >= 1 && (segs == 1 || (seg_len >= 1 && seg_state && seg_decay)), "mix_timemix: bad segment arguments");
    if (batch == 0) return EXL3_MIX_OK;
    #define TM_ARGS o, out, out_ld, gate, gate_ld, norm_w, eps, state, r, r_ld, k, k_ld, v, v_ld, logw, u, cu, slots, pos0, batch, heads, dim, vdim, segs, seg_len, seg_state, seg_decay, dtype, stream
    if (segs == 1) return timemix_launch<TM_WHOLE>(TM_ARGS);
    int rc = timemix_launch<TM_SEG_LOCAL>(TM_ARGS);
    if (rc) return rc;
    const int64_t per = (int64_t) dim * vdim;
    hipLaunchKernelGGL(timemix_combine_kernel, dim3(batch, heads, (unsigned) ((per + 255) / 256)), dim3(256), 0, (hipStream_t) stream, state, seg_state, seg_decay, cu, slots, pos0, heads, dim,
                       vdim, segs, seg_len);
    if ((rc = mix_check_launch("mix_timemix (combine)"))) return rc;
    return timemix_launch<TM_SEG_FINAL>(TM_ARGS);
    #undef TM_ARGS
}

extern "C" int exl3_mix_timemix_step(void* out, int64_t out_ld, float* state, const void* r, int64_t r_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld, const void* gate,
                                     int64_t gate_ld, const void* t, int64_t t_ld, const void* w2, const float* w0, const float* u, const float* norm_w, const int32_t* tok_pos,
                                     const int32_t* slots, int n, int heads, int dim, int vdim, int rank, float eps, int dtype, void* stream)
{
    MIX_CHECK(out && state && r && k && v && gate && t && w2 && w0 && u && norm_w && tok_pos && slots && n >= 0, "mix_timemix_step: null pointer");
    if (int rc = timemix_check("mix_timemix_step", heads, dim, vdim)) return rc;
    MIX_CHECK(r_ld >= (int64_t) heads * dim && k_ld >= (int64_t) heads * dim && v_ld >= (int64_t) heads * vdim && gate_ld >= (int64_t) heads * vdim && out_ld >= (int64_t) heads * vdim &&
              rank > 0 && rank <= 4096 && t_ld >= rank, "mix_timemix_step: bad row strides or rank %d (<= 4096)", rank);
    if (n == 0) return EXL3_MIX_OK;
    const bool by4 = vdim % 4 == 0 && (uintptr_t) state % 16 == 0;
    MIX_CHECK(by4 || vdim <= TS_THREADS, "mix_timemix_step: vdim %d must be a multiple of 4 or at most %d", vdim, TS_THREADS);
    const int cg = by4 ? vdim / 4 : vdim;
    const size_t sm = ((size_t) (TS_THREADS / cg) * vdim + 4 * dim + rank) * sizeof(float);
    #define TS_LAUNCH(VV) hipLaunchKernelGGL((timemix_step_kernel<T, VV>), dim3(n, heads), dim3(TS_THREADS), sm, (hipStream_t) stream, (T*) out, out_ld, state, (const T*) r, r_ld, (const T*) k, \
                                             k_ld, (const T*) v, v_ld, (const T*) gate, gate_ld, (const T*) t, t_ld, (const T*) w2, w0, u, norm_w, tok_pos, slots, heads, dim, vdim, rank, eps)
    MIX_DISPATCH_T(dtype, if (by4) TS_LAUNCH(4); else TS_LAUNCH(1));
    #undef TS_LAUNCH
    return mix_check_launch("mix_timemix_step");
}
