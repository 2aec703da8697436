// Retention: linear attention with one fixed decay per head, no softmax and no denominator.  Per head S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, with q and k
// rotated by their position and k scaled.  Everything between the projections and the output norm is float32: the rotated vectors never leave LDS, the products
// run on the float32 matrix instruction, the state [slot][head][dim][vdim] is float32.
//
// Prompt steps walk a sequence in tiles of TT tokens.  With a fixed decay a tile is three products and no recurrence inside it:
//   O = diag(decay^(t+1)) (Q S) + (Q K^T . D) V,   D[t][j] = decay^(t-j) for j <= t, else 0
//   S <- decay^T S + (diag(decay^(T-1-t)) K)^T V
// Long prompts are cut into segments of whole tiles that run in parallel: a pass that leaves every segment's own contribution to the state, a walk over the
// segments that turns those into the state each one starts from, and the pass that computes outputs.
//
// v_mfma_f32_16x16x4_f32: operand lane (g = lane / 16, c = lane % 16) holds row / column c and contraction slot g; result lane (g, c) holds rows 4g .. 4g+3 of column
// c.  Reading contraction slot g of step i as index 4g + i of a block of 16 makes four steps of an operand one 16-byte LDS read, and makes the registers of
// the state (rows 4g + i of a 16 x 16 block) the B operand of Q S as they stand: the state of a wave's 16 value columns stays in registers.
// One workgroup = one head, 64 value columns, 4 waves of 16 columns; the score tiles of Q K^T are shared out over the waves and go through LDS.
#include "mix_common.cuh"

typedef float f32x4 __attribute__((ext_vector_type(4)));

#define RT_WAVES 4
#define RT_THREADS 256
#define RT_COLS 64
#define RT_WHOLE 0
#define RT_SEG_LOCAL 1
#define RT_SEG_FINAL 2

__device__ __forceinline__ void rt_pair(int i, int half, int interleaved, int& a, int& b) { a = interleaved ? 2 * i : i; b = interleaved ? 2 * i + 1 : i + half; }

// DT: 16-row blocks of the (zero-padded) key dim.  pw [heads][pw_ld]: decay^0, decay^1, ... (at least TT + 1 of them).
template <typename T, int DT, int TT, int MODE>
__global__ __launch_bounds__(RT_THREADS) void retention_chunk_kernel(float* __restrict__ o, float* __restrict__ state, const T* __restrict__ q, int64_t q_ld, const T* __restrict__ k,
                                                                     int64_t k_ld, const T* __restrict__ v, int64_t v_ld, const float* __restrict__ pw, int pw_ld,
                                                                     const float* __restrict__ freq, int rot_dims, int interleaved,
                                                                     const int32_t* __restrict__ cu, const int32_t* __restrict__ slots, const int32_t* __restrict__ pos0,
                                                                     int heads, int dim, int vdim, float k_scale, int segs, int seg_len, float* __restrict__ seg_state)
{
    constexpr int DP = DT * 16, LS = DP + 4, PS = TT + 4, TB = TT / 16;
    __shared__ __attribute__((aligned(16))) float ks[TT * LS];
    __shared__ __attribute__((aligned(16))) float qs[MODE == RT_SEG_LOCAL ? 4 : TT * LS];
    __shared__ __attribute__((aligned(16))) float ps[MODE == RT_SEG_LOCAL ? 4 : TT * PS];
    __shared__ float dw[TT + 1];                                      // decay^0 .. decay^TT
    const int b = (MODE == RT_WHOLE) ? blockIdx.x : blockIdx.x / segs, h = blockIdx.y;
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
    const int col = blockIdx.z * RT_COLS + w * 16 + c;
    const bool col_ok = col < vdim;
    const int seq_first = cu[b];
    int first = seq_first, last = cu[b + 1];
    float* st = state + ((int64_t) slots[b] * heads + h) * dim * vdim;
    bool resume = pos0[b] > 0;
    const int p_first = pos0[b];
    if (MODE != RT_WHOLE)
    {
        first += (blockIdx.x - b * segs) * seg_len;
        last = min(last, first + seg_len);
        if (first >= last) return;                                    // uniform: a shorter sequence has fewer segments
        st = seg_state + ((int64_t) blockIdx.x * heads + h) * dim * vdim;
        resume = (MODE == RT_SEG_FINAL);
    }
    for (int i = threadIdx.x; i <= TT; i += RT_THREADS) dw[i] = pw[(int64_t) h * pw_ld + i];
    f32x4 S[DT];
    #pragma unroll
    for (int kt = 0; kt < DT; ++kt)
    {
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int r = kt * 16 + 4 * g + i;
            S[kt][i] = (resume && col_ok && r < dim) ? st[(int64_t) r * vdim + col] : 0.f;
        }
    }
    const int half = rot_dims >> 1, rest = DP - rot_dims;
    for (int n0 = first; n0 < last; n0 += TT)
    {
        const int tc = min(TT, last - n0);
        __syncthreads();                                              // the previous tile's LDS reads are over (and dw is there)
        for (int idx = threadIdx.x; idx < TT * half; idx += RT_THREADS)
        {
            const int t = idx / half, i = idx - t * half;
            int a, bb;
            rt_pair(i, half, interleaved, a, bb);
            float q0 = 0.f, q1 = 0.f, k0 = 0.f, k1 = 0.f;
            if (t < tc)
            {
                float sn, cs;
                sincosf((float) (p_first + (n0 - seq_first) + t) * freq[i], &sn, &cs);
                const T* kr = k + (int64_t) (n0 + t) * k_ld + (int64_t) h * dim;
                const float ku = to_f(kr[a]), kv = to_f(kr[bb]);
                k0 = (ku * cs - kv * sn) * k_scale; k1 = (kv * cs + ku * sn) * k_scale;
                if (MODE != RT_SEG_LOCAL)
                {
                    const T* qr = q + (int64_t) (n0 + t) * q_ld + (int64_t) h * dim;
                    const float qu = to_f(qr[a]), qv = to_f(qr[bb]);
                    q0 = qu * cs - qv * sn; q1 = qv * cs + qu * sn;
                }
            }
            ks[t * LS + a] = k0; ks[t * LS + bb] = k1;
            if (MODE != RT_SEG_LOCAL) { qs[t * LS + a] = q0; qs[t * LS + bb] = q1; }
        }
        if (rest > 0)
        {
            for (int idx = threadIdx.x; idx < TT * rest; idx += RT_THREADS)
            {
                const int t = idx / rest, i = rot_dims + (idx - t * rest);
                const bool ok = t < tc && i < dim;
                ks[t * LS + i] = ok ? to_f(k[(int64_t) (n0 + t) * k_ld + (int64_t) h * dim + i]) * k_scale : 0.f;
                if (MODE != RT_SEG_LOCAL) qs[t * LS + i] = ok ? to_f(q[(int64_t) (n0 + t) * q_ld + (int64_t) h * dim + i]) : 0.f;
            }
        }
        float vr[TB * 4];                                             // v of tokens 16 tb + 4g + i, this lane's column
        #pragma unroll
        for (int e = 0; e < TB * 4; ++e)
        {
            const int t = (e >> 2) * 16 + 4 * g + (e & 3);
            vr[e] = (t < tc && col_ok) ? to_f(v[(int64_t) (n0 + t) * v_ld + (int64_t) h * vdim + col]) : 0.f;
        }
        __syncthreads();
        if (MODE != RT_SEG_LOCAL)
        {
            // score tiles (rt, ct), ct <= rt, shared out over the waves
            #pragma unroll
            for (int rt = 0; rt < TB; ++rt)
            {
                #pragma unroll
                for (int ct = 0; ct <= rt; ++ct)
                {
                    if (((rt * (rt + 1) / 2 + ct) & (RT_WAVES - 1)) != w) continue;
                    f32x4 sc = f32x4{0.f, 0.f, 0.f, 0.f};
                    #pragma unroll
                    for (int kt = 0; kt < DT; ++kt)
                    {
                        const f32x4 a = *(const f32x4*) (qs + (rt * 16 + c) * LS + kt * 16 + 4 * g);
                        const f32x4 bq = *(const f32x4*) (ks + (ct * 16 + c) * LS + kt * 16 + 4 * g);
                        #pragma unroll
                        for (int i = 0; i < 4; ++i) sc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], bq[i], sc, 0, 0, 0);
                    }
                    #pragma unroll
                    for (int i = 0; i < 4; ++i)
                    {
                        const int row = rt * 16 + 4 * g + i, key = ct * 16 + c;
                        ps[row * PS + key] = row >= key ? sc[i] * dw[row >= key ? row - key : 0] : 0.f;
                    }
                }
            }
            // what the tile reads from the state before it
            f32x4 acc[TB];
            #pragma unroll
            for (int rt = 0; rt < TB; ++rt)
            {
                acc[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
                #pragma unroll
                for (int kt = 0; kt < DT; ++kt)
                {
                    const f32x4 a = *(const f32x4*) (qs + (rt * 16 + c) * LS + kt * 16 + 4 * g);
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) acc[rt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], S[kt][i], acc[rt], 0, 0, 0);
                }
                #pragma unroll
                for (int i = 0; i < 4; ++i) acc[rt][i] *= dw[rt * 16 + 4 * g + i + 1];
            }
            __syncthreads();                                          // the scores are in LDS
            #pragma unroll
            for (int rt = 0; rt < TB; ++rt)
            {
                #pragma unroll
                for (int tb = 0; tb <= rt; ++tb)
                {
                    const f32x4 a = *(const f32x4*) (ps + (rt * 16 + c) * PS + tb * 16 + 4 * g);
                    #pragma unroll
                    for (int i = 0; i < 4; ++i) acc[rt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], vr[tb * 4 + i], acc[rt], 0, 0, 0);
                }
                #pragma unroll
                for (int i = 0; i < 4; ++i)
                {
                    const int t = rt * 16 + 4 * g + i;
                    if (t < tc && col_ok) o[((int64_t) (n0 + t) * heads + h) * vdim + col] = acc[rt][i];
                }
            }
        }
        // the state after the tile
        const float full = dw[tc];
        #pragma unroll
        for (int kt = 0; kt < DT; ++kt) S[kt] *= full;
        #pragma unroll
        for (int tb = 0; tb < TB; ++tb)
        {
            #pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const int t = tb * 16 + 4 * g + i;
                const float vw = vr[tb * 4 + i] * dw[max(tc - 1 - t, 0)];      // t >= tc: v is zero there
                #pragma unroll
                for (int kt = 0; kt < DT; ++kt) S[kt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[t * LS + kt * 16 + c], vw, S[kt], 0, 0, 0);
            }
        }
    }
    if (MODE == RT_SEG_FINAL) return;
    #pragma unroll
    for (int kt = 0; kt < DT; ++kt)
    {
        #pragma unroll
        for (int i = 0; i < 4; ++i)
        {
            const int r = kt * 16 + 4 * g + i;
            if (col_ok && r < dim) st[(int64_t) r * vdim + col] = S[kt][i];
        }
    }
}

// Between the two segment passes: every segment's own contribution in seg_state becomes the state it starts from; the state after the last one goes to the slot.
#define RT_AHEAD 8
__global__ __launch_bounds__(256) void retention_combine_kernel(float* __restrict__ state, float* seg_state, const float* __restrict__ pw, int pw_ld, const int32_t* __restrict__ cu,
                                                                const int32_t* __restrict__ slots, const int32_t* __restrict__ pos0, int heads, int dim, int vdim, int segs,
                                                                int seg_len)
{
    const int b = blockIdx.x, h = blockIdx.y;
    const int64_t per = (int64_t) dim * vdim;
    const int rows = cu[b + 1] - cu[b];
    const int used = min(segs, (rows + seg_len - 1) / seg_len);
    float* st = state + ((int64_t) slots[b] * heads + h) * per;
    const bool resume = pos0[b] > 0;
    const double lam = (double) pw[(int64_t) h * pw_ld + 1];
    const float dfull = (float) pow(lam, (double) seg_len), dlast = (float) pow(lam, (double) (rows - (used - 1) * seg_len));
    const int64_t e = (int64_t) blockIdx.z * 256 + threadIdx.x;
    if (e >= per) return;
    float S = resume ? st[e] : 0.f;
    for (int s0 = 0; s0 < used; s0 += RT_AHEAD)                       // several segments' loads in flight, then their sums in order
    {
        float local[RT_AHEAD];
        #pragma unroll
        for (int u = 0; u < RT_AHEAD; ++u) local[u] = s0 + u < used ? seg_state[(((int64_t) b * segs + s0 + u) * heads + h) * per + e] : 0.f;
        #pragma unroll
        for (int u = 0; u < RT_AHEAD; ++u)
        {
            if (s0 + u >= used) break;
            seg_state[(((int64_t) b * segs + s0 + u) * heads + h) * per + e] = S;
            S = (s0 + u == used - 1 ? dlast : dfull) * S + local[u];
        }
    }
    st[e] = S;
}

// Steps of one row per sequence: rotation, state update, read-out, head norm and gate in one launch, one workgroup per (sequence, head).  A thread owns V
// neighbouring value columns of every (threads / column groups)-th row of the state; partial read-outs meet in LDS.  out = o / rms(o) * silu(gate).
#define RS_THREADS 512
template <typename T, int V>
__global__ __launch_bounds__(RS_THREADS) void retention_step_kernel(T* __restrict__ out, int64_t out_ld, float* __restrict__ state, const T* __restrict__ q, int64_t q_ld,
                                                                    const T* __restrict__ k, int64_t k_ld, const T* __restrict__ v, int64_t v_ld, const T* __restrict__ gate,
                                                                    int64_t gate_ld, const float* __restrict__ pw, int pw_ld, const float* __restrict__ freq, int rot_dims,
                                                                    int interleaved, const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ slots, int heads, int dim,
                                                                    int vdim, float k_scale, float eps)
{
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ float red[RS_THREADS / 64];
    const int cg = (vdim + V - 1) / V;                                // column groups (vdim is a multiple of V)
    const int rp = RS_THREADS / cg;                                   // rows of the state in flight
    float* part = smem;                                               // [rp][vdim]
    float* qs = part + rp * vdim;                                     // [dim]
    float* ks = qs + dim;
    const int n = blockIdx.x, h = blockIdx.y;
    const int pos = tok_pos[n], half = rot_dims >> 1;
    const T* qr = q + (int64_t) n * q_ld + (int64_t) h * dim;
    const T* kr = k + (int64_t) n * k_ld + (int64_t) h * dim;
    for (int i = threadIdx.x; i < half; i += RS_THREADS)
    {
        int a, b;
        rt_pair(i, half, interleaved, a, b);
        float sn, cs;
        sincosf((float) pos * freq[i], &sn, &cs);
        const float qu = to_f(qr[a]), qv = to_f(qr[b]), ku = to_f(kr[a]), kv = to_f(kr[b]);
        qs[a] = qu * cs - qv * sn; qs[b] = qv * cs + qu * sn;
        ks[a] = (ku * cs - kv * sn) * k_scale; ks[b] = (kv * cs + ku * sn) * k_scale;
    }
    for (int i = rot_dims + threadIdx.x; i < dim; i += RS_THREADS) { qs[i] = to_f(qr[i]); ks[i] = to_f(kr[i]) * k_scale; }
    __syncthreads();
    const float lam = pw[(int64_t) h * pw_ld + 1];
    const bool resume = pos > 0;
    const int r0 = threadIdx.x / cg, c0 = (threadIdx.x - r0 * cg) * V;
    float* st = state + ((int64_t) slots[n] * heads + h) * dim * vdim;
    if (r0 < rp)
    {
        const T* vp = v + (int64_t) n * v_ld + (int64_t) h * vdim + c0;
        float vv[V], acc[V];
        #pragma unroll
        for (int e = 0; e < V; ++e) { vv[e] = to_f(vp[e]); acc[e] = 0.f; }
        #pragma unroll 4
        for (int r = r0; r < dim; r += rp)
        {
            float* sp = st + (int64_t) r * vdim + c0;
            float s[V];
            if constexpr (V == 4) { const float4 t = resume ? *(const float4*) sp : make_float4(0.f, 0.f, 0.f, 0.f); s[0] = t.x; s[1] = t.y; s[2] = t.z; s[V - 1] = t.w; }
            else s[0] = resume ? sp[0] : 0.f;
            const float kk = ks[r], qq = qs[r];
            #pragma unroll
            for (int e = 0; e < V; ++e) { s[e] = lam * s[e] + kk * vv[e]; acc[e] += qq * s[e]; }
            if constexpr (V == 4) *(float4*) sp = make_float4(s[0], s[1], s[2], s[V - 1]); else sp[0] = s[0];
        }
        #pragma unroll
        for (int e = 0; e < V; ++e) part[r0 * vdim + c0 + e] = acc[e];
    }
    __syncthreads();
    float ss = 0.f;
    for (int c = threadIdx.x; c < vdim; c += RS_THREADS)
    {
        float s = 0.f;
        for (int r = 0; r < rp; ++r) s += part[r * vdim + c];
        part[c] = s;                                                  // the column's own first row: read by this thread only
        ss += s * s;
    }
    ss = block_sum<RS_THREADS / 64>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float) vdim + eps);
    for (int c = threadIdx.x; c < vdim; c += RS_THREADS)
        out[(int64_t) n * out_ld + (int64_t) h * vdim + c] = from_f<T>(part[c] * inv * silu_f(to_f(gate[(int64_t) n * gate_ld + (int64_t) h * vdim + c])));
}

static int retention_check(const char* what, int heads, int dim, int vdim, int rot_dims, const float* freq, int pw_ld, int need)
{
    MIX_CHECK(heads > 0 && heads <= 65535 && dim > 0 && dim <= 256 && vdim > 0 && vdim <= 1024, "%s: dim %d (<= 256) / vdim %d (<= 1024) out of range", what, dim, vdim);
    MIX_CHECK(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (rot_dims == 0 || freq), "%s: %d rotated entries of %d", what, rot_dims, dim);
    MIX_CHECK(pw_ld >= need, "%s: the table of powers holds %d of %d entries", what, pw_ld, need);
    return EXL3_MIX_OK;
}

template <int MODEV>
static int retention_launch(float* o, float* state, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld, const float* pw, int pw_ld,
                            const float* freq, int rot_dims, int interleaved, const int32_t* cu, const int32_t* slots, const int32_t* pos0, int batch, int heads, int dim, int vdim,
                            float k_scale, int segs, int seg_len, float* seg_state, int dtype, void* stream)
{
    const dim3 grid(batch * segs, heads, (vdim + RT_COLS - 1) / RT_COLS);
    #define RT_LAUNCH(DTV, TTV) hipLaunchKernelGGL((retention_chunk_kernel<T, DTV, TTV, MODEV>), grid, dim3(RT_THREADS), 0, (hipStream_t) stream, o, state, (const T*) q, q_ld, \
                                                   (const T*) k, k_ld, (const T*) v, v_ld, pw, pw_ld, freq, rot_dims, interleaved, cu, slots, pos0, heads, dim, vdim, k_scale, segs, \
                                                   seg_len, seg_state)
    MIX_DISPATCH_T(dtype, if (dim <= 32) RT_LAUNCH(2, 32); else if (dim <= 64) RT_LAUNCH(4, 32); else if (dim <= 128) RT_LAUNCH(8, 32); else RT_LAUNCH(16, 16));
    #undef RT_LAUNCH
    return mix_check_launch("mix_retention");
}

extern "C" int exl3_mix_retention(float* o, float* state, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld, const float* pw, int pw_ld,
                                  const float* freq, int rot_dims, int interleaved, const int32_t* cu, const int32_t* slots, const int32_t* pos0, int batch, int heads, int dim,
                                  int vdim, float k_scale, int segs, int seg_len, float* seg_state, int dtype, void* stream)
{
    MIX_CHECK(o && state && q && k && v && pw && cu && slots && pos0 && batch >= 0, "mix_retention: null pointer");
    if (int rc = retention_check("mix_retention", heads, dim, vdim, rot_dims, freq, pw_ld, 33)) return rc;
    MIX_CHECK(q_ld >= (int64_t) heads * dim && k_ld >= (int64_t) heads * dim && v_ld >= (int64_t) heads * vdim, "mix_retention: bad row strides");
    MIX_CHECK(segs >= 1 && (segs == 1 || (seg_len >= 1 && seg_state)), "mix_retention: bad segment arguments");
    if (batch == 0) return EXL3_MIX_OK;
    #define RT_ARGS o, state, q, q_ld, k, k_ld, v, v_ld, pw, pw_ld, freq, rot_dims, interleaved, cu, slots, pos0, batch, heads, dim, vdim, k_scale, segs, seg_len, seg_state, dtype, stream
    if (segs == 1) return retention_launch<RT_WHOLE>(RT_ARGS);
    int rc = retention_launch<RT_SEG_LOCAL>(RT_ARGS);
    if (rc) return rc;
    const int64_t per = (int64_t) dim * vdim;
    hipLaunchKernelGGL(retention_combine_kernel, dim3(batch, heads, (unsigned) ((per + 255) / 256)), dim3(256), 0, (hipStream_t) stream, state, seg_state, pw, pw_ld, cu, slots, pos0, heads,
                       dim, vdim, segs, seg_len);
    if ((rc = mix_check_launch("mix_retention (combine)"))) return rc;
    return retention_launch<RT_SEG_FINAL>(RT_ARGS);
    #undef RT_ARGS
}

extern "C" int exl3_mix_retention_step(void* out, int64_t out_ld, float* state, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                                       const void* gate, int64_t gate_ld, const float* pw, int pw_ld, const float* freq, int rot_dims, int interleaved, const int32_t* tok_pos,
                                       const int32_t* slots, int n, int heads, int dim, int vdim, float k_scale, float eps, int dtype, void* stream)
{
    MIX_CHECK(out && state && q && k && v && gate && pw && tok_pos && slots && n >= 0, "mix_retention_step: null pointer");
    if (int rc = retention_check("mix_retention_step", heads, dim, vdim, rot_dims, freq, pw_ld, 2)) return rc;
    MIX_CHECK(q_ld >= (int64_t) heads * dim && k_ld >= (int64_t) heads * dim && v_ld >= (int64_t) heads * vdim && gate_ld >= (int64_t) heads * vdim && out_ld >= (int64_t) heads * vdim,
              "mix_retention_step: bad row strides");
    if (n == 0) return EXL3_MIX_OK;
    const bool by4 = vdim % 4 == 0 && (uintptr_t) state % 16 == 0;
    MIX_CHECK(by4 || vdim <= RS_THREADS, "mix_retention_step: vdim %d must be a multiple of 4 or at most %d", vdim, RS_THREADS);
    const int cg = by4 ? vdim / 4 : vdim;
    const size_t sm = ((size_t) (RS_THREADS / cg) * vdim + 2 * dim) * sizeof(float);
    #define RS_LAUNCH(VV) hipLaunchKernelGGL((retention_step_kernel<T, VV>), dim3(n, heads), dim3(RS_THREADS), sm, (hipStream_t) stream, (T*) out, out_ld, state, (const T*) q, q_ld, \
                                             (const T*) k, k_ld, (const T*) v, v_ld, (const T*) gate, gate_ld, pw, pw_ld, freq, rot_dims, interleaved, tok_pos, slots, heads, dim, vdim, \
                                             k_scale, eps)
    MIX_DISPATCH_T(dtype, if (by4) RS_LAUNCH(4); else RS_LAUNCH(1));
    #undef RS_LAUNCH
    return mix_check_launch("mix_retention_step");
}
